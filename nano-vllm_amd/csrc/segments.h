// Recurrences over long portions, cut into segments along time that run side by side: where a sequence's segments keep what
// they hand on.  A first launch runs every segment but a sequence's last from a zero state and leaves its end state; the last
// one's place takes the sequence's start state (the second launch overwrites the slot); in the second launch a segment folds what
// is in front of it into its start state and runs as usual.  Only sequences with more than one segment have places: theirs are
// numbered through in the order of the batch, so that single rows beside long portions cost nothing.
#pragma once
#include "nv_common.h"

namespace nv {

// Segments of a sequence with len rows in the step.
__host__ __device__ __forceinline__ int segment_count(int len, int seg_len, int nseg) {
    const int n = (len + seg_len - 1) / seg_len;
    return n < nseg ? n : nseg;
}

// Places needed by a step of T rows: a sequence with several segments has at most twice as many as it has whole ones.
inline int64_t segment_places(int64_t T, int seg_len) { return 2 * T / seg_len + 1; }

// First place of sequence b; to be called by all 256 threads of a workgroup.
__device__ __forceinline__ int segment_first_place(const int* cu_q, int b, int seg_len, int nseg) {
    __shared__ int red[4];
    int n = 0;
    for (int i = threadIdx.x; i < b; i += 256) {
        const int len = cu_q[i + 1] - cu_q[i];
        if (len > seg_len) n += segment_count(len, seg_len, nseg);
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) n += __shfl_xor(n, o);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = n;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

}  // namespace nv
