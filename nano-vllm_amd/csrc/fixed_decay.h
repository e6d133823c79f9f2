// The linear memory with one constant decay per head: what its two launches share.
//   S <- decay_h S + silu(k) silu(v)^T;   o = S^T silu(q)        (the write comes first; o in fp32)
#pragma once
#include "nv_common.h"

namespace nv {

struct FixedDecayArgs {
    const void *q, *k, *v;                     // q, k: [T, H * Dk]; v: [T, H * Dv], as projected, with row strides
    int64_t q_stride, k_stride, v_stride;
    const float* decay;                        // [H]
    float* state;                              // [slots, H, Dk, Dv]
    float* out;                                // [T, H * Dv]
    int64_t out_stride;
    const int *cu_q, *cu_k, *slots;
    int num_seqs, H, Dk, Dv;
};

// Token by token with the state in registers, every sequence with at most max_rows rows in the step; any sizes up to 256 x 256.
int launch_fixed_decay_rows(const FixedDecayArgs& f, int dtype, int max_rows, hipStream_t s);

}  // namespace nv
