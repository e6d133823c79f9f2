// What the tiled matrix-product kernels share: the MFMA of an element type on 16 x 16 tiles whose operands both hold the
// contraction index contiguously in LDS, and the 16-byte fetch of a row piece with zeros beyond the row's end.
#pragma once
#include "nv_common.h"

namespace nv {

template <typename T> struct TileMma;
template <> struct TileMma<__bf16> {
    static constexpr int kVec = 8, kPad = 8, kStep = 32, kBK = 64;
    // the 32-deep product of gfx950: a lane holds 8 consecutive k of its row (16-byte LDS reads)
    static __device__ __forceinline__ f32x4 run(const __bf16* a, const __bf16* b, int lg, f32x4 c) {
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(a + 8 * lg), *(const bf16x8*)(b + 8 * lg), c, 0, 0, 0);
    }
};
template <> struct TileMma<float> {
    static constexpr int kVec = 4, kPad = 4, kStep = 4, kBK = 32;
    static __device__ __forceinline__ f32x4 run(const float* a, const float* b, int lg, f32x4 c) {
        return __builtin_amdgcn_mfma_f32_16x16x4f32(a[lg], b[lg], c, 0, 0, 0);
    }
};

// 16 bytes (kVec elements) of a row starting at k0, zeros past K or for a missing row
template <typename T>
__device__ __forceinline__ uint4 tile_fetch(const T* row, int k0, int K, bool vec_ok) {
    constexpr int V = TileMma<T>::kVec;
    if (row == nullptr || k0 >= K) return make_uint4(0, 0, 0, 0);
    if (vec_ok && k0 + V <= K) return *(const uint4*)(row + k0);
    __attribute__((aligned(16))) T tmp[V];
#pragma unroll
    for (int i = 0; i < V; ++i) tmp[i] = k0 + i < K ? row[k0 + i] : (T)0.f;
    return *(const uint4*)tmp;
}

}  // namespace nv
