// V neighbouring columns of a row in registers as fp32: one 16-byte (fp32) or 8-byte (bf16) access for V = 4, one element
// for V = 1.
#pragma once
#include "nv_common.h"

namespace nv {

template <int V> struct Cols { float v[V]; };

template <int V>
__device__ __forceinline__ Cols<V> row_load(const float* p) {
    Cols<V> o;
    if constexpr (V == 4) {
        const float4 u = *(const float4*)p;
        o.v[0] = u.x; o.v[1] = u.y; o.v[2] = u.z; o.v[3] = u.w;
    } else {
        o.v[0] = p[0];
    }
    return o;
}
template <int V>
__device__ __forceinline__ Cols<V> row_load(const __bf16* p) {
    Cols<V> o;
    if constexpr (V == 4) {
        const uint2 u = *(const uint2*)p;
        o.v[0] = bf16_lo(u.x); o.v[1] = bf16_hi(u.x); o.v[2] = bf16_lo(u.y); o.v[3] = bf16_hi(u.y);
    } else {
        o.v[0] = (float)p[0];
    }
    return o;
}
template <int V>
__device__ __forceinline__ void row_store(float* p, const Cols<V>& c) {
    if constexpr (V == 4) *(float4*)p = make_float4(c.v[0], c.v[1], c.v[2], c.v[3]);
    else p[0] = c.v[0];
}
template <int V>
__device__ __forceinline__ void row_store(__bf16* p, const Cols<V>& c) {
    if constexpr (V == 4) *(uint2*)p = make_uint2(pack_bf16(c.v[0], c.v[1]), pack_bf16(c.v[2], c.v[3]));
    else p[0] = (__bf16)c.v[0];
}

}  // namespace nv
