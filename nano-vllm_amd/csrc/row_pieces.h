// V neighbouring columns of a row in registers as fp32: one 16-byte (fp32) or 8-byte (bf16) access for V = 4, one element
// for V = 1, V = 8 as two accesses (fp32) or one of 16 bytes (bf16).
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
    } else if constexpr (V == 8) {
        const float4 u = *(const float4*)p, w = *(const float4*)(p + 4);
        o.v[0] = u.x; o.v[1] = u.y; o.v[2] = u.z; o.v[3] = u.w;
        o.v[4] = w.x; o.v[5] = w.y; o.v[6] = w.z; o.v[7] = w.w;
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
    } else if constexpr (V == 8) {
        const uint4 u = *(const uint4*)p;
        o.v[0] = bf16_lo(u.x); o.v[1] = bf16_hi(u.x); o.v[2] = bf16_lo(u.y); o.v[3] = bf16_hi(u.y);
        o.v[4] = bf16_lo(u.z); o.v[5] = bf16_hi(u.z); o.v[6] = bf16_lo(u.w); o.v[7] = bf16_hi(u.w);
    } else {
        o.v[0] = (float)p[0];
    }
    return o;
}
template <int V>
__device__ __forceinline__ void row_store(float* p, const Cols<V>& c) {
    if constexpr (V == 4) {
        *(float4*)p = make_float4(c.v[0], c.v[1], c.v[2], c.v[3]);
    } else if constexpr (V == 8) {
        *(float4*)p = make_float4(c.v[0], c.v[1], c.v[2], c.v[3]);
        *(float4*)(p + 4) = make_float4(c.v[4], c.v[5], c.v[6], c.v[7]);
    } else p[0] = c.v[0];
}
template <int V>
__device__ __forceinline__ void row_store(__bf16* p, const Cols<V>& c) {
    if constexpr (V == 4)
        *(uint2*)p = make_uint2(pack_bf16(c.v[0], c.v[1]), pack_bf16(c.v[2], c.v[3]));
    else if constexpr (V == 8)
        *(uint4*)p = make_uint4(pack_bf16(c.v[0], c.v[1]), pack_bf16(c.v[2], c.v[3]), pack_bf16(c.v[4], c.v[5]), pack_bf16(c.v[6], c.v[7]));
    else p[0] = (__bf16)c.v[0];
}

}  // namespace nv
