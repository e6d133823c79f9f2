// Latent attention: what goes in front of the paged attention launch when keys and values are cached as ONE
// normalised low-rank latent per token plus one rotated key part shared by all heads.
//
// Attention then runs in the latent space as multi-query attention: the key up-projection has been applied to the
// query (q_lat = Uk_h^T q_plain, a matrix product done by the caller), the cached "key" of a token is
// [c | rot(k_r)] (rank + R wide), its "value" is c, and the value up-projection is applied to the attention output.
//
// nv_latent_prep_store, per token t at position p:
//     c        = ckv[t, :rank] / sqrt(mean(ckv[t, :rank]^2) + eps) * latent_w          (fp32, then the cache dtype)
//     k_r      = rot_p(ckv[t, rank:])
//     q_full[t, h] = [q_lat[t, h] | rot_p(q[t, h, Dq - R:])]
//     k_cache[slot(t)] = [c | k_r],   v_cache[slot(t)] = c                             (slot < 0: not stored; v_cache
//                                                                                       absent: values alias the keys)
// rot_p turns pair i by the angle p * freq[i] (fp32 product) with cos and sin both times `mag`; the pair is
// (2i, 2i+1) when `interleaved`, else (i, i + R/2).  The frequencies are a table of the caller's (plain powers of a
// base, or blended for long contexts).
//
// Without a rotated part there is nothing to assemble: nv_latent_store normalises and scatters the latent alone, and the
// latent-space queries go to the attention as the projection leaves them.
//
// nv_head_linear, the two up-projections as one launch each (and any other per-head product of a few dozen to a few
// hundred columns):
//     y[t, h, n] = sum_k x[t, h, k] * w[h, n, k]            optionally times sigmoid(gate[t, h * N + n])
// x may be a slice of a wider row, y is [T, H, N] as the next launch reads it: no transposed copies around a batched
// product.  A workgroup of four waves takes 64 (16) rows x 128 (64) columns of one head; the weight rows are the
// matrix core's first operand, so that a lane ends up with four neighbouring columns of one row and stores them at once.
#include <algorithm>

#include "mfma_tile.h"
#include "row_pieces.h"
#include "../../include/nanovllm_hip_mixers.h"

namespace nv {

template <typename T>
__global__ __launch_bounds__(256) void latent_prep_store_kernel(
    const T* __restrict__ q, int64_t q_stride, int Dq, const T* __restrict__ q_lat, int64_t ql_stride_t,
    int64_t ql_stride_h, const T* __restrict__ ckv, int64_t ckv_stride, const float* __restrict__ latent_w,
    const float* __restrict__ freq, float mag, int interleaved, const int64_t* __restrict__ positions,
    const int* __restrict__ slot_mapping, T* __restrict__ q_full, T* __restrict__ k_cache, T* __restrict__ v_cache,
    int H, int rank, int R, float eps) {
    __shared__ float red[4];
    __shared__ float cs[2 * 512];                  // cos | sin of the token's angles, R / 2 <= 512 each
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, half = R >> 1, Dk = rank + R;
    const float pos = (float)positions[t];
    for (int i = tid; i < half; i += 256) {
        const float ang = pos * freq[i];
        cs[i] = cosf(ang) * mag;
        cs[512 + i] = sinf(ang) * mag;
    }
    const T* crow = ckv + t * ckv_stride;
    float ss = 0.f;
    for (int c = tid; c < rank; c += 256) {
        const float v = (float)crow[c];
        ss += v * v;
    }
    ss = wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();                               // also publishes cs
    const float rstd = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)rank + eps);
    const int64_t slot = slot_mapping != nullptr ? slot_mapping[t] : -1;
    if (slot >= 0) {
        T* krow = k_cache + slot * Dk;
        for (int c = tid; c < rank; c += 256) {
            const T v = (T)((float)crow[c] * rstd * latent_w[c]);
            krow[c] = v;
            if (v_cache != nullptr) v_cache[slot * rank + c] = v;      // (absent when the values alias the key rows)
        }
        for (int i = tid; i < half; i += 256) {
            const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
            const float a = (float)crow[rank + ia], b = (float)crow[rank + ib];
            krow[rank + ia] = (T)(a * cs[i] - b * cs[512 + i]);
            krow[rank + ib] = (T)(b * cs[i] + a * cs[512 + i]);
        }
    }
    for (int h = 0; h < H; ++h) {
        T* qo = q_full + (t * H + h) * Dk;
        const T* ql = q_lat + t * ql_stride_t + h * ql_stride_h;
        for (int c = tid; c < rank; c += 256) qo[c] = ql[c];
        const T* qr = q + t * q_stride + (int64_t)h * Dq + (Dq - R);
        for (int i = tid; i < half; i += 256) {
            const int ia = interleaved ? 2 * i : i, ib = interleaved ? 2 * i + 1 : i + half;
            const float a = (float)qr[ia], b = (float)qr[ib];
            qo[rank + ia] = (T)(a * cs[i] - b * cs[512 + i]);
            qo[rank + ib] = (T)(b * cs[i] + a * cs[512 + i]);
        }
    }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void latent_store_kernel(const T* __restrict__ ckv, int64_t ckv_stride,
                                                           const float* __restrict__ latent_w, const int* __restrict__ slot_mapping,
                                                           T* __restrict__ cache, int64_t num_slots, int64_t tokens, int rank,
                                                           float eps) {
    const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);      // one wave per token
    if (t >= tokens) return;
    const int64_t slot = slot_mapping[t];
    if (slot < 0 || slot >= num_slots) return;
    const int lane = threadIdx.x & 63;
    const T* row = ckv + t * ckv_stride;
    float ss = 0.f;
    for (int c = lane * V; c < rank; c += 64 * V) {
        const Cols<V> a = row_load<V>(row + c);
#pragma unroll
        for (int e = 0; e < V; ++e) ss += a.v[e] * a.v[e];
    }
    const float rstd = 1.0f / sqrtf(wave_sum(ss) / (float)rank + eps);
    for (int c = lane * V; c < rank; c += 64 * V) {
        const Cols<V> a = row_load<V>(row + c), w = row_load<V>(latent_w + c);
        Cols<V> o;
#pragma unroll
        for (int e = 0; e < V; ++e) o.v[e] = a.v[e] * rstd * w.v[e];
        row_store<V>(cache + slot * rank + c, o);
    }
}

template <typename T, int MT, int NT>
__global__ __launch_bounds__(256) void head_linear_kernel(const T* __restrict__ x, int64_t x_stride, const T* __restrict__ w,
                                                          const T* __restrict__ gate, int64_t gate_stride, T* __restrict__ y,
                                                          int64_t rows_all, int H, int N, int K, int row_tiles, int col_tiles,
                                                          int vec_ok, int out_vec) {
    using M = TileMma<T>;
    constexpr int BK = M::kBK, BM = 16 * MT, BN = 64 * NT, LD = BK + M::kPad, KV = BK / M::kVec;
    constexpr int X_IT = (BM * KV + 255) / 256, W_IT = (BN * KV + 255) / 256;
    __shared__ __attribute__((aligned(16))) T Xs[BM * LD];
    __shared__ __attribute__((aligned(16))) T Ws[BN * LD];
    // workgroups go to the 8 XCDs in turn: give each a consecutive range of items, which share a head's weights
    const int per_xcd = gridDim.x / 8;
    int item = blockIdx.x;
    if (item < per_xcd * 8) item = (item % 8) * per_xcd + item / 8;
    const int rt = item % row_tiles, ct = (item / row_tiles) % col_tiles, h = item / (row_tiles * col_tiles);
    const int64_t t0 = (int64_t)rt * BM;
    const int n0 = ct * BN, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lq = lane & 15, lg = lane >> 4;
    const T* x_row[X_IT];
    const T* w_row[W_IT];
#pragma unroll
    for (int i = 0; i < X_IT; ++i) {
        const int it = tid + 256 * i, r = it / KV;
        x_row[i] = (it < BM * KV && t0 + r < rows_all) ? x + (t0 + r) * x_stride + (int64_t)h * K : nullptr;
    }
#pragma unroll
    for (int i = 0; i < W_IT; ++i) {
        const int it = tid + 256 * i, n = n0 + it / KV;
        w_row[i] = (it < BN * KV && n < N) ? w + ((int64_t)h * N + n) * K : nullptr;
    }
    uint4 x_reg[X_IT], w_reg[W_IT];
    auto fetch = [&](int k0) {
#pragma unroll
        for (int i = 0; i < X_IT; ++i) x_reg[i] = tile_fetch<T>(x_row[i], k0 + ((tid + 256 * i) % KV) * M::kVec, K, vec_ok != 0);
#pragma unroll
        for (int i = 0; i < W_IT; ++i) w_reg[i] = tile_fetch<T>(w_row[i], k0 + ((tid + 256 * i) % KV) * M::kVec, K, vec_ok != 0);
    };
    f32x4 acc[NT][MT];
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int m = 0; m < MT; ++m) acc[n][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    fetch(0);
    for (int k0 = 0; k0 < K; k0 += BK) {
        __syncthreads();                               // the previous slices have been consumed
#pragma unroll
        for (int i = 0; i < X_IT; ++i) {
            const int it = tid + 256 * i;
            if (it < BM * KV) *(uint4*)(Xs + (it / KV) * LD + (it % KV) * M::kVec) = x_reg[i];
        }
#pragma unroll
        for (int i = 0; i < W_IT; ++i) {
            const int it = tid + 256 * i;
            if (it < BN * KV) *(uint4*)(Ws + (it / KV) * LD + (it % KV) * M::kVec) = w_reg[i];
        }
        __syncthreads();
        if (k0 + BK < K) fetch(k0 + BK);
#pragma unroll
        for (int kk = 0; kk < BK; kk += M::kStep) {
#pragma unroll
            for (int n = 0; n < NT; ++n) {
                const T* wrow = Ws + ((wave * NT + n) * 16 + lq) * LD + kk;
#pragma unroll
                for (int m = 0; m < MT; ++m) acc[n][m] = M::run(wrow, Xs + (m * 16 + lq) * LD + kk, lg, acc[n][m]);
            }
        }
    }
    const int64_t ld = (int64_t)H * N;
#pragma unroll
    for (int m = 0; m < MT; ++m) {
        const int64_t t = t0 + m * 16 + lq;
        if (t >= rows_all) continue;
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
            const int n = n0 + (wave * NT + nt) * 16 + 4 * lg;          // this lane's four columns
            const int64_t col = (int64_t)h * N + n;
            if (out_vec) {                                               // (N is a multiple of 4: all four or none)
                if (n >= N) continue;
                Cols<4> o;
#pragma unroll
                for (int e = 0; e < 4; ++e) o.v[e] = acc[nt][m][e];
                if (gate != nullptr) {
                    const Cols<4> g = row_load<4>(gate + t * gate_stride + col);
#pragma unroll
                    for (int e = 0; e < 4; ++e) o.v[e] /= 1.0f + expf(-g.v[e]);
                }
                row_store<4>(y + t * ld + col, o);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    if (n + e >= N) continue;
                    float o = acc[nt][m][e];
                    if (gate != nullptr) o /= 1.0f + expf(-(float)gate[t * gate_stride + col + e]);
                    y[t * ld + col + e] = (T)o;
                }
            }
        }
    }
}

template <typename T>
static void launch_head_linear(const void* x, int64_t x_stride, const void* w, const void* gate, int64_t gate_stride, void* y,
                               int64_t rows, int H, int N, int K, bool big, hipStream_t s) {
    const int vec = TileMma<T>::kVec, esz = (int)sizeof(T);
    const int vec_ok = K % vec == 0 && x_stride % vec == 0 && ((uintptr_t)x | (uintptr_t)w) % 16 == 0;
    const int out_vec = N % 4 == 0 && gate_stride % 4 == 0 && ((uintptr_t)y | (uintptr_t)gate) % (4 * esz) == 0;
    const int bm = big ? 64 : 16, bn = big && esz == 2 ? 128 : 64;
    const int rt = (int)((rows + bm - 1) / bm), ct = (N + bn - 1) / bn;
#define NV_HEADS(MT, NT)                                                                                                \
    hipLaunchKernelGGL((head_linear_kernel<T, MT, NT>), dim3((unsigned)((int64_t)rt * ct * H)), dim3(256), 0, s, (const T*)x, \
                       x_stride, (const T*)w, (const T*)gate, gate_stride, (T*)y, rows, H, N, K, rt, ct, vec_ok, out_vec)
    if (big && esz == 2) NV_HEADS(4, 2);
    else if (big) NV_HEADS(4, 1);
    else NV_HEADS(1, 1);
#undef NV_HEADS
}

}  // namespace nv

extern "C" int nv_latent_prep_store(const void* q, int64_t q_stride, int Dq, const void* q_lat, int64_t ql_stride_t,
                                    int64_t ql_stride_h, const void* ckv, int64_t ckv_stride, const float* latent_w,
                                    const float* freq, float mag, int interleaved, const int64_t* positions,
                                    const int32_t* slot_mapping, void* q_full, void* k_cache, void* v_cache, int dtype,
                                    int64_t T, int H, int rank, int R, float eps, void* stream) {
    using namespace nv;
    NV_REQUIRE(T >= 0 && H > 0 && rank > 0 && R >= 0 && Dq >= R, NV_ERR_INVALID_ARG, "nv_latent_prep_store: bad sizes");
    if (T == 0) return NV_OK;
    NV_REQUIRE(q && q_lat && ckv && latent_w && positions && q_full, NV_ERR_INVALID_ARG,
               "nv_latent_prep_store: null pointer");
    NV_REQUIRE(!slot_mapping || k_cache, NV_ERR_INVALID_ARG, "nv_latent_prep_store: scatter needs the key cache");
    NV_REQUIRE(R % 2 == 0 && R <= 1024 && (R == 0 || freq), NV_ERR_INVALID_ARG,
               "nv_latent_prep_store: the rotated part (%d) must be even, at most 1024, with its frequencies", R);
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_latent_prep_store: bad dtype");
    NV_REQUIRE(T < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_latent_prep_store: launch too large");
    hipStream_t s = (hipStream_t)stream;
    if (dtype == NV_DTYPE_BF16)
        hipLaunchKernelGGL(latent_prep_store_kernel<__bf16>, dim3((unsigned)T), dim3(256), 0, s, (const __bf16*)q, q_stride,
                           Dq, (const __bf16*)q_lat, ql_stride_t, ql_stride_h, (const __bf16*)ckv, ckv_stride, latent_w,
                           freq, mag, interleaved, positions, slot_mapping, (__bf16*)q_full, (__bf16*)k_cache,
                           (__bf16*)v_cache, H, rank, R, eps);
    else
        hipLaunchKernelGGL(latent_prep_store_kernel<float>, dim3((unsigned)T), dim3(256), 0, s, (const float*)q, q_stride,
                           Dq, (const float*)q_lat, ql_stride_t, ql_stride_h, (const float*)ckv, ckv_stride, latent_w,
                           freq, mag, interleaved, positions, slot_mapping, (float*)q_full, (float*)k_cache,
                           (float*)v_cache, H, rank, R, eps);
    return check_launch("nv_latent_prep_store");
}

extern "C" int nv_latent_store(const void* ckv, int64_t ckv_stride, const float* latent_w, const int32_t* slot_mapping,
                               void* cache, int64_t num_slots, int dtype, int64_t T, int rank, float eps, void* stream) {
    using namespace nv;
    NV_REQUIRE(T >= 0 && rank > 0 && num_slots > 0 && ckv_stride >= rank, NV_ERR_INVALID_ARG, "nv_latent_store: bad sizes");
    if (T == 0) return NV_OK;
    NV_REQUIRE(ckv && latent_w && slot_mapping && cache, NV_ERR_INVALID_ARG, "nv_latent_store: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_latent_store: bad dtype");
    const int64_t grid = (T + 3) / 4;
    NV_REQUIRE(grid < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_latent_store: launch too large");
    const bool bf = dtype == NV_DTYPE_BF16;
    const bool vec = rank % 4 == 0 && ckv_stride % 4 == 0 && ((uintptr_t)ckv | (uintptr_t)cache) % (bf ? 8 : 16) == 0 &&
                     (uintptr_t)latent_w % 16 == 0;
#define NV_STORE(TT, V)                                                                                                    \
    hipLaunchKernelGGL((latent_store_kernel<TT, V>), dim3((unsigned)grid), dim3(256), 0, (hipStream_t)stream, (const TT*)ckv, \
                       ckv_stride, latent_w, slot_mapping, (TT*)cache, num_slots, T, rank, eps)
    if (bf && vec) NV_STORE(__bf16, 4);
    else if (bf) NV_STORE(__bf16, 1);
    else if (vec) NV_STORE(float, 4);
    else NV_STORE(float, 1);
#undef NV_STORE
    return check_launch("nv_latent_store");
}

extern "C" int nv_head_linear(const void* x, int64_t x_stride, const void* w, const void* gate, int64_t gate_stride, void* y,
                              int dtype, int64_t T, int H, int N, int K, void* stream) {
    using namespace nv;
    NV_REQUIRE(T >= 0 && H > 0 && N > 0 && K > 0 && x_stride >= (int64_t)H * K, NV_ERR_INVALID_ARG, "nv_head_linear: bad sizes");
    NV_REQUIRE(!gate || gate_stride >= (int64_t)H * N, NV_ERR_INVALID_ARG, "nv_head_linear: bad gate stride");
    if (T == 0) return NV_OK;
    NV_REQUIRE(x && w && y, NV_ERR_INVALID_ARG, "nv_head_linear: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_head_linear: bad dtype");
    // large tiles once they still give every CU two workgroups
    const bool big = ((T + 63) / 64) * ((N + 127) / 128) * H >= 512;
    NV_REQUIRE(((T + 15) / 16) * ((N + 63) / 64) * H < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_head_linear: launch too large");
    if (!gate) gate_stride = 0;
    if (dtype == NV_DTYPE_BF16) launch_head_linear<__bf16>(x, x_stride, w, gate, gate_stride, y, T, H, N, K, big, (hipStream_t)stream);
    else launch_head_linear<float>(x, x_stride, w, gate, gate_stride, y, T, H, N, K, big, (hipStream_t)stream);
    return check_launch("nv_head_linear");
}
