// What stands around two mixers that run side by side on one input, and around a stream that is read un-normed.
//
// nv_row_norm_rope_store   in front of nv_attn_scoremod_paged when queries and keys are RMS-normed over the WHOLE projection
//                          (all heads at once, one weight per column): norm, rotate-half rotary on the first rot_dims
//                          dimensions of every head (pair (i, i + rot_dims/2), angle = position * freq[i] as an fp32 product,
//                          full-precision sincosf, cos and sin times `magnitude`), the prepared queries written, keys and
//                          values scattered into the paged cache.
// nv_join_gated            the two mixers' outputs on their way into ONE output product:
//                              y[:, :H Dv]  = left_scale  * sigmoid(head_gate[h]) * attn[h]
//                              y[:, H Dv:]  = right_scale * sigmoid(gate) * mem / sqrt(mean(mem^2) + eps) * norm_w
//                          (attn in the matmul dtype, mem fp32, the mean over the whole row of mem).
// nv_clamped_glu_rows      y = g sigmoid(alpha g) (u + shift) for rows [gate | up], g = min(gate, limit), u = clamp(up, +-limit).
// nv_scale_softcap         y = cap tanh(scale x / cap) in fp32 (cap = 0: scale x).
#include "row_pieces.h"
#include "../../include/nanovllm_hip_mixers.h"

namespace nv {

constexpr int kPmThreads = 256;
constexpr int kPmMaxLdsCols = 15 * 1024;        // columns of q and k together that are kept in LDS

__device__ __forceinline__ float pm_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// Two sums over the workgroup through one exchange.
__device__ __forceinline__ void pm_block_sum2(float& a, float& b, float (*red)[kPmThreads / 64]) {
    a = wave_sum(a);
    b = wave_sum(b);
    if ((threadIdx.x & 63) == 0) {
        red[0][threadIdx.x >> 6] = a;
        red[1][threadIdx.x >> 6] = b;
    }
    __syncthreads();
    a = (red[0][0] + red[0][1]) + (red[0][2] + red[0][3]);
    b = (red[1][0] + red[1][1]) + (red[1][2] + red[1][3]);
}

struct PrepArgs {
    const void *q, *k, *v;
    int64_t q_stride, k_stride, v_stride;
    const float *q_norm, *k_norm, *freq;
    float eps, magnitude;
    int rot_dims;
    const int64_t* positions;
    const int* slots;
    void *q_out, *k_cache, *v_cache;
    int H, G, D, Dv;
};

// A workgroup per token.  KEEP: the weighted row [q | k] stays in LDS between its two uses (the partner of a rotated
// dimension belongs to another thread); otherwise it is read again.  V columns at a time.
template <typename T, int V, bool KEEP>
__global__ __launch_bounds__(kPmThreads) void row_norm_rope_store_kernel(const PrepArgs a) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    __shared__ float red[2][kPmThreads / 64];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, H = a.H, G = a.G, D = a.D, Dv = a.Dv, nq = H * D, nk = G * D, half = a.rot_dims / 2;
    float* cs = smem;                                            // [half] cos, [half] sin
    float* row = smem + ((2 * half + 3) & ~3);                   // [nq + nk]
    const T* qr = (const T*)a.q + t * a.q_stride;
    const T* kr = (const T*)a.k + t * a.k_stride;
    const int slot = a.slots != nullptr ? a.slots[t] : -1;
    const float pos = (float)a.positions[t];
    for (int i = tid; i < half; i += kPmThreads) {
        float sn, c;
        sincosf(pos * a.freq[i], &sn, &c);
        cs[i] = c * a.magnitude;
        cs[half + i] = sn * a.magnitude;
    }
    float sq = 0.f, sk = 0.f;
    for (int c = tid * V; c < nq + nk; c += kPmThreads * V) {
        const bool is_q = c < nq;
        const Cols<V> x = is_q ? row_load<V>(qr + c) : row_load<V>(kr + (c - nq));
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < V; ++e) ss += x.v[e] * x.v[e];
        if (is_q) sq += ss;
        else sk += ss;
        if constexpr (KEEP) {
            const Cols<V> w = is_q ? row_load<V>(a.q_norm + c) : row_load<V>(a.k_norm + (c - nq));
            Cols<V> y;
#pragma unroll
            for (int e = 0; e < V; ++e) y.v[e] = x.v[e] * w.v[e];
            row_store<V>(row + c, y);
        }
    }
    pm_block_sum2(sq, sk, red);                                  // (its barrier also covers cs and row)
    const float rq = 1.0f / sqrtf(sq / (float)nq + a.eps), rk = 1.0f / sqrtf(sk / (float)nk + a.eps);
    auto weighted = [&](int c) {
        if constexpr (KEEP) return row_load<V>(row + c);
        const bool is_q = c < nq;
        Cols<V> x = is_q ? row_load<V>(qr + c) : row_load<V>(kr + (c - nq));
        const Cols<V> w = is_q ? row_load<V>(a.q_norm + c) : row_load<V>(a.k_norm + (c - nq));
#pragma unroll
        for (int e = 0; e < V; ++e) x.v[e] *= w.v[e];
        return x;
    };
    for (int c = tid * V; c < nq + nk; c += kPmThreads * V) {
        const bool is_q = c < nq;
        if (!is_q && slot < 0) continue;
        const float rs = is_q ? rq : rk;
        const int d = (is_q ? c : c - nq) % D;                   // (V divides the head size and half of its rotated part)
        Cols<V> x = weighted(c);
        if (d < 2 * half) {
            const bool low = d < half;
            const int i = low ? d : d - half;
            const Cols<V> y = weighted(low ? c + half : c - half);
            const Cols<V> cc = row_load<V>(cs + i), sn = row_load<V>(cs + half + i);
#pragma unroll
            for (int e = 0; e < V; ++e) x.v[e] = low ? x.v[e] * cc.v[e] - y.v[e] * sn.v[e] : x.v[e] * cc.v[e] + y.v[e] * sn.v[e];
        }
#pragma unroll
        for (int e = 0; e < V; ++e) x.v[e] *= rs;
        row_store<V>(is_q ? (T*)a.q_out + t * nq + c : (T*)a.k_cache + (int64_t)slot * nk + (c - nq), x);
    }
    if (slot >= 0) {
        const T* vr = (const T*)a.v + t * a.v_stride;
        T* dst = (T*)a.v_cache + (int64_t)slot * G * Dv;
        for (int c = tid * V; c < G * Dv; c += kPmThreads * V) row_store<V>(dst + c, row_load<V>(vr + c));
    }
}

struct JoinArgs {
    const void* attn;
    int64_t attn_stride;
    const void* head_gate;
    int64_t head_gate_stride;
    int H, Dv;
    float left_scale;
    const float* mem;
    int64_t mem_stride;
    const float* norm_w;
    const void* gate;
    int64_t gate_stride;
    int cols;                                  // of mem
    float eps, right_scale;
    void* y;                                   // [T, H Dv + cols]
};

template <typename T, int V, int NI>
__global__ __launch_bounds__(kPmThreads) void join_gated_kernel(const JoinArgs a) {
    __shared__ float red[2][kPmThreads / 64];
    const int64_t t = blockIdx.x;
    const int tid = threadIdx.x, nl = a.H * a.Dv;
    const float* mr = a.mem + t * a.mem_stride;
    const T* gr = (const T*)a.gate + t * a.gate_stride;
    T* yr = (T*)a.y + t * (int64_t)(nl + a.cols);
    Cols<V> m[NI], gt[NI];
    float ss = 0.f, none = 0.f;
#pragma unroll
    for (int k = 0; k < NI; ++k) {
        const int c = (tid + k * kPmThreads) * V;
        if (c < a.cols) {
            m[k] = row_load<V>(mr + c);
            gt[k] = row_load<V>(gr + c);
#pragma unroll
            for (int e = 0; e < V; ++e) ss += m[k].v[e] * m[k].v[e];
        }
    }
    const T* ar = (const T*)a.attn + t * a.attn_stride;
    const T* hg = (const T*)a.head_gate + t * a.head_gate_stride;
    for (int c = tid * V; c < nl; c += kPmThreads * V) {         // (V divides the value size: one head per piece)
        Cols<V> x = row_load<V>(ar + c);
        const float s = a.left_scale * pm_sigmoid((float)hg[c / a.Dv]);
#pragma unroll
        for (int e = 0; e < V; ++e) x.v[e] *= s;
        row_store<V>(yr + c, x);
    }
    pm_block_sum2(ss, none, red);
    const float rs = a.right_scale / sqrtf(ss / (float)a.cols + a.eps);
#pragma unroll
    for (int k = 0; k < NI; ++k) {
        const int c = (tid + k * kPmThreads) * V;
        if (c < a.cols) {
            const Cols<V> w = row_load<V>(a.norm_w + c);
#pragma unroll
            for (int e = 0; e < V; ++e) m[k].v[e] *= rs * w.v[e] * pm_sigmoid(gt[k].v[e]);
            row_store<V>(yr + nl + c, m[k]);
        }
    }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void clamped_glu_rows_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ y,
                                                               int inter, int pieces, int64_t n, float limit, float alpha,
                                                               float shift) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int64_t r = i / pieces;
    const int c = (int)(i - r * pieces) * V;
    const Cols<V> g = row_load<V>(x + r * x_stride + c), u = row_load<V>(x + r * x_stride + inter + c);
    Cols<V> o;
#pragma unroll
    for (int e = 0; e < V; ++e) {
        const float gg = fminf(g.v[e], limit), uu = fminf(fmaxf(u.v[e], -limit), limit);
        if constexpr (sizeof(T) == 2)      // (the result is rounded to bf16: the hardware's exponential and reciprocal are enough)
            o.v[e] = gg * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * alpha * gg)) * (uu + shift);
        else
            o.v[e] = gg / (1.0f + expf(-alpha * gg)) * (uu + shift);
    }
    row_store<V>(y + r * inter + c, o);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void scale_softcap_kernel(const T* __restrict__ x, float* __restrict__ y, int64_t n, float scale,
                                                            float cap) {
    const int64_t i = ((int64_t)blockIdx.x * 256 + threadIdx.x) * V;
    if (i >= n) return;
    Cols<V> v = row_load<V>(x + i);
#pragma unroll
    for (int e = 0; e < V; ++e) {
        v.v[e] *= scale;
        if (cap > 0.f) v.v[e] = cap * tanhf(v.v[e] / cap);
    }
    row_store<V>(y + i, v);
}

template <typename T>
static bool launch_join(const JoinArgs& a, bool vec, int64_t rows, hipStream_t s) {
    const int V = vec ? 4 : 1, per = (a.cols + kPmThreads * V - 1) / (kPmThreads * V);
#define NV_JOIN(VV, N)                                                                                              \
    if (V == VV && per <= N) {                                                                                        \
        hipLaunchKernelGGL((join_gated_kernel<T, VV, N>), dim3((unsigned)rows), dim3(kPmThreads), 0, s, a);           \
        return true;                                                                                                  \
    }
    NV_JOIN(4, 1) NV_JOIN(4, 2) NV_JOIN(4, 4) NV_JOIN(4, 8) NV_JOIN(4, 16)
    NV_JOIN(1, 1) NV_JOIN(1, 4) NV_JOIN(1, 16) NV_JOIN(1, 64)
#undef NV_JOIN
    return false;
}

}  // namespace nv

extern "C" int nv_row_norm_rope_store(const void* q, const void* k, const void* v, int64_t q_stride, int64_t k_stride,
                                      int64_t v_stride, const float* q_norm, const float* k_norm, float eps, const float* freq,
                                      int rot_dims, float magnitude, const int64_t* positions, const int32_t* slot_mapping,
                                      void* q_out, void* k_cache, void* v_cache, int dtype, int64_t T, int H, int G, int D,
                                      int Dv, void* stream) {
    using namespace nv;
    NV_REQUIRE(T >= 0 && H > 0 && G > 0 && D > 0 && Dv > 0, NV_ERR_INVALID_ARG, "nv_row_norm_rope_store: bad sizes");
    NV_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= D && (rot_dims == 0 || freq), NV_ERR_INVALID_ARG,
               "nv_row_norm_rope_store: rot_dims=%d must be even, at most D=%d, with a frequency table", rot_dims, D);
    if (T == 0) return NV_OK;
    NV_REQUIRE(q && k && v && q_norm && k_norm && positions && q_out, NV_ERR_INVALID_ARG, "nv_row_norm_rope_store: null pointer");
    NV_REQUIRE(!slot_mapping || (k_cache && v_cache), NV_ERR_INVALID_ARG, "nv_row_norm_rope_store: scatter needs the caches");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_row_norm_rope_store: bad dtype");
    NV_REQUIRE(T < (1LL << 31) && (int64_t)(H + G) * D < (1 << 30) && (int64_t)G * Dv < (1 << 30) && rot_dims <= 1024,
               NV_ERR_UNSUPPORTED, "nv_row_norm_rope_store: launch too large");
    hipStream_t s = (hipStream_t)stream;
    const bool bf = dtype == NV_DTYPE_BF16;
    const PrepArgs a{q,        k,         v,            q_stride, k_stride, v_stride, q_norm, k_norm, freq, eps, magnitude,
                     rot_dims, positions, slot_mapping, q_out,    k_cache,  v_cache,  H,      G,      D,    Dv};
    const bool vec = D % 4 == 0 && Dv % 4 == 0 && rot_dims % 8 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && v_stride % 4 == 0 &&
                     ((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)v_cache) %
                             (bf ? 8 : 16) == 0 &&
                     ((uintptr_t)q_norm | (uintptr_t)k_norm) % 16 == 0;
    const bool keep = (H + G) * D <= kPmMaxLdsCols - 1024;
    const size_t lds = sizeof(float) * (((size_t)rot_dims + 3 & ~(size_t)3) + (keep ? (size_t)(H + G) * D : 0));
#define NV_PREP(T_, V, K) hipLaunchKernelGGL((row_norm_rope_store_kernel<T_, V, K>), dim3((unsigned)T), dim3(kPmThreads), lds, s, a)
#define NV_PREP_T(T_)              \
    if (vec && keep) NV_PREP(T_, 4, true); \
    else if (vec) NV_PREP(T_, 4, false);   \
    else if (keep) NV_PREP(T_, 1, true);   \
    else NV_PREP(T_, 1, false)
    if (bf) { NV_PREP_T(__bf16); } else { NV_PREP_T(float); }
#undef NV_PREP_T
#undef NV_PREP
    return check_launch("nv_row_norm_rope_store");
}

extern "C" int nv_join_gated(const void* attn, int64_t attn_stride, const void* head_gate, int64_t head_gate_stride, int H, int Dv,
                             float left_scale, const float* mem, int64_t mem_stride, const float* norm_w, const void* gate,
                             int64_t gate_stride, int cols, float eps, float right_scale, void* y, int dtype, int64_t rows,
                             void* stream) {
    using namespace nv;
    NV_REQUIRE(rows >= 0 && H > 0 && Dv > 0 && cols > 0 && cols <= 16384, NV_ERR_INVALID_ARG, "nv_join_gated: bad sizes");
    if (rows == 0) return NV_OK;
    NV_REQUIRE(attn && head_gate && mem && norm_w && gate && y, NV_ERR_INVALID_ARG, "nv_join_gated: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_join_gated: bad dtype");
    NV_REQUIRE(rows < (1LL << 31) && (int64_t)H * Dv < (1 << 30), NV_ERR_UNSUPPORTED, "nv_join_gated: launch too large");
    hipStream_t s = (hipStream_t)stream;
    const bool bf = dtype == NV_DTYPE_BF16;
    const JoinArgs a{attn,   attn_stride, head_gate, head_gate_stride, H,    Dv,          left_scale, mem, mem_stride,
                     norm_w, gate,        gate_stride, cols,           eps,  right_scale, y};
    const bool vec = Dv % 4 == 0 && cols % 4 == 0 && attn_stride % 4 == 0 && mem_stride % 4 == 0 && gate_stride % 4 == 0 &&
                     ((uintptr_t)attn | (uintptr_t)gate | (uintptr_t)y) % (bf ? 8 : 16) == 0 &&
                     ((uintptr_t)mem | (uintptr_t)norm_w) % 16 == 0;
    NV_REQUIRE(bf ? launch_join<__bf16>(a, vec, rows, s) : launch_join<float>(a, vec, rows, s), NV_ERR_UNSUPPORTED,
               "nv_join_gated: no kernel for %d columns", cols);
    return check_launch("nv_join_gated");
}

extern "C" int nv_clamped_glu_rows(const void* x, int64_t x_stride, void* y, int dtype, int64_t rows, int inter, float limit,
                                   float alpha, float shift, void* stream) {
    using namespace nv;
    NV_REQUIRE(rows >= 0 && inter > 0 && x_stride >= 2 * (int64_t)inter, NV_ERR_INVALID_ARG, "nv_clamped_glu_rows: bad sizes");
    if (rows == 0) return NV_OK;
    NV_REQUIRE(x && y, NV_ERR_INVALID_ARG, "nv_clamped_glu_rows: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_clamped_glu_rows: bad dtype");
    const bool bf = dtype == NV_DTYPE_BF16;
    const bool vec = inter % 8 == 0 && x_stride % 8 == 0 && ((uintptr_t)x | (uintptr_t)y) % 16 == 0;
    const int pieces = vec ? inter / 8 : inter;
    const int64_t n = rows * pieces, grid = (n + 255) / 256;
    NV_REQUIRE(grid < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_clamped_glu_rows: launch too large");
    hipStream_t s = (hipStream_t)stream;
#define NV_GLU(T, V)                                                                                                 \
    hipLaunchKernelGGL((clamped_glu_rows_kernel<T, V>), dim3((unsigned)grid), dim3(256), 0, s, (const T*)x, x_stride, \
                       (T*)y, inter, pieces, n, limit, alpha, shift)
    if (bf && vec) NV_GLU(__bf16, 8);
    else if (bf) NV_GLU(__bf16, 1);
    else if (vec) NV_GLU(float, 8);
    else NV_GLU(float, 1);
#undef NV_GLU
    return check_launch("nv_clamped_glu_rows");
}

extern "C" int nv_scale_softcap(const void* x, float* y, int dtype, int64_t n, float scale, float cap, void* stream) {
    using namespace nv;
    NV_REQUIRE(n >= 0 && cap >= 0.f, NV_ERR_INVALID_ARG, "nv_scale_softcap: bad sizes");
    if (n == 0) return NV_OK;
    NV_REQUIRE(x && y, NV_ERR_INVALID_ARG, "nv_scale_softcap: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_scale_softcap: bad dtype");
    const bool bf = dtype == NV_DTYPE_BF16;
    const bool vec = n % 4 == 0 && (uintptr_t)x % (bf ? 8 : 16) == 0 && (uintptr_t)y % 16 == 0;
    const int64_t grid = (n / (vec ? 4 : 1) + 255) / 256;
    NV_REQUIRE(grid < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_scale_softcap: launch too large");
    hipStream_t s = (hipStream_t)stream;
#define NV_CAP(T, V) \
    hipLaunchKernelGGL((scale_softcap_kernel<T, V>), dim3((unsigned)grid), dim3(256), 0, s, (const T*)x, y, n, scale, cap)
    if (bf && vec) NV_CAP(__bf16, 4);
    else if (bf) NV_CAP(__bf16, 1);
    else if (vec) NV_CAP(float, 4);
    else NV_CAP(float, 1);
#undef NV_CAP
    return check_launch("nv_scale_softcap");
}
