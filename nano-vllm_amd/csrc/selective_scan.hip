// Selective scan: a diagonal linear recurrence per channel whose decay and input depend on the token, state [C, N] (channel
// x state) in fp32, carried per SEQUENCE in numbered slots (a sequence whose rows start at position 0 starts from a zero
// state whatever its slot holds):
//
//   dt = softplus(dt_raw + dt_bias)                                       one per token and channel
//   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;   y_c = sum_n S[c, n] C_n + D_c x_c
//   out_c = y_c * silu(z_c)
//
// B and C are vectors [N] per token shared by all channels.  Everything behind the raw inputs is fp32.
//
// Layout: L lanes share a channel and own SPL of its states each, in registers; a workgroup of 256 threads takes 256 / L
// channels of one sequence.  16 tokens at a time are prepared into LDS (softplus and dt x once per token and channel, B and
// C once per token), the next 16 tokens' inputs being on their way into registers meanwhile; the token loop has no
// barrier: two small LDS reads per vector, one exponential and three multiply-adds per state, a sum over the L lanes.
//
// A step with too few (sequence, channel) pairs to fill the chip is cut into segments along time (segments.h); what a segment
// leaves is its end state and its sum of dt per channel: the decay of a whole segment is exp(A * sum dt).  Leading single
// tokens have a launch of their own.
#include <algorithm>

#include "row_pieces.h"
#include "segments.h"
#include "../../include/nanovllm_hip_mixers.h"

namespace nv {

constexpr int kScThreads = 256;
constexpr int kScTile = 16;                    // tokens prepared at a time

constexpr float kScLog2e = 1.4426950408889634f, kScLn2 = 0.6931471805599453f;

// log(1 + exp(x)) = max(x, 0) + log1p(u), u = exp(-|x|); log1p(u) = u log(w) / (w - 1) with w = 1 + u rounded (the rounding
// of w cancels: D. Goldberg, "What Every Computer Scientist Should Know About Floating-Point Arithmetic", theorem 4).
__device__ __forceinline__ float sc_softplus(float x) {
    const float u = __builtin_amdgcn_exp2f(-fabsf(x) * kScLog2e), w = 1.0f + u, d = w - 1.0f;
    const float l = d == 0.f ? u : __builtin_amdgcn_logf(w) * kScLn2 * (u * __builtin_amdgcn_rcpf(d));
    return fmaxf(x, 0.f) + l;
}
__device__ __forceinline__ float sc_silu(float x) {
    return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-kScLog2e * x));
}

// The SPL states n0 .. of a channel's row of N: in pieces of four where the row allows it.  `in` says whether the lane has any.
template <int SPL>
__device__ __forceinline__ void sc_load_states(const float* row, int n0, int N, bool in, float* s) {
#pragma unroll
    for (int i = 0; i < SPL; i += 4) {
        float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
        if (N % 4 == 0) {
            if (in && n0 + i < N) v = *(const float4*)(row + n0 + i);
        } else if (in) {
            if (n0 + i < N) v.x = row[n0 + i];
            if (n0 + i + 1 < N) v.y = row[n0 + i + 1];
            if (n0 + i + 2 < N) v.z = row[n0 + i + 2];
            if (n0 + i + 3 < N) v.w = row[n0 + i + 3];
        }
        s[i] = v.x; s[i + 1] = v.y; s[i + 2] = v.z; s[i + 3] = v.w;
    }
}
template <int SPL>
__device__ __forceinline__ void sc_store_states(float* row, int n0, int N, const float* s) {
#pragma unroll
    for (int i = 0; i < SPL; i += 4) {
        if (N % 4 == 0) {
            if (n0 + i < N) *(float4*)(row + n0 + i) = make_float4(s[i], s[i + 1], s[i + 2], s[i + 3]);
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (n0 + i + e < N) row[n0 + i + e] = s[i + e];
        }
    }
}

// Sum over aligned groups of L lanes; every lane of the group gets it.
template <int L>
__device__ __forceinline__ float sc_group_sum(float x) {
    if constexpr (L >= 2) x += dpp_f32<0xB1>(x);      // quad_perm [1,0,3,2]
    if constexpr (L >= 4) x += dpp_f32<0x4E>(x);      // quad_perm [2,3,0,1]
    if constexpr (L >= 8) x += dpp_f32<0x141>(x);     // row_half_mirror
    if constexpr (L >= 16) x += dpp_f32<0x140>(x);    // row_mirror
    if constexpr (L >= 32) x += __shfl_xor(x, 16);
    if constexpr (L >= 64) x += __shfl_xor(x, 32);
    return x;
}

template <typename T>
struct ScArgs {
    const T *x, *dt_raw, *z, *Bm, *Cm;         // [T, C], [T, C], [T, C], [T, N], [T, N] with row strides
    int64_t x_stride, dt_stride, z_stride, b_stride, c_stride;
    const float *dt_bias, *A, *D;              // [C], [C, N], [C]
    float* state;                              // [slots, C, N]
    T* out;                                    // [T, C]
    int64_t out_stride;
    const int *cu_q, *cu_k, *slots;
    int C, N;
    int seg_len, nseg;                         // tokens per segment (a multiple of kScTile), segments of the longest sequence
    float *seg_state, *seg_dt;                 // [places, C, N], [places, C]
};

// Four neighbouring columns of a row as they lie in memory (zeros from `cols` on): what is on its way must not be touched.
template <typename T> struct ScRaw;
template <> struct ScRaw<__bf16> { typedef uint2 type; };
template <> struct ScRaw<float> { typedef float4 type; };
template <bool VEC, typename T>
__device__ __forceinline__ typename ScRaw<T>::type sc_fetch4(const T* row, int c, int cols, bool in) {
    typedef typename ScRaw<T>::type R;
    R r = {};
    if (in) {
        if constexpr (VEC) {
            r = *(const R*)(row + c);
        } else {
            T* e = (T*)&r;
#pragma unroll
            for (int i = 0; i < 4; ++i)
                if (c + i < cols) e[i] = row[c + i];
        }
    }
    return r;
}
__device__ __forceinline__ Cols<4> sc_widen(uint2 r) {
    return Cols<4>{{bf16_lo(r.x), bf16_hi(r.x), bf16_lo(r.y), bf16_hi(r.y)}};
}
__device__ __forceinline__ Cols<4> sc_widen(float4 r) { return Cols<4>{{r.x, r.y, r.z, r.w}}; }

enum { kScWhole = 0, kScSummary = 1, kScFinal = 2 };

// VEC: rows of x, dt_raw, z, out, B and C may be walked in pieces of four columns.
template <typename T, int L, int SPL, int MODE, bool VEC>
__global__ __launch_bounds__(kScThreads) void selective_scan_kernel(const ScArgs<T> a) {
    constexpr int CPB = kScThreads / L;                          // channels of the workgroup
    constexpr int NP = L * SPL;                                  // states, padded
    constexpr int PIECES = kScTile * CPB / 4;                    // four-channel pieces of a tile
    constexpr int IT = (PIECES + kScThreads - 1) / kScThreads;
    constexpr int BPIECES = kScTile * NP / 4;                    // four-state pieces of B and of C
    constexpr int IB = (BPIECES + kScThreads - 1) / kScThreads;
    __shared__ float2 dts[kScTile][CPB];                         // (dt, dt x)
    __shared__ __attribute__((aligned(16))) float bs[kScTile][NP], cs[kScTile][NP];
    __shared__ __attribute__((aligned(16))) float ys[kScTile][CPB];
    const int b = blockIdx.x, c0 = blockIdx.y * CPB, seg = blockIdx.z;
    const int q0 = a.cu_q[b], len_q = a.cu_q[b + 1] - q0;
    if (len_q <= 0) return;
    const int first = seg * a.seg_len, last_seg = segment_count(len_q, a.seg_len, a.nseg) - 1;
    if (seg > last_seg) return;
    const int start = (a.cu_k[b + 1] - a.cu_k[b]) - len_q;
    const int tid = threadIdx.x, ch = tid / L, sub = tid % L;
    const int C = a.C, N = a.N, c = c0 + ch;
    const bool live = c < C;
    float* slot_state = a.state + ((int64_t)a.slots[b] * C + c) * N;
    const int n0 = sub * SPL;
    float A2[SPL], S[SPL];                                       // A log2(e); the state
    sc_load_states<SPL>(a.A + (int64_t)c * N, n0, N, live, A2);
#pragma unroll
    for (int i = 0; i < SPL; ++i) {
        A2[i] *= kScLog2e;
        S[i] = 0.f;
    }
    int64_t place = 0;                                           // of the sequence's first segment
    if (MODE != kScWhole && last_seg > 0) place = segment_first_place(a.cu_q, b, a.seg_len, a.nseg);
    if constexpr (MODE == kScSummary) {
        if (last_seg == 0) return;                               // nobody folds
        if (seg == last_seg) {                                   // the start state is handed on from here: the second launch
            if (!live) return;                                   // overwrites the slot
            sc_load_states<SPL>(slot_state, n0, N, start > 0, S);
            sc_store_states<SPL>(a.seg_state + ((place + seg) * C + c) * N, n0, N, S);
            return;
        }
    } else {
        if (MODE == kScFinal && last_seg > 0) {
            sc_load_states<SPL>(a.seg_state + ((place + last_seg) * C + c) * N, n0, N, live, S);
            for (int s = 0; s < seg; ++s) {
                const int64_t at = (place + s) * C + c;
                const float dsum = live ? a.seg_dt[at] : 0.f;
                float loc[SPL];
                sc_load_states<SPL>(a.seg_state + at * N, n0, N, live, loc);
#pragma unroll
                for (int i = 0; i < SPL; ++i) S[i] = __builtin_amdgcn_exp2f(dsum * A2[i]) * S[i] + loc[i];
            }
        } else {
            sc_load_states<SPL>(slot_state, n0, N, live && start > 0, S);
        }
    }
    float dt_sum = 0.f;
    // the thread's four channels wherever it prepares or writes tokens (the threads are whole rows of pieces)
    const int cl = (tid % (CPB / 4)) * 4, cc = c0 + cl;
    float bias[4], skip[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        bias[e] = cc + e < C ? a.dt_bias[cc + e] : 0.f;
        skip[e] = cc + e < C ? a.D[cc + e] : 0.f;
    }
    const int stop = seg == last_seg ? len_q : first + a.seg_len;
    // the tile that comes next, as it arrives, and (x, z) of the one that is being scanned
    typename ScRaw<T>::type ndt[IT], nx[IT], nz[IT], x_cur[IT], z_cur[IT], nb[IB], nc[IB];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int k = 0; k < IT; ++k) {
            const int p = tid + k * kScThreads, tt = p / (CPB / 4);
            const bool in = p < PIECES && t0 + tt < stop && cc < C;
            const int64_t t = q0 + t0 + tt;
            ndt[k] = sc_fetch4<VEC>(a.dt_raw + t * a.dt_stride, cc, C, in);
            nx[k] = sc_fetch4<VEC>(a.x + t * a.x_stride, cc, C, in);
            if constexpr (MODE != kScSummary) nz[k] = sc_fetch4<VEC>(a.z + t * a.z_stride, cc, C, in);
        }
#pragma unroll
        for (int k = 0; k < IB; ++k) {
            const int p = tid + k * kScThreads, tt = p / (NP / 4), n = (p % (NP / 4)) * 4;
            const bool in = p < BPIECES && t0 + tt < stop && n < N;
            const int64_t t = q0 + t0 + tt;
            nb[k] = sc_fetch4<VEC>(a.Bm + t * a.b_stride, n, N, in);
            if constexpr (MODE != kScSummary) nc[k] = sc_fetch4<VEC>(a.Cm + t * a.c_stride, n, N, in);
        }
    };
    fetch(first);
    for (int t0 = first; t0 < stop; t0 += kScTile) {
        const int nt = min(kScTile, stop - t0);
        __syncthreads();                                         // the previous tile has been scanned and written
#pragma unroll
        for (int k = 0; k < IT; ++k) {
            const int p = tid + k * kScThreads, tt = p / (CPB / 4);
            x_cur[k] = nx[k];
            if constexpr (MODE != kScSummary) z_cur[k] = nz[k];
            if (p < PIECES) {
                const Cols<4> dr = sc_widen(ndt[k]), xr = sc_widen(nx[k]);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    // (dt = 0 behind the portion's end: those steps leave the state as it is)
                    const float dt = tt < nt ? sc_softplus(dr.v[e] + bias[e]) : 0.f;
                    dts[tt][cl + e] = make_float2(dt, dt * xr.v[e]);
                }
            }
        }
#pragma unroll
        for (int k = 0; k < IB; ++k) {
            const int p = tid + k * kScThreads, tt = p / (NP / 4), n = (p % (NP / 4)) * 4;
            if (p < BPIECES) {
                row_store<4>(&bs[tt][n], sc_widen(nb[k]));
                if constexpr (MODE != kScSummary) row_store<4>(&cs[tt][n], sc_widen(nc[k]));
            }
        }
        __syncthreads();
        if (t0 + kScTile < stop) fetch(t0 + kScTile);
        // ---- the recurrence over the tile, no barrier inside ---------------------------------------------
        for (int t4 = 0; t4 < nt; t4 += 4) {                     // four tokens at a time: their exponentials overlap
            float y[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float2 d = dts[t4 + u][ch];
                const float* bt = &bs[t4 + u][sub * SPL];
                const float* ct = &cs[t4 + u][sub * SPL];
                y[u] = 0.f;
#pragma unroll
                for (int i = 0; i < SPL; ++i) {
                    S[i] = __builtin_amdgcn_exp2f(d.x * A2[i]) * S[i] + d.y * bt[i];
                    if constexpr (MODE != kScSummary) y[u] += S[i] * ct[i];
                }
                if constexpr (MODE == kScSummary) dt_sum += d.x;
            }
            if constexpr (MODE != kScSummary) {
#pragma unroll
                for (int u = 0; u < 4; ++u) y[u] = sc_group_sum<L>(y[u]);
                if (sub == 0) {
#pragma unroll
                    for (int u = 0; u < 4; ++u) ys[t4 + u][ch] = y[u];
                }
            }
        }
        if constexpr (MODE != kScSummary) {
            __syncthreads();
#pragma unroll
            for (int k = 0; k < IT; ++k) {
                const int p = tid + k * kScThreads, tt = p / (CPB / 4);
                if (p >= PIECES || tt >= nt || cc >= C) continue;
                const Cols<4> xr = sc_widen(x_cur[k]), zr = sc_widen(z_cur[k]);
                Cols<4> o;
#pragma unroll
                for (int e = 0; e < 4; ++e) o.v[e] = (ys[tt][cl + e] + skip[e] * xr.v[e]) * sc_silu(zr.v[e]);
                T* dst = a.out + (int64_t)(q0 + t0 + tt) * a.out_stride + cc;
                if constexpr (VEC) {
                    row_store<4>(dst, o);
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (cc + e < C) dst[e] = (T)o.v[e];
                }
            }
        }
    }
    if (!live) return;
    if constexpr (MODE == kScSummary) {
        const int64_t at = (place + seg) * C + c;
        if (sub == 0) a.seg_dt[at] = dt_sum;
        sc_store_states<SPL>(a.seg_state + at * N, n0, N, S);
    } else if (seg == last_seg) {
        sc_store_states<SPL>(slot_state, n0, N, S);
    }
}

// One token per sequence: nothing is worth preparing, every lane reads what it needs.
template <typename T, int L, int SPL>
__global__ __launch_bounds__(kScThreads) void selective_scan_single_kernel(const ScArgs<T> a) {
    constexpr int CPB = kScThreads / L;
    const int b = blockIdx.x, t = a.cu_q[b];
    if (a.cu_q[b + 1] - t != 1) return;
    const bool fresh = a.cu_k[b + 1] - a.cu_k[b] == 1;
    const int ch = threadIdx.x / L, sub = threadIdx.x % L, c = blockIdx.y * CPB + ch, C = a.C, N = a.N, n0 = sub * SPL;
    const bool live = c < C;
    const int cc = live ? c : C - 1;
    float* slot_state = a.state + ((int64_t)a.slots[b] * C + cc) * N;
    float A[SPL], S[SPL];
    sc_load_states<SPL>(slot_state, n0, N, live && !fresh, S);
    sc_load_states<SPL>(a.A + (int64_t)cc * N, n0, N, live, A);
    const float x = (float)a.x[(int64_t)t * a.x_stride + cc], z = (float)a.z[(int64_t)t * a.z_stride + cc];
    const float dt = sc_softplus((float)a.dt_raw[(int64_t)t * a.dt_stride + cc] + a.dt_bias[cc]);
    const T *bp = a.Bm + (int64_t)t * a.b_stride, *cp = a.Cm + (int64_t)t * a.c_stride;
    const float dx = dt * x, dt2 = dt * kScLog2e;
    float y = 0.f;
#pragma unroll
    for (int i = 0; i < SPL; ++i) {
        const int n = n0 + i;
        const float bn = n < N ? (float)bp[n] : 0.f, cn = n < N ? (float)cp[n] : 0.f;
        S[i] = __builtin_amdgcn_exp2f(dt2 * A[i]) * S[i] + dx * bn;
        y += S[i] * cn;
    }
    y = sc_group_sum<L>(y);
    if (!live) return;
    sc_store_states<SPL>(slot_state, n0, N, S);
    if (sub == 0) a.out[(int64_t)t * a.out_stride + c] = (T)((y + a.D[c] * x) * sc_silu(z));
}

struct ScPlan {
    int L, SPL, nseg, seg_len;
    int64_t ws_floats;
};

// Lanes per channel and states per lane from N; segments so that the launch has about four waves per SIMD.  The sequences that
// count are the long ones: T rows make at most that many portions of the longest one's length.
static ScPlan sc_plan(int B, int64_t T, int C, int N, int max_seqlen_q, int lead) {
    ScPlan p{1, 4, 1, 0, 0};
    B -= lead;
    T -= lead;
    while (p.L * 4 < N) p.L *= 2;
    const int mq = std::max(1, max_seqlen_q);
    const int64_t seqs = std::max<int64_t>(0, std::min<int64_t>(B, (T + mq - 1) / mq));
    // eight states per lane (half the lanes, less work per token beside the states) when there are plenty of waves
    if (p.L >= 4 && seqs * C * p.L / 64 >= 8192) {
        p.SPL = 8;
        p.L /= 2;
    }
    const int64_t waves = std::max<int64_t>(1, seqs * C * p.L / 64);
    p.seg_len = (mq + kScTile - 1) / kScTile * kScTile;
    if (seqs > 0 && waves < 2048 && mq >= 256) {
        const int want = (int)std::min<int64_t>((4096 + waves - 1) / waves, 16);
        p.nseg = std::max(1, std::min(want, mq / 128));
        p.seg_len = ((mq + p.nseg - 1) / p.nseg + kScTile - 1) / kScTile * kScTile;
        p.nseg = (mq + p.seg_len - 1) / p.seg_len;
    }
    if (p.nseg > 1) p.ws_floats = segment_places(T, p.seg_len) * C * (N + 1);
    return p;
}

template <typename T, int L, int SPL>
static void launch_scan(const ScArgs<T>& a, int B, hipStream_t s) {
    constexpr int CPB = kScThreads / L;
    const dim3 grid((unsigned)B, (unsigned)((a.C + CPB - 1) / CPB), (unsigned)a.nseg), block(kScThreads);
    if (a.nseg == 1) {
        hipLaunchKernelGGL((selective_scan_kernel<T, L, SPL, kScWhole, true>), grid, block, 0, s, a);
        return;
    }
    hipLaunchKernelGGL((selective_scan_kernel<T, L, SPL, kScSummary, true>), grid, block, 0, s, a);
    hipLaunchKernelGGL((selective_scan_kernel<T, L, SPL, kScFinal, true>), grid, block, 0, s, a);
}

template <typename T>
static int run_scan(ScArgs<T> a, const ScPlan& p, bool vec, int lead, int B, hipStream_t s) {
    const int lanes = p.L * p.SPL / 4;                           // at four states per lane
    if (lead > 0) {
        bool done = false;
#define NV_SC_SINGLE(LL)                                                                                                       \
    if (lanes == LL) {                                                                                                          \
        constexpr int CPS = kScThreads / LL;                                                                                    \
        hipLaunchKernelGGL((selective_scan_single_kernel<T, LL, 4>), dim3((unsigned)lead, (unsigned)((a.C + CPS - 1) / CPS)),    \
                           dim3(kScThreads), 0, s, a);                                                                          \
        done = true;                                                                                                            \
    }
        NV_SC_SINGLE(1) NV_SC_SINGLE(2) NV_SC_SINGLE(4) NV_SC_SINGLE(8) NV_SC_SINGLE(16) NV_SC_SINGLE(32) NV_SC_SINGLE(64)
#undef NV_SC_SINGLE
        NV_REQUIRE(done, NV_ERR_UNSUPPORTED, "nv_selective_scan: no kernel for %d lanes", lanes);
        const int rc = check_launch("nv_selective_scan (single tokens)");
        if (rc != NV_OK || lead == B) return rc;
        a.cu_q += lead;                                          // (row numbers stay those of the step)
        a.cu_k += lead;
        a.slots += lead;
        B -= lead;
    }
    if (!vec) {                                                  // rows of odd sizes: one plain form
        a.nseg = 1;
#define NV_SC_PLAIN(LL)                                                                                                        \
    if (lanes == LL) {                                                                                                          \
        constexpr int CPB = kScThreads / LL;                                                                                    \
        hipLaunchKernelGGL((selective_scan_kernel<T, LL, 4, kScWhole, false>), dim3((unsigned)B, (unsigned)((a.C + CPB - 1) / CPB)), \
                           dim3(kScThreads), 0, s, a);                                                                          \
        return check_launch("nv_selective_scan");                                                                               \
    }
        NV_SC_PLAIN(1) NV_SC_PLAIN(2) NV_SC_PLAIN(4) NV_SC_PLAIN(8) NV_SC_PLAIN(16) NV_SC_PLAIN(32) NV_SC_PLAIN(64)
#undef NV_SC_PLAIN
    }
#define NV_SC(LL, SS)                                                                                                          \
    if (p.L == LL && p.SPL == SS) {                                                                                             \
        launch_scan<T, LL, SS>(a, B, s);                                                                                        \
        return check_launch("nv_selective_scan");                                                                               \
    }
    NV_SC(1, 4) NV_SC(2, 4) NV_SC(4, 4) NV_SC(8, 4) NV_SC(16, 4) NV_SC(32, 4) NV_SC(64, 4)
    NV_SC(2, 8) NV_SC(4, 8) NV_SC(8, 8) NV_SC(16, 8) NV_SC(32, 8)
#undef NV_SC
    set_error("nv_selective_scan: no kernel for %d lanes x %d states", p.L, p.SPL);
    return NV_ERR_UNSUPPORTED;
}

}  // namespace nv

extern "C" int64_t nv_selective_scan_workspace_bytes(int num_seqs, int64_t T, int C, int N, int max_seqlen_q, int leading_singles) {
    if (num_seqs <= 0 || T <= 0 || leading_singles < 0 || leading_singles > num_seqs || C <= 0 || N <= 0 || N > 256) return 0;
    return nv::sc_plan(num_seqs, T, C, N, max_seqlen_q, leading_singles).ws_floats * (int64_t)sizeof(float);
}

extern "C" int nv_selective_scan(const void* x, int64_t x_stride, const void* dt_raw, int64_t dt_stride, const void* z,
                                 int64_t z_stride, const void* Bm, int64_t b_stride, const void* Cm, int64_t c_stride,
                                 const float* dt_bias, const float* A, const float* D_skip, float* state, void* out,
                                 int64_t out_stride, const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k,
                                 const int32_t* state_slots, int num_seqs, int64_t T, int C, int N, int max_seqlen_q,
                                 int leading_singles, int dtype,
                                 void* workspace, int64_t workspace_bytes, void* stream) {
    using namespace nv;
    NV_REQUIRE(num_seqs >= 0 && T >= 0 && C > 0 && N > 0 && max_seqlen_q >= 1 && leading_singles >= 0 &&
                   leading_singles <= num_seqs,
               NV_ERR_INVALID_ARG, "nv_selective_scan: bad sizes");
    if (num_seqs == 0 || T == 0) return NV_OK;
    NV_REQUIRE(x && dt_raw && z && Bm && Cm && dt_bias && A && D_skip && state && out && cu_seqlens_q && cu_seqlens_k &&
                   state_slots,
               NV_ERR_INVALID_ARG, "nv_selective_scan: null pointer");
    NV_REQUIRE(N <= 256, NV_ERR_UNSUPPORTED, "nv_selective_scan: %d states per channel exceed 256", N);
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_selective_scan: bad dtype");
    const ScPlan p = sc_plan(num_seqs, T, C, N, max_seqlen_q, leading_singles);
    NV_REQUIRE(C / 4 < 65535, NV_ERR_UNSUPPORTED, "nv_selective_scan: launch too large");
    NV_REQUIRE(p.ws_floats == 0 || (workspace && workspace_bytes >= p.ws_floats * (int64_t)sizeof(float)), NV_ERR_WORKSPACE,
               "nv_selective_scan: workspace of %lld bytes, need %lld", (long long)workspace_bytes,
               (long long)(p.ws_floats * (int64_t)sizeof(float)));
    hipStream_t s = (hipStream_t)stream;
    float* seg_state = (float*)workspace;
    float* seg_dt = p.nseg > 1 ? seg_state + segment_places(T - leading_singles, p.seg_len) * C * N : nullptr;
    const int align = dtype == NV_DTYPE_BF16 ? 8 : 16;
    const bool vec = C % 4 == 0 && x_stride % 4 == 0 && dt_stride % 4 == 0 && z_stride % 4 == 0 && out_stride % 4 == 0 &&
                     N % 4 == 0 && b_stride % 4 == 0 && c_stride % 4 == 0 &&
                     ((uintptr_t)x | (uintptr_t)dt_raw | (uintptr_t)z | (uintptr_t)out | (uintptr_t)Bm | (uintptr_t)Cm) % align == 0;
    if (dtype == NV_DTYPE_BF16) {
        const ScArgs<__bf16> a{(const __bf16*)x, (const __bf16*)dt_raw, (const __bf16*)z, (const __bf16*)Bm, (const __bf16*)Cm,
                               x_stride, dt_stride, z_stride, b_stride, c_stride, dt_bias, A, D_skip, state, (__bf16*)out,
                               out_stride, cu_seqlens_q, cu_seqlens_k, state_slots, C, N, p.seg_len, p.nseg, seg_state, seg_dt};
        return run_scan<__bf16>(a, p, vec, leading_singles, num_seqs, s);
    }
    const ScArgs<float> a{(const float*)x, (const float*)dt_raw, (const float*)z, (const float*)Bm, (const float*)Cm, x_stride,
                          dt_stride, z_stride, b_stride, c_stride, dt_bias, A, D_skip, state, (float*)out, out_stride,
                          cu_seqlens_q, cu_seqlens_k, state_slots, C, N, p.seg_len, p.nseg, seg_state, seg_dt};
    return run_scan<float>(a, p, vec, leading_singles, num_seqs, s);
}
