// Linear attention with one constant decay per head (lightning attention), state [Dk, Dv] in fp32 per head and sequence:
//
//   q = silu(q_raw), k = silu(k_raw), v = silu(v_raw);   S_t = decay_h S_(t-1) + k_t v_t^T;   o_t = S_t^T q_t
//
// Single tokens stream the state through once (read, decayed, written, read out); portions of a few tokens run token by token
// with the state in registers (gated_memory.hip); longer ones in chunks of 64 tokens on the matrix cores:
// with tokens i, j of a chunk and the state S in front of it
//
//   o_i = decay^(i+1) S^T q_i + sum_(j <= i) decay^(i-j) (q_i . k_j) v_j
//   S  <- decay^n S + sum_j decay^(n-1-j) k_j v_j^T                                (n tokens in the chunk)
//
// One workgroup of four waves per (sequence, head, 64 value columns).  q, k, v of a chunk are staged in LDS after their SiLU
// (bf16, as activations are), the next chunk's rows being on their way into registers meanwhile.  Wave w scores queries
// 16 w .. 16 w + 15 against the keys in front of them and hands the decayed scores to all waves; every wave owns 16 value
// columns, keeps the state of those columns in its accumulators, reads it, adds the chunk's own part and updates it.  What
// is fp32 in the token-by-token form and an operand here (decayed scores, the state that is read, decayed values) enters
// as the sum of two bf16 numbers, a product each, so about 16 bits of it count.
//
// All products are v_mfma_f32_16x16x32_bf16.  Accumulators of one product are the operand of the next in place: a lane
// holds rows 4 g .. 4 g + 3 of two stacked 16-row tiles (g: its group of 16 lanes), so the contraction index runs in the
// order 16 (e / 4) + 4 g + e % 4, and the other operand is read in the same order (two 8-byte reads, or two transposed ones).
//
// Long portions in a step that does not fill the chip are cut into segments (segments.h); the decay of a whole segment is
// decay^length.
#include <algorithm>

#include "fixed_decay.h"
#include "mfma_tile.h"
#include "row_pieces.h"
#include "segments.h"
#include "../../include/nanovllm_hip_mixers.h"

namespace nv {

typedef __attribute__((address_space(3))) s16x4 fd_lds_s16x4;

constexpr int kFdChunk = 64;
constexpr int kFdFewRows = NV_FEW_ROWS;                 // portions of at most this many tokens run token by token
constexpr int kFdVs = 64 + 8;                  // LDS row of the values, in elements

struct FdParams {
    FixedDecayArgs f;
    int seg_len, nseg;                         // tokens per segment (a multiple of kFdChunk)
    float* seg_state;                          // [places, H, Dk, Dv]
};

__device__ __forceinline__ float fd_silu(float x) {
    return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
}
__device__ __forceinline__ uint4 fd_silu8(uint4 u) {
    return make_uint4(pack_bf16(fd_silu(bf16_lo(u.x)), fd_silu(bf16_hi(u.x))), pack_bf16(fd_silu(bf16_lo(u.y)), fd_silu(bf16_hi(u.y))),
                      pack_bf16(fd_silu(bf16_lo(u.z)), fd_silu(bf16_hi(u.z))), pack_bf16(fd_silu(bf16_lo(u.w)), fd_silu(bf16_hi(u.w))));
}
// 8 columns of a row from c0 on, zeros past `cols` or for a missing row.  One guarded load and nothing else in the whole-piece
// form: a choice between two forms at run time would make every load wait for the one before.
template <bool VEC>
__device__ __forceinline__ uint4 fd_fetch(const __bf16* row, int c0, int cols) {
    if constexpr (VEC) {
        uint4 r = make_uint4(0, 0, 0, 0);
        if (row != nullptr && c0 < cols) r = *(const uint4*)(row + c0);
        return r;
    } else {
        return tile_fetch<__bf16>(row, c0, cols, false);
    }
}
// x = hi + lo, each bf16
__device__ __forceinline__ void fd_split(const float* x, bf16x8& hi, bf16x8& lo) {
#pragma unroll
    for (int e = 0; e < 8; ++e) {
        hi[e] = (__bf16)x[e];
        lo[e] = (__bf16)(x[e] - (float)hi[e]);
    }
}
__device__ __forceinline__ bf16x8 fd_join(s16x4 a, s16x4 b) {
    typedef __attribute__((ext_vector_type(8))) short s16x8;
    s16x8 v;
    v[0] = a[0]; v[1] = a[1]; v[2] = a[2]; v[3] = a[3];
    v[4] = b[0]; v[5] = b[1]; v[6] = b[2]; v[7] = b[3];
    return __builtin_bit_cast(bf16x8, v);
}
// column c0 + (lane & 15) of rows row0 + 4 g .. + 3 and row0 + 16 + 4 g .. + 3 of an LDS matrix with `ld` elements per row
__device__ __forceinline__ bf16x8 fd_columns(const __bf16* m, int ld, int row0, int c0, int lane) {
    const int i16 = lane & 15, g = lane >> 4;
    const __bf16* p = m + (row0 + 4 * g + (i16 >> 2)) * ld + c0 + (i16 & 3) * 4;
    return fd_join(__builtin_amdgcn_ds_read_tr16_b64_v4i16((fd_lds_s16x4*)p),
                   __builtin_amdgcn_ds_read_tr16_b64_v4i16((fd_lds_s16x4*)(p + 16 * ld)));
}
__device__ __forceinline__ f32x4 fd_mma(bf16x8 a, bf16x8 b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

enum { kFdWhole = 0, kFdSummary = 1, kFdFinal = 2 };

// VEC: rows of q, k, v may be read and rows of out written in 16-byte pieces.
template <int DKT, int MODE, bool VEC>
__global__ __launch_bounds__(256) void fixed_decay_chunk_kernel(const FdParams p) {
    constexpr int DK = 32 * DKT, QS = DK + 8;
    extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
    __bf16* qs = (__bf16*)smem;                                  // [64][QS]
    __bf16* ks = qs + kFdChunk * QS;                             // [64][QS]
    __bf16* vs = ks + kFdChunk * QS;                             // [64][kFdVs]
    bf16x8* ps = (bf16x8*)(vs + kFdChunk * kFdVs);               // [query tile][key half][high, low][lane]
    float* pw = (float*)(ps + 4 * 2 * 2 * 64);                   // [65] powers of the decay
    const FixedDecayArgs& f = p.f;
    const int H = f.H, Dk = f.Dk, Dv = f.Dv;
    const int b = blockIdx.x, h = blockIdx.y % H, cg = blockIdx.y / H, seg = blockIdx.z;
    const int q0 = f.cu_q[b], len_q = f.cu_q[b + 1] - q0;
    if (len_q <= kFdFewRows) return;
    const int first = seg * p.seg_len, last_seg = segment_count(len_q, p.seg_len, p.nseg) - 1;
    if (seg > last_seg) return;
    const int start = (f.cu_k[b + 1] - f.cu_k[b]) - len_q;
    const int tid = threadIdx.x, lane = tid & 63, l15 = lane & 15, g = lane >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int col = cg * 64 + wave * 16 + l15;                   // the lane's value column of the state
    const float decay = f.decay[h];
    float* slot_state = f.state + ((int64_t)f.slots[b] * H + h) * (int64_t)Dk * Dv;
    int64_t place = 0;                                           // of the sequence's first segment
    if (MODE != kFdWhole && last_seg > 0) place = segment_first_place(f.cu_q, b, p.seg_len, p.nseg);
    auto seg_at = [&](int s) { return p.seg_state + ((place + s) * H + h) * (int64_t)Dk * Dv; };

    f32x4 S[2 * DKT];                                            // S[t][r]: key channel 16 t + 4 g + r, value column col
#pragma unroll
    for (int t = 0; t < 2 * DKT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[t][r] = 0.f;
    // Entries outside the state are read from its edge and not written: all loads of a state are in flight together.
    auto load_state = [&](const float* m, f32x4* to) {
#pragma unroll
        for (int t = 0; t < 2 * DKT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) to[t][r] = m[(int64_t)min(16 * t + 4 * g + r, Dk - 1) * Dv + min(col, Dv - 1)];
    };
    auto store_state = [&](float* m) {
#pragma unroll
        for (int t = 0; t < 2 * DKT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int d = 16 * t + 4 * g + r;
                if (d < Dk && col < Dv) m[(int64_t)d * Dv + col] = S[t][r];
            }
    };
    if constexpr (MODE == kFdSummary) {
        if (last_seg == 0) return;                               // nobody folds
        if (seg == last_seg) {                                   // the start state is handed on from here: the second launch
            if (start > 0) load_state(slot_state, S);            // overwrites the slot
            store_state(seg_at(seg));
            return;
        }
    } else {
        if (MODE == kFdFinal && last_seg > 0) {
            load_state(seg_at(last_seg), S);
            const float over = powf(decay, (float)p.seg_len);
            f32x4 loc[2 * DKT];
            for (int s = 0; s < seg; ++s) {
                load_state(seg_at(s), loc);
#pragma unroll
                for (int t = 0; t < 2 * DKT; ++t)
#pragma unroll
                    for (int r = 0; r < 4; ++r) S[t][r] = over * S[t][r] + loc[t][r];
            }
        } else if (start > 0) {
            load_state(slot_state, S);
        }
        // (what stands for entries outside the state meets zeros in k and is never read out: q is zero there, and so is the
        // value column's output not written)
    }
    if (tid <= kFdChunk) pw[tid] = powf(decay, (float)tid);
    const int stop = seg == last_seg ? len_q : first + p.seg_len;

    uint4 rq[DKT], rk[DKT], rv[2];                               // the chunk that comes next, as it arrives
    auto fetch = [&](int t0) {
#pragma unroll
        for (int i = 0; i < DKT; ++i) {
            const int pc = tid + 256 * i, row = pc / (4 * DKT), d0 = (pc % (4 * DKT)) * 8;
            const int64_t t = q0 + t0 + row;
            const bool in = t0 + row < stop;
            if constexpr (MODE != kFdSummary)
                rq[i] = fd_fetch<VEC>(in ? (const __bf16*)f.q + t * f.q_stride + (int64_t)h * Dk : nullptr, d0, Dk);
            rk[i] = fd_fetch<VEC>(in ? (const __bf16*)f.k + t * f.k_stride + (int64_t)h * Dk : nullptr, d0, Dk);
        }
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const int pc = tid + 256 * i, row = pc >> 3, c0 = cg * 64 + (pc & 7) * 8;
            const bool in = t0 + row < stop;
            rv[i] = fd_fetch<VEC>(in ? (const __bf16*)f.v + (int64_t)(q0 + t0 + row) * f.v_stride + (int64_t)h * Dv : nullptr,
                                       c0, Dv);
        }
    };
    fetch(first);
    for (int t0 = first; t0 < stop; t0 += kFdChunk) {
        const int nt = min(kFdChunk, stop - t0);
        __syncthreads();                                         // everybody is done with the previous chunk
#pragma unroll
        for (int i = 0; i < DKT; ++i) {
            const int pc = tid + 256 * i, row = pc / (4 * DKT), d0 = (pc % (4 * DKT)) * 8;
            if constexpr (MODE != kFdSummary) *(uint4*)(qs + row * QS + d0) = fd_silu8(rq[i]);
            *(uint4*)(ks + row * QS + d0) = fd_silu8(rk[i]);
        }
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            const int pc = tid + 256 * i;
            *(uint4*)(vs + (pc >> 3) * kFdVs + (pc & 7) * 8) = fd_silu8(rv[i]);
        }
        __syncthreads();
        if (t0 + kFdChunk < stop) fetch(t0 + kFdChunk);
        bf16x8 vf[2];                                            // the lane's value column, keys 32 m + (the order above)
#pragma unroll
        for (int m = 0; m < 2; ++m) vf[m] = fd_columns(vs, kFdVs, 32 * m, 16 * wave, lane);
        if constexpr (MODE != kFdSummary) {
            // ---- decayed scores of the wave's 16 queries against the keys up to them -----------------------
            {
                bf16x8 qf[DKT];
                const int i = 16 * wave + l15;
#pragma unroll
                for (int kk = 0; kk < DKT; ++kk) qf[kk] = *(const bf16x8*)(qs + i * QS + 32 * kk + 8 * g);
#pragma unroll
                for (int m = 0; m < 2; ++m) {
                    if (2 * m > wave) continue;
                    float w[8];
#pragma unroll
                    for (int half = 0; half < 2; ++half) {
                        const int jt = 2 * m + half;
                        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
                        if (jt <= wave) {
#pragma unroll
                            for (int kk = 0; kk < DKT; ++kk)
                                acc = fd_mma(*(const bf16x8*)(ks + (16 * jt + l15) * QS + 32 * kk + 8 * g), qf[kk], acc);
                        }
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int j = 16 * jt + 4 * g + r;
                            w[4 * half + r] = j <= i ? acc[r] * pw[i - j] : 0.f;
                        }
                    }
                    bf16x8 hi, lo;
                    fd_split(w, hi, lo);
                    ps[((wave * 2 + m) * 2 + 0) * 64 + lane] = hi;
                    ps[((wave * 2 + m) * 2 + 1) * 64 + lane] = lo;
                }
            }
            // ---- what the state in front of the chunk gives to its queries --------------------------------
            f32x4 o[4];
#pragma unroll
            for (int it = 0; it < 4; ++it) o[it] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int m = 0; m < DKT; ++m) {
                const float sv[8] = {S[2 * m][0],     S[2 * m][1],     S[2 * m][2],     S[2 * m][3],
                                     S[2 * m + 1][0], S[2 * m + 1][1], S[2 * m + 1][2], S[2 * m + 1][3]};
                bf16x8 hi, lo;
                fd_split(sv, hi, lo);
#pragma unroll
                for (int it = 0; it < 4; ++it) {
                    const __bf16* qr = qs + (16 * it + l15) * QS + 32 * m + 4 * g;
                    const bf16x8 qp = fd_join(*(const s16x4*)qr, *(const s16x4*)(qr + 16));
                    o[it] = fd_mma(hi, qp, o[it]);
                    o[it] = fd_mma(lo, qp, o[it]);
                }
            }
#pragma unroll
            for (int it = 0; it < 4; ++it) {
                const float d = pw[16 * it + l15 + 1];
#pragma unroll
                for (int r = 0; r < 4; ++r) o[it][r] *= d;
            }
            __syncthreads();                                     // the scores of all waves are there
            // ---- the chunk's own keys -----------------------------------------------------------------------
#pragma unroll
            for (int it = 0; it < 4; ++it) {
#pragma unroll
                for (int m = 0; m < 2; ++m) {
                    if (2 * m > it) continue;
                    o[it] = fd_mma(vf[m], ps[((it * 2 + m) * 2 + 0) * 64 + lane], o[it]);
                    o[it] = fd_mma(vf[m], ps[((it * 2 + m) * 2 + 1) * 64 + lane], o[it]);
                }
                const int i = 16 * it + l15, c = cg * 64 + 16 * wave + 4 * g;
                if (i < nt && c < Dv) {
                    float* dst = f.out + (int64_t)(q0 + t0 + i) * f.out_stride + (int64_t)h * Dv + c;
                    if constexpr (VEC) {
                        *(float4*)dst = make_float4(o[it][0], o[it][1], o[it][2], o[it][3]);
                    } else {
#pragma unroll
                        for (int r = 0; r < 4; ++r)
                            if (c + r < Dv) dst[r] = o[it][r];
                    }
                }
            }
        }
        // ---- the state behind the chunk ------------------------------------------------------------------------
        const float dn = pw[nt];
#pragma unroll
        for (int t = 0; t < 2 * DKT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[t][r] *= dn;
#pragma unroll
        for (int m = 0; m < 2; ++m) {
            float w[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int j = 32 * m + 16 * (e >> 2) + 4 * g + (e & 3);
                w[e] = (float)vf[m][e] * pw[max(nt - 1 - j, 0)];     // (rows beyond the portion are zero)
            }
            bf16x8 hi, lo;
            fd_split(w, hi, lo);
#pragma unroll
            for (int t = 0; t < 2 * DKT; ++t) {
                const bf16x8 kf = fd_columns(ks, QS, 32 * m, 16 * t, lane);
                S[t] = fd_mma(kf, hi, S[t]);
                S[t] = fd_mma(kf, lo, S[t]);
            }
        }
    }
    if (MODE == kFdSummary) store_state(seg_at(seg));
    else if (seg == last_seg) store_state(slot_state);
}

// ------------------------------------------------------------------------------------------------ one token
// One workgroup per (sequence, head): V value columns per thread (16-byte pieces of the state's rows), the rows over the
// thread groups, eight rows of a thread in flight; the groups' parts of o meet in LDS.
template <typename T, int V>
__global__ __launch_bounds__(256) void fixed_decay_single_kernel(const FixedDecayArgs f, int pieces) {
    constexpr int U = 8;
    extern __shared__ __attribute__((aligned(16))) float fd_smem[];
    const int H = f.H, Dk = f.Dk, Dv = f.Dv;
    float *ks = fd_smem, *qs = ks + Dk, *os = qs + Dk;           // [Dk], [Dk], [groups][Dv]
    const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int t = f.cu_q[b];
    if (f.cu_q[b + 1] - t != 1) return;
    const bool fresh = f.cu_k[b + 1] - f.cu_k[b] == 1;
    for (int d = tid; d < Dk; d += 256) {
        const float k = (float)((const T*)f.k)[(int64_t)t * f.k_stride + (int64_t)h * Dk + d];
        const float q = (float)((const T*)f.q)[(int64_t)t * f.q_stride + (int64_t)h * Dk + d];
        ks[d] = k / (1.0f + expf(-k));
        qs[d] = q / (1.0f + expf(-q));
    }
    const int c = (tid % pieces) * V, group = tid / pieces, groups = 256 / pieces;      // (pieces is a power of two)
    const bool live = c < Dv;
    float v[V], o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) {
        v[e] = live ? (float)((const T*)f.v)[(int64_t)t * f.v_stride + (int64_t)h * Dv + c + e] : 0.f;
        v[e] = v[e] / (1.0f + expf(-v[e]));
        o[e] = 0.f;
    }
    const float decay = f.decay[h];
    float* st = f.state + ((int64_t)f.slots[b] * H + h) * (int64_t)Dk * Dv + c;
    __syncthreads();
    for (int d0 = group; d0 < Dk; d0 += groups * U) {
        Cols<V> s[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int d = d0 + u * groups;
#pragma unroll
            for (int e = 0; e < V; ++e) s[u].v[e] = 0.f;
            if (live && d < Dk && !fresh) s[u] = row_load<V>(st + (int64_t)d * Dv);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int d = d0 + u * groups;
            if (d >= Dk) break;
#pragma unroll
            for (int e = 0; e < V; ++e) {
                s[u].v[e] = decay * s[u].v[e] + ks[d] * v[e];
                o[e] += s[u].v[e] * qs[d];
            }
            if (live) row_store<V>(st + (int64_t)d * Dv, s[u]);
        }
    }
    if (live) {
#pragma unroll
        for (int e = 0; e < V; ++e) os[group * Dv + c + e] = o[e];
    }
    __syncthreads();
    for (int i = tid; i < Dv; i += 256) {
        float sum = 0.f;
        for (int j = 0; j < groups; ++j) sum += os[j * Dv + i];
        f.out[(int64_t)t * f.out_stride + (int64_t)h * Dv + i] = sum;
    }
}

template <typename T>
static void launch_single(const FixedDecayArgs& f, hipStream_t s) {
    const bool vec = f.Dv % 4 == 0;                              // (states start on 16 bytes, slots are whole rows)
    const int cols = vec ? f.Dv / 4 : f.Dv;
    int pieces = 1;
    while (pieces < cols) pieces *= 2;                           // at most 256
    const size_t lds = sizeof(float) * (2 * (size_t)f.Dk + (size_t)(256 / pieces) * f.Dv);
    const dim3 grid((unsigned)f.num_seqs, (unsigned)f.H), block(256);
    if (vec) hipLaunchKernelGGL((fixed_decay_single_kernel<T, 4>), grid, block, lds, s, f, pieces);
    else hipLaunchKernelGGL((fixed_decay_single_kernel<T, 1>), grid, block, lds, s, f, pieces);
}

struct FdPlan {
    int nseg, seg_len;
    int64_t ws_floats;
};

static bool fd_chunked(int Dk, int Dv, int dtype, int max_seqlen_q) {
    return dtype == NV_DTYPE_BF16 && Dk <= 128 && Dv <= 256 && max_seqlen_q > kFdFewRows;
}

// Segments so that the launch has about two workgroups per CU.  The sequences that count are the long ones: T rows make at most
// that many portions of the longest one's length.
static FdPlan fd_plan(int B, int64_t T, int H, int Dk, int Dv, int max_seqlen_q, int lead) {
    B -= lead;
    T -= lead;
    const int mq = std::max(1, max_seqlen_q);
    FdPlan p{1, (mq + kFdChunk - 1) / kFdChunk * kFdChunk, 0};
    const int64_t groups = std::max<int64_t>(1, std::min<int64_t>(B, (T + mq - 1) / mq)) * H * ((Dv + 63) / 64);
    if (B > 0 && groups < 256 && mq >= 512) {
        const int want = (int)std::min<int64_t>((512 + groups - 1) / groups, 16);
        p.nseg = std::max(1, std::min(want, mq / 256));
        p.seg_len = ((mq + p.nseg - 1) / p.nseg + kFdChunk - 1) / kFdChunk * kFdChunk;
        p.nseg = (mq + p.seg_len - 1) / p.seg_len;
    }
    if (p.nseg > 1) p.ws_floats = segment_places(T, p.seg_len) * H * Dk * Dv;
    return p;
}

template <int DKT>
static void launch_chunks(const FdParams& p, bool vec, hipStream_t s) {
    const size_t lds = sizeof(__bf16) * (2 * kFdChunk * (32 * DKT + 8) + kFdChunk * kFdVs) + sizeof(bf16x8) * 4 * 2 * 2 * 64 +
                       sizeof(float) * (kFdChunk + 1);
    const dim3 grid((unsigned)p.f.num_seqs, (unsigned)(p.f.H * ((p.f.Dv + 63) / 64)), (unsigned)p.nseg), block(256);
    if (!vec) {                                                  // rows of odd sizes: one plain form (the plan has one segment)
        hipLaunchKernelGGL((fixed_decay_chunk_kernel<DKT, kFdWhole, false>), grid, block, lds, s, p);
    } else if (p.nseg == 1) {
        hipLaunchKernelGGL((fixed_decay_chunk_kernel<DKT, kFdWhole, true>), grid, block, lds, s, p);
    } else {
        hipLaunchKernelGGL((fixed_decay_chunk_kernel<DKT, kFdSummary, true>), grid, block, lds, s, p);
        hipLaunchKernelGGL((fixed_decay_chunk_kernel<DKT, kFdFinal, true>), grid, block, lds, s, p);
    }
}

}  // namespace nv

extern "C" int64_t nv_fixed_decay_workspace_bytes(int num_seqs, int64_t T, int H, int Dk, int Dv, int max_seqlen_q,
                                                  int leading_singles, int dtype) {
    if (num_seqs <= 0 || T <= 0 || leading_singles < 0 || leading_singles > num_seqs || H <= 0 || Dk <= 0 || Dv <= 0 || !nv::fd_chunked(Dk, Dv, dtype, max_seqlen_q)) return 0;
    return nv::fd_plan(num_seqs, T, H, Dk, Dv, max_seqlen_q, leading_singles).ws_floats * (int64_t)sizeof(float);
}

extern "C" int nv_fixed_decay_memory(const void* q, const void* k, const void* v, int64_t q_stride, int64_t k_stride,
                                     int64_t v_stride, const float* decay, float* state, float* out, int64_t out_stride,
                                     const int32_t* cu_seqlens_q, const int32_t* cu_seqlens_k, const int32_t* state_slots,
                                     int num_seqs, int64_t T, int H, int Dk, int Dv, int max_seqlen_q, int leading_singles,
                                     int portions, int dtype,
                                     void* workspace, int64_t workspace_bytes, void* stream) {
    using namespace nv;
    NV_REQUIRE(num_seqs >= 0 && T >= 0 && H > 0 && Dk > 0 && Dv > 0 && max_seqlen_q >= 1 && leading_singles >= 0 &&
                   leading_singles <= num_seqs,
               NV_ERR_INVALID_ARG,
               "nv_fixed_decay_memory: bad sizes");
    if (num_seqs == 0 || T == 0) return NV_OK;
    NV_REQUIRE(q && k && v && decay && state && out && cu_seqlens_q && cu_seqlens_k && state_slots, NV_ERR_INVALID_ARG,
               "nv_fixed_decay_memory: null pointer");
    NV_REQUIRE(Dk <= 256 && Dv <= 256, NV_ERR_UNSUPPORTED, "nv_fixed_decay_memory: Dk=%d, Dv=%d exceed 256", Dk, Dv);
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_fixed_decay_memory: bad dtype");
    NV_REQUIRE((int64_t)H * ((Dv + 63) / 64) < 65536, NV_ERR_UNSUPPORTED, "nv_fixed_decay_memory: launch too large");
    hipStream_t s = (hipStream_t)stream;
    FdParams p{};
    p.f = FixedDecayArgs{q,          k,          v,          q_stride, k_stride, v_stride, decay, state, out,
                         out_stride, cu_seqlens_q, cu_seqlens_k, state_slots, num_seqs, H,        Dk,       Dv};
    const bool chunked = fd_chunked(Dk, Dv, dtype, max_seqlen_q);
    if (leading_singles > 0) {
        NV_REQUIRE((uintptr_t)state % 16 == 0, NV_ERR_INVALID_ARG, "nv_fixed_decay_memory: the state must start on 16 bytes");
        p.f.num_seqs = leading_singles;
        if (dtype == NV_DTYPE_BF16) launch_single<__bf16>(p.f, s);
        else launch_single<float>(p.f, s);
        const int rc = check_launch("nv_fixed_decay_memory (single tokens)");
        if (rc != NV_OK || leading_singles == num_seqs) return rc;
        p.f.num_seqs = num_seqs - leading_singles;               // (row numbers stay those of the step)
        p.f.cu_q += leading_singles;
        p.f.cu_k += leading_singles;
        p.f.slots += leading_singles;
    }
    if ((portions & (NV_PORTION_SINGLE | NV_PORTION_FEW)) || (!chunked && (portions & NV_PORTION_LONG))) {
        const int rc = launch_fixed_decay_rows(p.f, dtype, chunked ? kFdFewRows : 1 << 30, s);
        if (rc != NV_OK) return rc;
    }
    if (!chunked || !(portions & NV_PORTION_LONG)) return NV_OK;
    const FdPlan plan = fd_plan(num_seqs, T, H, Dk, Dv, max_seqlen_q, leading_singles);
    NV_REQUIRE(plan.ws_floats == 0 || (workspace && workspace_bytes >= plan.ws_floats * (int64_t)sizeof(float)), NV_ERR_WORKSPACE,
               "nv_fixed_decay_memory: workspace of %lld bytes, need %lld", (long long)workspace_bytes,
               (long long)(plan.ws_floats * (int64_t)sizeof(float)));
    const bool vec = Dk % 8 == 0 && Dv % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 && v_stride % 8 == 0 && out_stride % 4 == 0 &&
                     ((uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)out) % 16 == 0;
    p.nseg = vec ? plan.nseg : 1;
    p.seg_len = plan.seg_len;
    p.seg_state = (float*)workspace;
    if (Dk <= 32) launch_chunks<1>(p, vec, s);
    else if (Dk <= 64) launch_chunks<2>(p, vec, s);
    else if (Dk <= 96) launch_chunks<3>(p, vec, s);
    else launch_chunks<4>(p, vec, s);
    return check_launch("nv_fixed_decay_memory");
}
