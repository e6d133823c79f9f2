// Paged attention in latent space on the matrix cores: every query head of a sequence attends to ONE cached row per token
// whose first Dv columns are also the token's value (bf16, causal, fp32 softmax, an optional learned sink per head that
// joins the denominator only).
//
// With one key row for all heads the queries of a sequence are simply the rows (token, head) of a matrix
// [len_q * H, D], in the order the projection leaves them.  Both kernels work on wave tiles of 32 such rows:
//     S^T (keys x rows) = C Q^T       v_mfma_f32_32x32x16_bf16: A = cached rows from LDS, B = Q^T held in registers
//     O^T (Dv x rows)  += C^T P^T     A = the SAME rows of LDS read transposed (ds_read_b64_tr_b16), B = P^T straight from the
//                                     S^T accumulators
// so a cached row is fetched once, by LDS-DMA, and serves as key and value.  A lane holds half the scores of one row: the
// running maximum is per lane pair and raised only when a score exceeds it by 2^8, so the accumulators are seldom rescaled.
//
//   rows kernel    sequences with several tokens in the step: a workgroup of four waves takes 128 rows; key tiles of 64
//                  (32 for wide rows) are staged once for the four waves, double-buffered.
//   single kernel  sequences with one token: a workgroup takes up to 32 heads; its four waves take the key tiles of 32 in
//                  turn, each staging its own (no barrier in the loop), and join their states through LDS.
//
// When a launch would leave most of the chip idle the keys are cut into ranges; the ranges' unnormalised states go through
// a workspace and a second launch.
//
// LDS image of a tile: 8-row x 32-column subtiles of 512 bytes, the 16-byte chunk within a subtile row XOR-ed by bits 2..3
// of the row; conflict-free for the row reads and for the transposed reads.
#include <algorithm>
#include <type_traits>

#include "nv_common.h"
#include "../../include/nanovllm_hip_mixers.h"

namespace nv {

typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
typedef __attribute__((ext_vector_type(8))) short s16x8;

constexpr float kLatRunInit = -1.0e30f;        // finite initial running maximum (keeps exp2 NaN-free)
constexpr float kLatRaise = 8.0f;              // log2 units: weights stay below 2^8 between raises
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kLatRows = 32;                   // rows of a wave
constexpr int kLatStageRow = 144;              // bytes per row of the output staging area (128 + 16: spreads the banks)

struct LatentParams {
    const __bf16* q;             // [T, H, D]
    const __bf16* cache;         // [num_blocks, block_size, D]
    __bf16* out;                 // [T, H, Dv]
    float* part;                 // [T * H, nsplit, Dv + 2] when nsplit > 1
    const int *cu_q, *cu_k, *block_tables;
    const float* sink;
    int B, H, max_blocks, block_size, tiles_per_block;
    int64_t num_blocks;
    float scale_log2;
    int Dv, dv_groups;           // value columns, and how many workgroups share them (wide rows: the accumulators of all
                                 // columns beside the queries would not fit the registers)
    int row_tiles;               // rows kernel: 128-row tiles of the longest sequence
    int head_groups;             // single kernel: groups of 32 heads
    int nsplit, tiles_per_split;
};

__device__ __forceinline__ float lat_max_xor32(float x) {
    const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    return fmaxf(__uint_as_float(r[0]), __uint_as_float(r[1]));
}
__device__ __forceinline__ float lat_sum_xor32(float x) {
    const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x), __float_as_uint(x), false, false);
    return __uint_as_float(r[0]) + __uint_as_float(r[1]);
}

// byte offset of 16-byte chunk `ch` of row `row` in the image of a tile whose rows are 32 * D32 columns wide
template <int D32>
__device__ __forceinline__ int lat_off(int row, int ch) {
    return 512 * D32 * (row >> 3) + 512 * (ch >> 2) + 64 * (row & 7) + 16 * ((ch & 3) ^ ((row >> 2) & 3));
}

// One 1-KiB piece of a tile: lane l fills bytes 16 l .. of it.  Which (row, chunk) of the tile that is.
template <int D32>
__device__ __forceinline__ void lat_piece(int piece, int lane, int& row, int& ch) {
    const int sub = 2 * piece + (lane >> 5);
    row = 8 * (sub / D32) + ((lane & 31) >> 2);
    ch = 4 * (sub % D32) + ((lane & 3) ^ ((row >> 2) & 3));
}

// The state of one wave: 32 rows of queries against the keys it is shown.
template <int D32, int DV32, int KB>
struct LatentWave {
    bf16x8 qf[2 * D32];
    f32x16 oacc[DV32];
    float m_run, l_run;

    __device__ __forceinline__ void init(const __bf16* qrow, int h) {
#pragma unroll
        for (int s = 0; s < 2 * D32; ++s) qf[s] = *(const bf16x8*)(qrow + 16 * s + 8 * h);
#pragma unroll
        for (int d = 0; d < DV32; ++d)
#pragma unroll
            for (int i = 0; i < 16; ++i) oacc[d][i] = 0.f;
        m_run = kLatRunInit;
        l_run = 0.f;
    }

    // A tile of 32 KB keys at `lds`, the first of them key kt; the lane's row sees keys <= qpos (masked: some row of the wave
    // does not see all of the tile).  The wave accumulates the value columns from 32 dv0 on.
    __device__ __forceinline__ void step(const unsigned char* lds, int lane, int kt, int qpos, bool masked, float scale_log2,
                                         int dv0) {
        const int r = lane & 31, h = lane >> 5, i16 = lane & 15, g16 = (lane >> 4) & 1;
        f32x16 sacc[KB];
#pragma unroll
        for (int kb = 0; kb < KB; ++kb) {
#pragma unroll
            for (int i = 0; i < 16; ++i) sacc[kb][i] = 0.f;
#pragma unroll
            for (int s = 0; s < 2 * D32; ++s) {
                const bf16x8 a = *(const bf16x8*)(lds + lat_off<D32>(kb * 32 + r, 2 * s + h));
                sacc[kb] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, qf[s], sacc[kb], 0, 0, 0);
            }
        }
        // register i of block kb is key kt + 32 kb + (i & 3) + 8 (i >> 2) + 4 h
        if (masked) {
#pragma unroll
            for (int kb = 0; kb < KB; ++kb)
#pragma unroll
                for (int i = 0; i < 16; ++i) {
                    const int key = kt + kb * 32 + (i & 3) + 8 * (i >> 2) + 4 * h;
                    sacc[kb][i] = key <= qpos ? sacc[kb][i] : -INFINITY;
                }
        }
        float tmax = sacc[0][0];
#pragma unroll
        for (int kb = 0; kb < KB; ++kb)
#pragma unroll
            for (int i = 0; i < 16; ++i) tmax = fmaxf(tmax, sacc[kb][i]);
        tmax = lat_max_xor32(tmax) * scale_log2;                 // (scale > 0)
        if (!__all(tmax <= m_run + kLatRaise)) {                 // rare after the first tiles
            const float m_new = fmaxf(m_run, tmax);
            const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
            m_run = m_new;
            l_run *= alpha;
#pragma unroll
            for (int d = 0; d < DV32; ++d)
#pragma unroll
                for (int i = 0; i < 16; ++i) oacc[d][i] *= alpha;
        }
        float psum = 0.f;
#pragma unroll
        for (int kb = 0; kb < KB; ++kb)
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const float e = __builtin_amdgcn_exp2f(__builtin_fmaf(sacc[kb][i], scale_log2, -m_run));
                sacc[kb][i] = e;
                psum += e;
            }
        l_run += psum;
#pragma unroll
        for (int s = 0; s < 2 * KB; ++s) {
            const int kb = s >> 1, s2 = s & 1;
            bf16x8 pb;
#pragma unroll
            for (int j = 0; j < 8; ++j) pb[j] = (__bf16)sacc[kb][8 * s2 + j];
            // keys of element j: 32 kb + 16 s2 + 8 (j >> 2) + 4 h + (j & 3)
            const int row1 = kb * 32 + 16 * s2 + 4 * h + (i16 >> 2);
#pragma unroll
            for (int d = 0; d < DV32; ++d) {
                const int ch = d * 4 + 2 * g16 + ((i16 & 3) >> 1), sub = 8 * (i16 & 1);
                const s16x4 v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(lds + 512 * dv0 + lat_off<D32>(row1, ch) + sub));
                const s16x4 v2 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4*)(lds + 512 * dv0 + lat_off<D32>(row1 + 8, ch) + sub));
                s16x8 va;
                va[0] = v1[0]; va[1] = v1[1]; va[2] = v1[2]; va[3] = v1[3];
                va[4] = v2[0]; va[5] = v2[1]; va[6] = v2[2]; va[7] = v2[3];
                oacc[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, va), pb, oacc[d], 0, 0, 0);
            }
        }
    }
};

__device__ __forceinline__ void lat_dma(const unsigned char* src, unsigned char* dst) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                     (__attribute__((address_space(3))) void*)dst, 16, 0, 0);
}

// first byte of the tile that starts at key `kt` (tiles do not straddle blocks; table entries are clamped into the cache)
__device__ __forceinline__ const unsigned char* lat_tile_base(const LatentParams& p, int entry, int off, int row_bytes) {
    const int64_t last = p.num_blocks - 1;
    const int64_t phys = entry < 0 ? 0 : (entry > last ? last : entry);
    return (const unsigned char*)p.cache + (phys * p.block_size + off) * (int64_t)row_bytes;
}

// 1 / denominator of a finished row, with the sink in it, and the factor of the accumulators
__device__ __forceinline__ float lat_finish(float m, float l, const float* sink, int head) {
    float f = 1.f;
    if (sink != nullptr) {
        const float s2 = sink[head] * kLog2e, m2 = fmaxf(m, s2);
        f = __builtin_amdgcn_exp2f(m - m2);
        l = l * f + __builtin_amdgcn_exp2f(s2 - m2);
    }
    return f / l;
}

// ------------------------------------------------------------------------------------------------ several tokens
template <int D32, int DV32, int KB, int OCC>
__global__ __launch_bounds__(256, OCC) void attn_latent_rows_kernel(const LatentParams p) {
    constexpr int D = 32 * D32, KT = 32 * KB, kTile = KT * D * 2, kPieces = D32 * KB / 2;
    static_assert(D32 * KB % 2 == 0, "a wave stages whole pieces");
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];      // two tiles; the output staging area at the end
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 31, h = lane >> 5;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int split = blockIdx.y, dv0 = blockIdx.z * DV32, Dv = p.Dv;
    const int b = blockIdx.x % p.B, qt = p.row_tiles - 1 - blockIdx.x / p.B;     // the latest (heaviest) tiles first
    const int q_begin = p.cu_q[b], n_q = p.cu_q[b + 1] - q_begin, n_k = p.cu_k[b + 1] - p.cu_k[b];
    const int rows = n_q * p.H, row0 = qt * 4 * kLatRows;
    if (n_q <= 1 || row0 >= rows) return;                    // (single tokens belong to the other kernel)
    const int start = n_k - n_q;
    const int rw0 = row0 + wave * kLatRows;                  // the wave's first row
    const bool wave_live = rw0 < rows;
    const int my_row = min(rw0 + r, rows - 1);
    const int qpos = start + my_row / p.H;
    const int wave_first_pos = start + min(rw0, rows - 1) / p.H, wave_last_pos = start + min(rw0 + kLatRows - 1, rows - 1) / p.H;
    const int last_key = start + (min(row0 + 4 * kLatRows, rows) - 1) / p.H;
    const int t_begin = split * p.tiles_per_split, t_end = min(last_key / KT + 1, t_begin + p.tiles_per_split);

    LatentWave<D32, DV32, KB> w;
    w.init(p.q + ((int64_t)q_begin * p.H + my_row) * D, h);

    const int* table = p.block_tables + (int64_t)b * p.max_blocks;
    int dma_row[kPieces];
    uint32_t dma_off[kPieces];
#pragma unroll
    for (int i = 0; i < kPieces; ++i) {
        int ch;
        lat_piece<D32>(wave * kPieces + i, lane, dma_row[i], ch);
        dma_off[i] = (uint32_t)(dma_row[i] * (D * 2) + ch * 16);
    }
    auto stage = [&](int buf, int entry, int t) {
        const unsigned char* base = lat_tile_base(p, __builtin_amdgcn_readfirstlane(entry), (t % p.tiles_per_block) * KT, D * 2);
        const int last = n_k - 1 - t * KT;                   // rows behind the sequence's end re-read its last row
        unsigned char* dst = lds + buf * kTile + wave * kPieces * 1024;
#pragma unroll
        for (int i = 0; i < kPieces; ++i)
            lat_dma(base + (dma_off[i] - (uint32_t)(max(dma_row[i] - last, 0) * (D * 2))), dst + i * 1024);
    };
    int entry_next = 0;
    if (t_begin < t_end) stage(0, table[t_begin / p.tiles_per_block], t_begin);
    if (t_begin + 1 < t_end) entry_next = table[(t_begin + 1) / p.tiles_per_block];
    int buf = 0;
    for (int t = t_begin; t < t_end; ++t) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();                                     // tile t has landed for all, the other buffer is free
        if (t + 1 < t_end) stage(buf ^ 1, entry_next, t + 1);
        if (t + 2 < t_end) entry_next = table[(t + 2) / p.tiles_per_block];
        const int kt = t * KT;
        if (wave_live && kt <= wave_last_pos)                // (uniform per wave)
            w.step(lds + buf * kTile, lane, kt, qpos, kt + KT - 1 > wave_first_pos, p.scale_log2, dv0);
        buf ^= 1;
    }
    const float l_tot = lat_sum_xor32(w.l_run);
    __syncthreads();                                         // every wave is done reading tiles
    if (!wave_live) return;
    // Lane (r, h) holds columns 32 d + 8 (i >> 2) + 4 h + (i & 3) of row r: through the wave's staging area to 128-byte row
    // segments.
    unsigned char* stg = lds + wave * (kLatRows * kLatStageRow);
    const int rows_here = rows - rw0;
    const int64_t grow = (int64_t)q_begin * p.H + rw0;
    if (p.nsplit > 1) {
        float* dst = p.part + (grow * p.nsplit + split) * (Dv + 2);
        const int64_t ld = (int64_t)p.nsplit * (Dv + 2);
        if (dv0 == 0 && h == 0 && r < rows_here) {
            dst[r * ld + Dv] = w.m_run;
            dst[r * ld + Dv + 1] = l_tot;
        }
        if (t_begin >= t_end) return;                        // no keys in this range: l = 0 says so
#pragma unroll
        for (int d = 0; d < DV32; ++d) {
#pragma unroll
            for (int g = 0; g < 4; ++g)
                *(float4*)(stg + r * kLatStageRow + (8 * g + 4 * h) * 4) =
                    make_float4(w.oacc[d][4 * g], w.oacc[d][4 * g + 1], w.oacc[d][4 * g + 2], w.oacc[d][4 * g + 3]);
#pragma unroll
            for (int it = 0; it < 8; ++it) {                 // (states are 8-byte aligned)
                const int c = it * 64 + lane, rr = c >> 4;
                const float2 v = *(const float2*)(stg + rr * kLatStageRow + (c & 15) * 8);
                if (rr < rows_here) *(float2*)(dst + rr * ld + (dv0 + d) * 32 + (c & 15) * 2) = v;
            }
        }
        return;
    }
    const float inv = lat_finish(w.m_run, l_tot, p.sink, my_row % p.H);
    __bf16* dst = p.out + grow * Dv + dv0 * 32;
#pragma unroll
    for (int d0 = 0; d0 < DV32; d0 += 2) {
        constexpr int kMax = 2;
        const int nd = d0 + kMax <= DV32 ? kMax : 1;
#pragma unroll
        for (int dd = 0; dd < kMax; ++dd) {
            if (d0 + dd >= DV32) continue;
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const f32x16& o = w.oacc[d0 + dd < DV32 ? d0 + dd : 0];
                *(uint2*)(stg + r * kLatStageRow + (dd * 32 + 8 * g + 4 * h) * 2) =
                    make_uint2(pack_bf16(o[4 * g] * inv, o[4 * g + 1] * inv), pack_bf16(o[4 * g + 2] * inv, o[4 * g + 3] * inv));
            }
        }
        const int per = 4 * nd;                              // 16-byte pieces per row
        for (int c = lane; c < kLatRows * per; c += 64) {
            const int rr = c / per, pc = c % per;
            const uint4 v = *(const uint4*)(stg + rr * kLatStageRow + pc * 16);
            if (rr < rows_here) *(uint4*)(dst + (int64_t)rr * Dv + d0 * 32 + pc * 8) = v;
        }
    }
}

// ------------------------------------------------------------------------------------------------ one token
template <int D32, int DV32, int NBUF, int OCC>
__global__ __launch_bounds__(256, OCC) void attn_latent_single_kernel(const LatentParams p) {
    constexpr int D = 32 * D32, Dw = 32 * DV32, KT = 32, kTile = KT * D * 2, kPieces = 2 * D32;
    extern __shared__ __attribute__((aligned(16))) unsigned char lds[];      // [4 waves][NBUF tiles], then [4][32] (m, l)
    const int tid = threadIdx.x, lane = tid & 63, r = lane & 31, h = lane >> 5;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int b = blockIdx.x, hg = blockIdx.z / p.dv_groups, split = blockIdx.y, Dv = p.Dv;
    const int dv0 = (blockIdx.z % p.dv_groups) * DV32;
    const int t0 = p.cu_q[b];
    if (p.cu_q[b + 1] - t0 != 1) return;                     // longer portions belong to the other kernel
    const int n_k = p.cu_k[b + 1] - p.cu_k[b];
    const int head0 = hg * kLatRows, heads = min(kLatRows, p.H - head0);
    const int t_begin = split * p.tiles_per_split, t_end = min((n_k + KT - 1) / KT, t_begin + p.tiles_per_split);

    const int* table = p.block_tables + (int64_t)b * p.max_blocks;
    unsigned char* mine = lds + wave * (NBUF * kTile);
    int row0, ch0;                                           // piece i is piece 0 shifted by 2 i subtiles
    lat_piece<D32>(0, lane, row0, ch0);
    auto stage = [&](int buf, int t) {
        const int entry = __builtin_amdgcn_readfirstlane(table[t / p.tiles_per_block]);
        const unsigned char* base = lat_tile_base(p, entry, (t % p.tiles_per_block) * KT, D * 2);
        const int last = n_k - 1 - t * KT;
#pragma unroll
        for (int i = 0; i < kPieces; ++i) {
            int row, ch;
            lat_piece<D32>(i, lane, row, ch);
            lat_dma(base + (uint32_t)(min(row, last) * (D * 2) + ch * 16), mine + buf * kTile + i * 1024);
        }
    };
    LatentWave<D32, DV32, 1> w;
    int t = t_begin + wave, buf = 0;
    if (t < t_end) stage(0, t);
    w.init(p.q + ((int64_t)t0 * p.H + head0 + min(r, heads - 1)) * D, h);
    for (; t < t_end; t += 4) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");     // this wave's own tile has landed
        if (NBUF == 2 && t + 4 < t_end) stage(buf ^ 1, t + 4);
        w.step(mine + buf * kTile, lane, t * KT, n_k - 1, t * KT + KT > n_k, p.scale_log2, dv0);
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // its reads are done before the buffer is filled again
        if (NBUF == 1 && t + 4 < t_end) stage(0, t + 4);
        if (NBUF == 2) buf ^= 1;
    }
    // ---- join the four waves: maxima and denominators, then the accumulators, 16 rows at a time through the tile areas ----
    const float l_tot = lat_sum_xor32(w.l_run);
    float* ml = (float*)(lds + 4 * NBUF * kTile);
    if (h == 0) {
        ml[(wave * kLatRows + r) * 2] = w.m_run;
        ml[(wave * kLatRows + r) * 2 + 1] = l_tot;
    }
    __syncthreads();
    float m_all = kLatRunInit;
#pragma unroll
    for (int i = 0; i < 4; ++i) m_all = fmaxf(m_all, ml[(i * kLatRows + r) * 2]);
    const float f = __builtin_amdgcn_exp2f(w.m_run - m_all);
    float* accs = (float*)lds;                               // [4 waves][16 rows][Dw]: at most the tile areas (Dw <= D)
    constexpr int kArea = NBUF * kTile / 4;                  // floats from one wave's area to the next
    static_assert(16 * Dw * 4 <= NBUF * kTile, "the join area fits a wave's tiles");
    for (int half = 0; half < 2 && half * 16 < heads; ++half) {
        __syncthreads();
        if ((r >> 4) == half) {
#pragma unroll
            for (int d = 0; d < DV32; ++d)
#pragma unroll
                for (int g = 0; g < 4; ++g)
                    *(float4*)(accs + wave * kArea + (r & 15) * Dw + d * 32 + 8 * g + 4 * h) =
                        make_float4(w.oacc[d][4 * g] * f, w.oacc[d][4 * g + 1] * f, w.oacc[d][4 * g + 2] * f, w.oacc[d][4 * g + 3] * f);
        }
        __syncthreads();
        const int n_rows = min(16, heads - half * 16);
        for (int i = tid; i < n_rows * (Dw / 4); i += 256) {
            const int row = i / (Dw / 4), c = (i % (Dw / 4)) * 4, hr = half * 16 + row;
            float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int x = 0; x < 4; ++x) {
                const float4 a = *(const float4*)(accs + x * kArea + row * Dw + c);
                s.x += a.x; s.y += a.y; s.z += a.z; s.w += a.w;
            }
            float m = kLatRunInit, l = 0.f;
#pragma unroll
            for (int x = 0; x < 4; ++x) m = fmaxf(m, ml[(x * kLatRows + hr) * 2]);
#pragma unroll
            for (int x = 0; x < 4; ++x) l += ml[(x * kLatRows + hr) * 2 + 1] * __builtin_amdgcn_exp2f(ml[(x * kLatRows + hr) * 2] - m);
            const int64_t grow = (int64_t)t0 * p.H + head0 + hr;
            if (p.nsplit > 1) {
                float* dst = p.part + (grow * p.nsplit + split) * (Dv + 2);
                *(float2*)(dst + dv0 * 32 + c) = make_float2(s.x, s.y);
                *(float2*)(dst + dv0 * 32 + c + 2) = make_float2(s.z, s.w);
                if (dv0 == 0 && c == 0) {
                    dst[Dv] = m;
                    dst[Dv + 1] = l;
                }
            } else {
                const float inv = lat_finish(m, l, p.sink, head0 + hr);
                *(uint2*)(p.out + grow * Dw + c) = make_uint2(pack_bf16(s.x * inv, s.y * inv), pack_bf16(s.z * inv, s.w * inv));
            }
        }
    }
}

// Joins the key ranges of a row (token, head): one wave per row.  only: 1 = rows of single-token sequences, 2 = the others.
__global__ __launch_bounds__(256) void attn_latent_merge_kernel(const LatentParams p, int Dv, int64_t total_rows, int only) {
    const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    if (row >= total_rows) return;
    const int lane = threadIdx.x & 63;
    const int t = (int)(row / p.H);
    int lo = 0, hi = p.B;
    while (hi - lo > 1) {
        const int mid = (lo + hi) >> 1;
        if (p.cu_q[mid] <= t) lo = mid; else hi = mid;
    }
    if ((p.cu_q[lo + 1] - p.cu_q[lo] == 1) != (only == 1)) return;
    const float* base = p.part + row * p.nsplit * (Dv + 2);
    // lane s holds range s (at most 32 of them): its share of the denominator and the factor of its accumulators
    float m = kLatRunInit, l = 0.f;
    if (lane < p.nsplit) {
        const float2 ml = *(const float2*)(base + lane * (Dv + 2) + Dv);
        l = ml.y;
        if (l > 0.f) m = ml.x;
    }
    float m_all = m;
#pragma unroll
    for (int o = 16; o > 0; o >>= 1) m_all = fmaxf(m_all, __shfl_xor(m_all, o));
    m_all = __shfl(m_all, 0);                                // (lanes 32.. hold nothing)
    const float f = l > 0.f ? __builtin_amdgcn_exp2f(m - m_all) : 0.f;      // 0: the range had no keys, its state is not read
    const float inv = lat_finish(m_all, wave_sum(l * f), p.sink, (int)(row % p.H));
    for (int c = 2 * lane; c < Dv; c += 128) {               // (Dv is even)
        float ox = 0.f, oy = 0.f;
#pragma unroll 8
        for (int s = 0; s < p.nsplit; ++s) {
            const float fs = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(f), s));   // (some lanes may sit this out)
            const float2 v = *(const float2*)(base + s * (Dv + 2) + c);
            ox += fs > 0.f ? fs * v.x : 0.f;
            oy += fs > 0.f ? fs * v.y : 0.f;
        }
        *(uint32_t*)(p.out + row * Dv + c) = pack_bf16(ox * inv, oy * inv);
    }
}

// ------------------------------------------------------------------------------------------------ launch plan
static bool latent_built(int D, int Dv) {
    if (D % 32 || Dv % 32) return false;
    const int d = D / 32, v = Dv / 32;
    if (d == v) return (d >= 1 && d <= 8) || d == 10 || d == 12 || d == 16;
    return (d == 5 && v == 4) || (d == 6 && v == 4) || (d == 8 && v == 6) || (d == 10 && v == 8) || (d == 18 && v == 16);
}
static int latent_tile_keys(int D) { return D <= 256 ? 64 : 32; }

struct LatentPlan {
    int nsplit, tiles_per_split;
};
// Key ranges: enough workgroups for the chip (a few per CU), not fewer than `min_tiles` tiles each.
static LatentPlan latent_plan(int64_t wgs, int max_k, int tile, int64_t want, int min_tiles) {
    const int tiles = std::max(1, (max_k + tile - 1) / tile);
    int64_t n = wgs > 0 ? (want + wgs - 1) / wgs : 1;
    n = std::max<int64_t>(1, std::min<int64_t>({n, (int64_t)tiles / min_tiles, (int64_t)32}));
    const int per = (int)((tiles + n - 1) / n);
    return {(tiles + per - 1) / per, per};
}
static LatentPlan latent_rows_plan(int B, int H, int max_q, int max_k, int D) {
    return latent_plan((int64_t)B * (((int64_t)max_q * H + 127) / 128), max_k, latent_tile_keys(D), 384, 8);
}
static LatentPlan latent_single_plan(int B, int H, int max_k) {
    return latent_plan((int64_t)B * ((H + 31) / 32), max_k, 32, 512, 8);
}

template <int D32, int DV32>
static int launch_latent_rows(LatentParams p, int max_q, int max_k, hipStream_t s) {
    constexpr int KB = D32 <= 8 ? 2 : 1, OCC = D32 <= 5 || (D32 == 6 && DV32 == 4) ? 2 : 1, D = 32 * D32;
    constexpr size_t rows_lds = (size_t)std::max(2 * 32 * KB * D * 2, 4 * kLatRows * kLatStageRow);
    static_assert(rows_lds <= 160 * 1024, "LDS of a compute unit");
    const void* fn = (const void*)attn_latent_rows_kernel<D32, DV32, KB, OCC>;
    static bool raised = rows_lds <= 64 * 1024;              // beyond the default limit of dynamic LDS: raise it once
    if (!raised) {
        if (hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)rows_lds) != hipSuccess) return NV_ERR_LAUNCH;
        raised = true;
    }
    const LatentPlan plan = latent_rows_plan(p.B, p.H, max_q, max_k, D);
    p.nsplit = plan.nsplit;
    p.tiles_per_split = plan.tiles_per_split;
    p.row_tiles = (int)(((int64_t)max_q * p.H + 127) / 128);
    p.tiles_per_block = p.block_size / (32 * KB);
    p.dv_groups = p.Dv / (32 * DV32);
    hipLaunchKernelGGL((attn_latent_rows_kernel<D32, DV32, KB, OCC>),
                       dim3((unsigned)(p.B * p.row_tiles), (unsigned)p.nsplit, (unsigned)p.dv_groups), dim3(256), rows_lds, s, p);
    return check_launch("nv_attn_latent_paged (rows kernel)");
}
template <int D32, int DV32>
static int launch_latent_single(LatentParams p, int max_k, hipStream_t s) {
    constexpr int OCC = D32 <= 6 ? 2 : 1, NBUF = D32 <= 5 ? 2 : 1, D = 32 * D32;
    constexpr size_t single_lds = (size_t)4 * NBUF * 32 * D * 2 + 4 * kLatRows * 8;
    static_assert(single_lds <= 160 * 1024, "LDS of a compute unit");
    const void* fn = (const void*)attn_latent_single_kernel<D32, DV32, NBUF, OCC>;
    static bool raised = single_lds <= 64 * 1024;              // beyond the default limit of dynamic LDS: raise it once
    if (!raised) {
        if (hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)single_lds) != hipSuccess) return NV_ERR_LAUNCH;
        raised = true;
    }
    const LatentPlan plan = latent_single_plan(p.B, p.H, max_k);
    p.nsplit = plan.nsplit;
    p.tiles_per_split = plan.tiles_per_split;
    p.head_groups = (p.H + 31) / 32;
    p.dv_groups = p.Dv / (32 * DV32);
    p.tiles_per_block = p.block_size / 32;
    hipLaunchKernelGGL((attn_latent_single_kernel<D32, DV32, NBUF, OCC>), dim3((unsigned)p.B, (unsigned)p.nsplit, (unsigned)(p.head_groups * p.dv_groups)),
                       dim3(256), single_lds, s, p);
    return check_launch("nv_attn_latent_paged (single kernel)");
}

}  // namespace nv

extern "C" int nv_attn_latent_ok(int D, int Dv, int block_size) {
    return nv::latent_built(D, Dv) && block_size > 0 && block_size % 64 == 0 ? 1 : 0;
}

extern "C" int64_t nv_attn_latent_workspace_bytes(int num_seqs, int64_t T, int H, int D, int Dv, int max_seqlen_q, int max_seqlen_k) {
    using namespace nv;
    if (num_seqs <= 0 || T <= 0 || H <= 0 || Dv <= 0 || max_seqlen_k <= 0) return 0;
    int n = latent_single_plan(num_seqs, H, max_seqlen_k).nsplit;
    if (max_seqlen_q > 1) n = std::max(n, latent_rows_plan(num_seqs, H, max_seqlen_q, max_seqlen_k, D).nsplit);
    return n > 1 ? T * H * n * (int64_t)(Dv + 2) * (int64_t)sizeof(float) : 0;
}

extern "C" int nv_attn_latent_paged(const void* q, const void* cache, void* out, const int32_t* cu_seqlens_q,
                                    const int32_t* cu_seqlens_k, const int32_t* block_tables, int num_seqs,
                                    int max_blocks_per_seq, int64_t T, int H, int D, int Dv, int64_t num_blocks, int block_size,
                                    float scale, const float* sink, int max_seqlen_q, int max_seqlen_k, int single_rows,
                                    void* workspace, int64_t workspace_bytes, void* stream) {
    using namespace nv;
    NV_REQUIRE(num_seqs >= 0 && T >= 0 && H > 0 && num_blocks > 0 && max_blocks_per_seq > 0, NV_ERR_INVALID_ARG,
               "nv_attn_latent_paged: bad sizes");
    NV_REQUIRE(nv_attn_latent_ok(D, Dv, block_size), NV_ERR_UNSUPPORTED,
               "nv_attn_latent_paged: no kernel for rows of %d, values of %d, blocks of %d", D, Dv, block_size);
    NV_REQUIRE(scale > 0.f, NV_ERR_UNSUPPORTED, "nv_attn_latent_paged: the scale must be positive");
    if (T == 0 || num_seqs == 0) return NV_OK;
    NV_REQUIRE(q && cache && out && cu_seqlens_q && cu_seqlens_k && block_tables, NV_ERR_INVALID_ARG,
               "nv_attn_latent_paged: null pointer");
    NV_REQUIRE(max_seqlen_q > 0 && max_seqlen_k > 0, NV_ERR_INVALID_ARG, "nv_attn_latent_paged: the longest lengths must be given");
    NV_REQUIRE(((uintptr_t)q | (uintptr_t)cache | (uintptr_t)out) % 16 == 0, NV_ERR_INVALID_ARG,
               "nv_attn_latent_paged: pointers must be 16-byte aligned");
    NV_REQUIRE(T * H < (1LL << 31) && num_seqs < 65536 * 16 && (int64_t)num_seqs * (((int64_t)max_seqlen_q * H + 127) / 128) < (1LL << 31) &&
                   num_blocks < (1LL << 31),
               NV_ERR_UNSUPPORTED, "nv_attn_latent_paged: launch too large");
    const int64_t need = nv_attn_latent_workspace_bytes(num_seqs, T, H, D, Dv, max_seqlen_q, max_seqlen_k);
    NV_REQUIRE(need == 0 || (workspace && workspace_bytes >= need && (uintptr_t)workspace % 16 == 0), NV_ERR_WORKSPACE,
               "nv_attn_latent_paged: workspace of %lld bytes, need %lld", (long long)workspace_bytes, (long long)need);
    const bool several = max_seqlen_q > 1, singles = single_rows != 0 || !several;
    LatentParams p{};
    p.q = (const __bf16*)q;
    p.cache = (const __bf16*)cache;
    p.out = (__bf16*)out;
    p.part = (float*)workspace;
    p.cu_q = cu_seqlens_q;
    p.cu_k = cu_seqlens_k;
    p.block_tables = block_tables;
    p.sink = sink;
    p.B = num_seqs;
    p.H = H;
    p.max_blocks = max_blocks_per_seq;
    p.block_size = block_size;
    p.num_blocks = num_blocks;
    p.scale_log2 = scale * kLog2e;
    p.Dv = Dv;
    hipStream_t s = (hipStream_t)stream;
    const auto merge = [&](const LatentPlan& plan, int only) {
        if (plan.nsplit <= 1) return (int)NV_OK;
        p.nsplit = plan.nsplit;
        hipLaunchKernelGGL(attn_latent_merge_kernel, dim3((unsigned)((T * H + 3) / 4)), dim3(256), 0, s, p, Dv, T * H, only);
        return check_launch("nv_attn_latent_paged (merge)");
    };
    int rc = NV_ERR_UNSUPPORTED;
    // row columns / 32, value columns / 32, value columns / 32 per workgroup
#define NV_LAT_ALL(X)                                                                                                      \
    X(1, 1, 1) X(2, 2, 2) X(3, 3, 3) X(4, 4, 4) X(5, 5, 5) X(6, 6, 6) X(7, 7, 7) X(8, 8, 8) X(10, 10, 5) X(12, 12, 6) X(16, 16, 8) \
        X(5, 4, 4) X(6, 4, 4) X(8, 6, 6) X(10, 8, 8) X(18, 16, 8)
    if (several) {
        switch (D / 32 * 100 + Dv / 32) {
#define NV_LAT_CASE(A, V, W) case A * 100 + V: rc = launch_latent_rows<A, W>(p, max_seqlen_q, max_seqlen_k, s); break;
            NV_LAT_ALL(NV_LAT_CASE)
#undef NV_LAT_CASE
        }
        if (rc == NV_OK) rc = merge(latent_rows_plan(num_seqs, H, max_seqlen_q, max_seqlen_k, D), 2);
        NV_REQUIRE(rc == NV_OK, rc, "nv_attn_latent_paged: the rows kernel could not be launched");
    }
    if (singles) {
        switch (D / 32 * 100 + Dv / 32) {
#define NV_LAT_CASE(A, V, W) case A * 100 + V: rc = launch_latent_single<A, W>(p, max_seqlen_k, s); break;
            NV_LAT_ALL(NV_LAT_CASE)
#undef NV_LAT_CASE
        }
        if (rc == NV_OK) rc = merge(latent_single_plan(num_seqs, H, max_seqlen_k), 1);
        NV_REQUIRE(rc == NV_OK, rc, "nv_attn_latent_paged: the single kernel could not be launched");
    }
    return NV_OK;
}
