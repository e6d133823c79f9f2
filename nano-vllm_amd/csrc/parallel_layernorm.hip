// An fp32 residual stream that every layer reads through TWO layer norms with biases (one per parallel sublayer), fed by
// token and position tables and by sublayers of which one is a mixture of experts.
//
// nv_embed_positions         x[t] = embed[id_t] + pos[position_t] in fp32.
// nv_stream_layernorm_pair   per row, in place on the fp32 stream r:
//                                r <- r + a1 + a2 + sum_j p_j + (sum of the weights of the choices without a product) * h
//                            with a1, a2 in the matmul dtype (each may be absent), p_j the fp32 outputs of the chosen
//                            experts, already weighted.  Choice j of a row is an expert with a product when its id is
//                            below `experts`; the others hand the row h (what the experts read) through, times their
//                            weight, and their p_j is not read.
//                                y1 <- LN(r) * w1 + b1                 in the matmul dtype
//                                y2 <- LN(r) * w2 + b2                 in the matmul dtype and / or fp32
//                            LN(r) = (r - mean) / sqrt(mean((r - mean)^2) + eps) once for both; each output may be absent.
// nv_silu_and_mul_rows       y = silu(gate) * up for rows [gate | up] of any even length, bf16 or fp32.
//
// One workgroup of 256 threads per row.  A thread keeps its columns in registers (NI pieces of V columns, every loop of
// compile-time length, so that all loads of a source are in flight at once); the mean, then the squared deviations are
// reduced through the four waves.
#include "row_pieces.h"
#include "../../include/nanovllm_hip_mixers.h"

namespace nv {

constexpr int kPlThreads = 256;

__device__ __forceinline__ float pl_block_sum(float x, float* red) {
    x = wave_sum(x);
    __syncthreads();                       // red may still be read from the previous reduction
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

template <typename T>
__global__ __launch_bounds__(256) void embed_positions_kernel(const int64_t* __restrict__ ids, const int64_t* __restrict__ positions,
                                                              const T* __restrict__ embed, const T* __restrict__ pos,
                                                              float* __restrict__ x, int cols, int64_t vocab,
                                                              int64_t max_positions) {
    const int64_t t = blockIdx.x;
    const int64_t id = ids[t], p = positions[t];
    const T* er = embed + (id < 0 ? 0 : id < vocab ? id : vocab - 1) * cols;                  // (never outside the tables)
    const T* pr = pos + (p < 0 ? 0 : p < max_positions ? p : max_positions - 1) * cols;
    for (int c = threadIdx.x; c < cols; c += 256) x[t * cols + c] = (float)er[c] + (float)pr[c];
}

template <typename T, int V, int NI>
__global__ __launch_bounds__(kPlThreads) void stream_layernorm_pair_kernel(
    float* __restrict__ resid, const T* __restrict__ add1, int64_t add1_stride, const T* __restrict__ add2,
    int64_t add2_stride, const float* __restrict__ parts, const int* __restrict__ ids, const float* __restrict__ weights,
    int n_parts, int experts, const T* __restrict__ through, int64_t through_stride, const float* __restrict__ w1,
    const float* __restrict__ b1, const float* __restrict__ w2, const float* __restrict__ b2, float eps,
    T* __restrict__ y1, T* __restrict__ y2, float* __restrict__ y2_f32, int cols) {
    __shared__ float red[kPlThreads / 64];
    const int64_t r = blockIdx.x;
    const int tid = threadIdx.x;
    float* rrow = resid + r * cols;
    Cols<V> v[NI];
    bool live[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        const int c = (tid + kPlThreads * i) * V;
        live[i] = c < cols;                        // (V divides cols)
        if (live[i]) v[i] = row_load<V>(rrow + c);
        else
#pragma unroll
            for (int e = 0; e < V; ++e) v[i].v[e] = 0.f;
    }
    Cols<V> s[NI];
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < V; ++e) s[i].v[e] = 0.f;
    const auto gather = [&](const auto* row, float g) {
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            if (!live[i]) continue;
            const Cols<V> a = row_load<V>(row + (tid + kPlThreads * i) * V);
#pragma unroll
            for (int e = 0; e < V; ++e) s[i].v[e] += g * a.v[e];
        }
    };
    bool changed = false;
    if (add1 != nullptr) { gather(add1 + r * add1_stride, 1.0f); changed = true; }
    if (add2 != nullptr) { gather(add2 + r * add2_stride, 1.0f); changed = true; }
    if (n_parts > 0) {
        float through_w = 0.f;
        changed = true;
        for (int j = 0; j < n_parts; ++j) {        // (the ids of a row are uniform over the workgroup)
            if (ids == nullptr || ids[r * n_parts + j] < experts) gather(parts + (r * n_parts + j) * cols, 1.0f);
            else through_w += weights[r * n_parts + j];
        }
        if (through != nullptr && through_w != 0.f) gather(through + r * through_stride, through_w);
    }
    if (changed) {
#pragma unroll
        for (int i = 0; i < NI; ++i) {
#pragma unroll
            for (int e = 0; e < V; ++e) v[i].v[e] += s[i].v[e];
            if (live[i]) row_store<V>(rrow + (tid + kPlThreads * i) * V, v[i]);
        }
    }
    if (w1 == nullptr && w2 == nullptr) return;
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int e = 0; e < V; ++e) sum += v[i].v[e];          // (columns past the end are zero)
    const float mean = pl_block_sum(sum, red) / (float)cols;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
        if (!live[i]) continue;
#pragma unroll
        for (int e = 0; e < V; ++e) {
            v[i].v[e] -= mean;
            ss += v[i].v[e] * v[i].v[e];
        }
    }
    const float rstd = 1.0f / sqrtf(pl_block_sum(ss, red) / (float)cols + eps);
    if (w1 != nullptr) {
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            if (!live[i]) continue;
            const int c = (tid + kPlThreads * i) * V;
            const Cols<V> w = row_load<V>(w1 + c), b = row_load<V>(b1 + c);
            Cols<V> o;
#pragma unroll
            for (int e = 0; e < V; ++e) o.v[e] = v[i].v[e] * rstd * w.v[e] + b.v[e];
            row_store<V>(y1 + r * cols + c, o);
        }
    }
    if (w2 != nullptr) {
#pragma unroll
        for (int i = 0; i < NI; ++i) {
            if (!live[i]) continue;
            const int c = (tid + kPlThreads * i) * V;
            const Cols<V> w = row_load<V>(w2 + c), b = row_load<V>(b2 + c);
            Cols<V> o;
#pragma unroll
            for (int e = 0; e < V; ++e) o.v[e] = v[i].v[e] * rstd * w.v[e] + b.v[e];
            if (y2 != nullptr) row_store<V>(y2 + r * cols + c, o);
            if (y2_f32 != nullptr) row_store<V>(y2_f32 + r * cols + c, o);
        }
    }
}

template <typename T, int V>
__global__ __launch_bounds__(256) void silu_and_mul_rows_kernel(const T* __restrict__ x, int64_t x_stride, T* __restrict__ y,
                                                                int inter, int pieces, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const int64_t r = i / pieces;
    const int c = (int)(i - r * pieces) * V;
    const Cols<V> g = row_load<V>(x + r * x_stride + c), u = row_load<V>(x + r * x_stride + inter + c);
    Cols<V> o;
#pragma unroll
    for (int e = 0; e < V; ++e) o.v[e] = g.v[e] / (1.0f + expf(-g.v[e])) * u.v[e];
    row_store<V>(y + r * inter + c, o);
}

struct PairArgs {
    float* resid;
    const void *add1, *add2, *through;
    int64_t add1_stride, add2_stride, through_stride;
    const float* parts;
    const int* ids;
    const float* weights;
    int n_parts, experts;
    const float *w1, *b1, *w2, *b2;
    float eps;
    void *y1, *y2;
    float* y2_f32;
    int64_t rows;
    int cols;
};

template <typename T>
static bool launch_pair(const PairArgs& a, bool vec, hipStream_t s) {
    const int V = vec ? 4 : 1, per_thread = (a.cols + kPlThreads * V - 1) / (kPlThreads * V);
#define NV_PAIR(VV, N)                                                                                                       \
    hipLaunchKernelGGL((stream_layernorm_pair_kernel<T, VV, N>), dim3((unsigned)a.rows), dim3(kPlThreads), 0, s, a.resid,     \
                       (const T*)a.add1, a.add1_stride, (const T*)a.add2, a.add2_stride, a.parts, a.ids, a.weights, a.n_parts, \
                       a.experts, (const T*)a.through, a.through_stride, a.w1, a.b1, a.w2, a.b2, a.eps, (T*)a.y1, (T*)a.y2,   \
                       a.y2_f32, a.cols)
    if (vec) {
        if (per_thread <= 1) NV_PAIR(4, 1);
        else if (per_thread <= 2) NV_PAIR(4, 2);
        else if (per_thread <= 4) NV_PAIR(4, 4);
        else if (per_thread <= 8) NV_PAIR(4, 8);
        else if (per_thread <= 16) NV_PAIR(4, 16);
        else return false;
    } else {
        if (per_thread <= 4) NV_PAIR(1, 4);
        else if (per_thread <= 16) NV_PAIR(1, 16);
        else if (per_thread <= 64) NV_PAIR(1, 64);
        else return false;
    }
#undef NV_PAIR
    return true;
}

}  // namespace nv

extern "C" int nv_embed_positions(const int64_t* ids, const int64_t* positions, const void* embed, const void* pos, float* x,
                                  int dtype, int64_t T, int cols, int64_t vocab, int64_t max_positions, void* stream) {
    using namespace nv;
    NV_REQUIRE(T >= 0 && cols > 0 && vocab > 0 && max_positions > 0, NV_ERR_INVALID_ARG, "nv_embed_positions: bad sizes");
    if (T == 0) return NV_OK;
    NV_REQUIRE(ids && positions && embed && pos && x, NV_ERR_INVALID_ARG, "nv_embed_positions: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_embed_positions: bad dtype");
    NV_REQUIRE(T < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_embed_positions: launch too large");
    if (dtype == NV_DTYPE_BF16)
        hipLaunchKernelGGL(embed_positions_kernel<__bf16>, dim3((unsigned)T), dim3(256), 0, (hipStream_t)stream, ids, positions,
                           (const __bf16*)embed, (const __bf16*)pos, x, cols, vocab, max_positions);
    else
        hipLaunchKernelGGL(embed_positions_kernel<float>, dim3((unsigned)T), dim3(256), 0, (hipStream_t)stream, ids, positions,
                           (const float*)embed, (const float*)pos, x, cols, vocab, max_positions);
    return check_launch("nv_embed_positions");
}

extern "C" int nv_stream_layernorm_pair(float* resid, const void* add1, int64_t add1_stride, const void* add2,
                                        int64_t add2_stride, const float* parts, const int32_t* ids, const float* weights,
                                        int n_parts, int experts, const void* through, int64_t through_stride,
                                        const float* w1, const float* b1, const float* w2, const float* b2, float eps,
                                        void* y1, void* y2, float* y2_f32, int dtype, int64_t rows, int cols, void* stream) {
    using namespace nv;
    NV_REQUIRE(rows >= 0 && cols > 0 && cols <= 16384, NV_ERR_INVALID_ARG, "nv_stream_layernorm_pair: bad sizes");
    if (rows == 0) return NV_OK;
    NV_REQUIRE(resid, NV_ERR_INVALID_ARG, "nv_stream_layernorm_pair: null stream");
    NV_REQUIRE(!parts || n_parts > 0, NV_ERR_INVALID_ARG, "nv_stream_layernorm_pair: parts without a count");
    NV_REQUIRE(!ids || (parts && weights), NV_ERR_INVALID_ARG, "nv_stream_layernorm_pair: ids go with parts and their weights");
    NV_REQUIRE(!through || ids, NV_ERR_INVALID_ARG, "nv_stream_layernorm_pair: a handed-through row needs the choices");
    NV_REQUIRE((!w1 || (b1 && y1)) && (!w2 || (b2 && (y2 || y2_f32))), NV_ERR_INVALID_ARG,
               "nv_stream_layernorm_pair: a norm needs its bias and an output");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_stream_layernorm_pair: bad dtype");
    NV_REQUIRE(rows < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_stream_layernorm_pair: launch too large");
    const PairArgs a{resid, add1, add2, through, add1_stride, add2_stride, through_stride, parts, ids, weights,
                     parts ? n_parts : 0, experts, w1, b1, w2, b2, eps, y1, y2, y2_f32, rows, cols};
    const bool bf = dtype == NV_DTYPE_BF16;
    const uintptr_t f32s = (uintptr_t)resid | (uintptr_t)parts | (uintptr_t)w1 | (uintptr_t)b1 | (uintptr_t)w2 |
                           (uintptr_t)b2 | (uintptr_t)y2_f32;
    const uintptr_t acts = (uintptr_t)add1 | (uintptr_t)add2 | (uintptr_t)through | (uintptr_t)y1 | (uintptr_t)y2;
    const bool strides = (!add1 || add1_stride % 4 == 0) && (!add2 || add2_stride % 4 == 0) && (!through || through_stride % 4 == 0);
    const bool vec = cols % 4 == 0 && strides && f32s % 16 == 0 && acts % (bf ? 8 : 16) == 0;
    const bool ok = bf ? launch_pair<__bf16>(a, vec, (hipStream_t)stream) : launch_pair<float>(a, vec, (hipStream_t)stream);
    NV_REQUIRE(ok, NV_ERR_UNSUPPORTED, "nv_stream_layernorm_pair: no kernel for %d columns", cols);
    return check_launch("nv_stream_layernorm_pair");
}

extern "C" int nv_silu_and_mul_rows(const void* x, int64_t x_stride, void* y, int dtype, int64_t rows, int inter,
                                    void* stream) {
    using namespace nv;
    NV_REQUIRE(rows >= 0 && inter > 0 && x_stride >= 2 * (int64_t)inter, NV_ERR_INVALID_ARG, "nv_silu_and_mul_rows: bad sizes");
    if (rows == 0) return NV_OK;
    NV_REQUIRE(x && y, NV_ERR_INVALID_ARG, "nv_silu_and_mul_rows: null pointer");
    NV_REQUIRE(dtype == NV_DTYPE_BF16 || dtype == NV_DTYPE_F32, NV_ERR_INVALID_ARG, "nv_silu_and_mul_rows: bad dtype");
    const bool bf = dtype == NV_DTYPE_BF16;
    const bool vec = inter % 4 == 0 && x_stride % 4 == 0 && ((uintptr_t)x | (uintptr_t)y) % (bf ? 8 : 16) == 0;
    const int pieces = vec ? inter / 4 : inter;
    const int64_t n = rows * pieces, grid = (n + 255) / 256;
    NV_REQUIRE(grid < (1LL << 31), NV_ERR_UNSUPPORTED, "nv_silu_and_mul_rows: launch too large");
    hipStream_t s = (hipStream_t)stream;
#define NV_SILU(T, V)                                                                                                \
    hipLaunchKernelGGL((silu_and_mul_rows_kernel<T, V>), dim3((unsigned)grid), dim3(256), 0, s, (const T*)x, x_stride, \
                       (T*)y, inter, pieces, n)
    if (bf && vec) NV_SILU(__bf16, 4);
    else if (bf) NV_SILU(__bf16, 1);
    else if (vec) NV_SILU(float, 4);
    else NV_SILU(float, 1);
#undef NV_SILU
    return check_launch("nv_silu_and_mul_rows");
}
