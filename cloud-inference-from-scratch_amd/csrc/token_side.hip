// What a layer adds to the stream from an embedding of the tokens that is the layer's own:
//
//   g = gelu_tanh(W_gate x) * e,   e = the token's row of the layer's columns of a table
//   x <- x + (W_proj g) / sqrt(mean((W_proj g)^2) + eps) * weight
//
// with x the float32 stream behind the layer's other branches.  `gated_token_rows` makes g from the first product.
#include "activation_forms.h"
#include "common.h"

namespace {

// z [tokens, dim] float32; out [tokens, dim]; table [vocab, ld], the layer's numbers from column `column` on.
template <typename T>
__global__ void gated_token_rows_kernel(const float* __restrict__ z, const T* __restrict__ table, long ld, int column,
                                        const int* __restrict__ ids, T* __restrict__ out, int dim, int vocab) {
    const int token = blockIdx.x;
    const int id = min(max(ids[token], 0), vocab - 1);
    const T* row = table + static_cast<size_t>(id) * ld + column;
    for (int i = threadIdx.x; i < dim; i += blockDim.x)
        out[static_cast<size_t>(token) * dim + i] =
            from_float<T>(gelu_tanh(z[static_cast<size_t>(token) * dim + i]) * to_float(row[i]));
}

// residual[row] += branch[row] (+ branch2[row]), float32 and in place; `rows` takes the new stream in the activation type.
template <typename B, typename T, int V>
__global__ void stream_rows_kernel(float* __restrict__ residual, const B* __restrict__ branch, const B* __restrict__ branch2,
                                   T* __restrict__ rows, long count) {
    const long i = (static_cast<long>(blockIdx.x) * blockDim.x + threadIdx.x) * V;
    if (i >= count) return;
    float x[V];
#pragma unroll
    for (int v = 0; v < V; ++v) {
        x[v] = residual[i + v];
        if (branch) x[v] += to_float(branch[i + v]);
        if (branch2) x[v] += to_float(branch2[i + v]);
    }
#pragma unroll
    for (int v = 0; v < V; ++v) {
        if (branch) residual[i + v] = x[v];
        if (rows) rows[i + v] = from_float<T>(x[v]);
    }
}

}  // namespace

CIE_API int cie_gated_token_rows(void* stream, int dtype, const float* z, const void* table, long ld, int column,
                                 const int* ids, void* out, int tokens, int dim, int vocab) {
    if (tokens < 0 || dim <= 0 || column < 0 || ld < static_cast<long>(column) + dim || vocab <= 0) return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int threads = dim >= 256 ? 256 : 64;
    if (dtype == CIE_F32)
        gated_token_rows_kernel<float><<<tokens, threads, 0, s>>>(z, static_cast<const float*>(table), ld, column, ids, static_cast<float*>(out), dim, vocab);
    else if (dtype == CIE_BF16)
        gated_token_rows_kernel<bf16_t><<<tokens, threads, 0, s>>>(z, static_cast<const bf16_t*>(table), ld, column, ids, static_cast<bf16_t*>(out), dim, vocab);
    else
        return CIE_BAD_ARGUMENT;
    return cie_after_launch();
}

// branch and branch2 (either may be absent, the second not without the first) are of type bdtype, rows of type dtype.
CIE_API int cie_stream_rows(void* stream, int bdtype, int dtype, float* residual, const void* branch, const void* branch2,
                            void* rows, int tokens, int hidden) {
    if (tokens < 0 || hidden <= 0 || (branch2 && !branch) || (!branch && !rows)) return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    const long count = static_cast<long>(tokens) * hidden;
    const bool by_four = hidden % 4 == 0;
    const long blocks = (count / (by_four ? 4 : 1) + 255) / 256;
    if (blocks > 0x7fffffffL) return CIE_BAD_ARGUMENT;
    const unsigned grid = static_cast<unsigned>(blocks);
    hipStream_t s = static_cast<hipStream_t>(stream);
#define CIE_STREAM_ROWS(B, T)                                                                                             \
    do {                                                                                                                  \
        if (by_four)                                                                                                      \
            stream_rows_kernel<B, T, 4><<<grid, 256, 0, s>>>(residual, static_cast<const B*>(branch), static_cast<const B*>(branch2), static_cast<T*>(rows), count); \
        else                                                                                                              \
            stream_rows_kernel<B, T, 1><<<grid, 256, 0, s>>>(residual, static_cast<const B*>(branch), static_cast<const B*>(branch2), static_cast<T*>(rows), count); \
    } while (0)
    if (dtype == CIE_F32 && (bdtype == CIE_F32 || !branch)) CIE_STREAM_ROWS(float, float);
    else if (dtype == CIE_BF16 && (bdtype == CIE_BF16 || !branch)) CIE_STREAM_ROWS(bf16_t, bf16_t);
    else if (dtype == CIE_BF16 && bdtype == CIE_F32) CIE_STREAM_ROWS(float, bf16_t);
    else return CIE_BAD_ARGUMENT;
#undef CIE_STREAM_ROWS
    return cie_after_launch();
}
