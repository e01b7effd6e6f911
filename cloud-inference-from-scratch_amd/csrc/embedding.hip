// Embedding gather: residual[t, :] = table[ids[t], :] * scale, widened to float32 (scale 1: as stored).
// The residual stream is float32 in both engine dtypes.  With `rows`, the same values are also written in the
// table's storage type, `ld_rows` numbers from row to row, for products that read the stream itself or the embedding's rows.
// With `feed` (int32 [tokens]) and `pool`: row t takes its token from pool[feed[t]] where feed[t] >= 0, so
// that a decode step can start from the tokens the step before it sampled, before the host has seen them.
// `ids_out`, if given, takes every row's token as it was taken (for what else a later layer looks up by token).
#include "common.h"

template <typename T>
__global__ void embed_kernel(const T* __restrict__ table, const int* __restrict__ ids,
                             const int* __restrict__ feed, const int* __restrict__ pool,
                             float* __restrict__ out, T* __restrict__ rows, long ld_rows, int hidden, int vocab,
                             float scale, int* __restrict__ ids_out) {
    const int token = blockIdx.x;
    int id = ids[token];
    if (feed != nullptr && feed[token] >= 0) id = pool[feed[token]];
    // Ids are validated on the host; clamp so that a stale padding row can never read outside.
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    if (ids_out && threadIdx.x == 0) ids_out[token] = id;
    const T* row = table + static_cast<size_t>(id) * hidden;
    float* dst = out + static_cast<size_t>(token) * hidden;
    T* copy = rows ? rows + static_cast<size_t>(token) * ld_rows : nullptr;
    for (int h = threadIdx.x; h < hidden; h += blockDim.x) {
        const float x = to_float(row[h]) * scale;
        dst[h] = x;
        if (copy) copy[h] = from_float<T>(x);
    }
}

CIE_API int cie_embed(void* stream, int dtype, const void* table, const int* ids, const int* feed,
                      const int* pool, float* out, void* rows, long ld_rows, int tokens, int hidden, int vocab, float scale,
                      int* ids_out) {
    if (tokens < 0 || hidden <= 0 || vocab <= 0 || (feed && !pool) || (rows && ld_rows < hidden)) return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == CIE_F32)
        embed_kernel<float><<<tokens, 256, 0, s>>>(static_cast<const float*>(table), ids, feed, pool, out, static_cast<float*>(rows), ld_rows, hidden, vocab, scale, ids_out);
    else if (dtype == CIE_BF16)
        embed_kernel<bf16_t><<<tokens, 256, 0, s>>>(static_cast<const bf16_t*>(table), ids, feed, pool, out, static_cast<bf16_t*>(rows), ld_rows, hidden, vocab, scale, ids_out);
    else
        return CIE_BAD_ARGUMENT;
    return cie_after_launch();
}

// The same gather for a model whose stream begins with a norm of the embedding's rows:
//   stream[t] = row / sqrt(mean(row^2) + eps) * weight,   row = table[ids[t]] * scale,
// float32, and with `next_weight` the RMS norm of the new stream row under that weight (the first layer's), stored in the
// table's type.  One workgroup per row, the row staged in LDS.
template <typename T>
__global__ void embed_normed_kernel(const T* __restrict__ table, const int* __restrict__ ids, const int* __restrict__ feed,
                                    const int* __restrict__ pool, const float* __restrict__ weight,
                                    float* __restrict__ out, int* __restrict__ ids_out,
                                    const float* __restrict__ next_weight, T* __restrict__ normed_out, int hidden,
                                    int vocab, float scale, float eps) {
    extern __shared__ float staged[];
    __shared__ float scratch[16];
    const int token = blockIdx.x;
    int id = ids[token];
    if (feed != nullptr && feed[token] >= 0) id = pool[feed[token]];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    if (ids_out && threadIdx.x == 0) ids_out[token] = id;
    const T* row = table + static_cast<size_t>(id) * hidden;
    float sum_sq = 0.f;
    for (int h = threadIdx.x; h < hidden; h += blockDim.x) {
        const float x = to_float(row[h]) * scale;
        staged[h] = x;
        sum_sq += x * x;
    }
    const float inv = 1.0f / sqrtf(block_sum(sum_sq, scratch) / static_cast<float>(hidden) + eps);
    float* dst = out + static_cast<size_t>(token) * hidden;
    float next_sq = 0.f;
    for (int h = threadIdx.x; h < hidden; h += blockDim.x) {
        const float x = (staged[h] * inv) * weight[h];
        dst[h] = x;
        staged[h] = x;
        next_sq += x * x;
    }
    if (!next_weight) return;
    const float next_inv = 1.0f / sqrtf(block_sum(next_sq, scratch) / static_cast<float>(hidden) + eps);
    T* normed = normed_out + static_cast<size_t>(token) * hidden;
    for (int h = threadIdx.x; h < hidden; h += blockDim.x)
        normed[h] = from_float<T>((staged[h] * next_inv) * next_weight[h]);
}

CIE_API int cie_embed_normed(void* stream, int dtype, const void* table, const int* ids, const int* feed, const int* pool,
                             const float* weight, float* out, int* ids_out, const float* next_weight, void* normed_out,
                             int tokens, int hidden, int vocab, float scale, float eps) {
    if (tokens < 0 || hidden <= 0 || hidden * sizeof(float) > 64 * 1024 || vocab <= 0 || (feed && !pool) || !weight || !out ||
        !(eps > 0.f) || (next_weight && !normed_out))
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int threads = tokens <= 64 ? 1024 : 256;
    const size_t lds = hidden * sizeof(float);
    if (dtype == CIE_F32)
        embed_normed_kernel<float><<<tokens, threads, lds, s>>>(
            static_cast<const float*>(table), ids, feed, pool, weight, out, ids_out, next_weight,
            static_cast<float*>(normed_out), hidden, vocab, scale, eps);
    else if (dtype == CIE_BF16)
        embed_normed_kernel<bf16_t><<<tokens, threads, lds, s>>>(
            static_cast<const bf16_t*>(table), ids, feed, pool, weight, out, ids_out, next_weight,
            static_cast<bf16_t*>(normed_out), hidden, vocab, scale, eps);
    else
        return CIE_BAD_ARGUMENT;
    return cie_after_launch();
}
