// Attention over compressed keys: what lies between the down projection and the paged attention kernels.
//
// A token's cache entry is one vector that every head shares: [turned part (R) | normed latent (C) | zeros], as wide
// as the attention kernels' head size D.  A query head is folded into the same space, [its turned part (R) | its plain
// part times the key expansion (C) | zeros], so that the kernels see one key head and as many query heads as the
// layer has, and a head's weighted sum of cache entries holds, in its latent part, what the value expansion reads.
//
// This kernel lays the rows out for the rotation-and-cache-write kernel that follows it:
//
//   proj  [tokens, ldp]: heads x [plain (P) | turned (R)] queries, then [latent (C) | turned key part (R)]
//   rows  [tokens, (heads + 2) * D]:
//     query head h : [0, R) = its turned part as projected (the next kernel turns it)   [R + C, D) = 0
//                    ([R, R + C) is filled by the block-diagonal product with the key expansion)
//     key          : [0, R) = the shared key part as projected   [R, R + C) = latent / rms(latent) * weight   rest 0
//     value        : [0, R) = 0                                  [R, R + C) = the same normed latent         rest 0
//
// The latent's mean square, the division and the weight are float32; one rounding to the activation type.
#include "common.h"

template <typename T, typename W>
__global__ void __launch_bounds__(256)
latent_rows_kernel(const T* __restrict__ proj, long ldp, const W* __restrict__ weight, T* __restrict__ rows,
                   int heads, int plain, int turned, int latent, int width, float eps) {
    __shared__ float scratch[16];
    const int token = blockIdx.x;
    const T* src = proj + static_cast<size_t>(token) * ldp;
    T* dst = rows + static_cast<size_t>(token) * (heads + 2) * width;
    const T* down = src + static_cast<size_t>(heads) * (plain + turned);
    float sum_sq = 0.f;
    for (int i = threadIdx.x; i < latent; i += blockDim.x) {
        const float c = to_float(down[i]);
        sum_sq += c * c;
    }
    const float inv = 1.0f / sqrtf(block_sum(sum_sq, scratch) / static_cast<float>(latent) + eps);
    T* key = dst + static_cast<size_t>(heads) * width;
    T* value = key + width;
    const T zero = from_float<T>(0.f);
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
        T k = zero, v = zero;
        if (i < turned) {
            k = down[latent + i];
        } else if (i < turned + latent) {
            const int c = i - turned;
            k = v = from_float<T>((to_float(down[c]) * inv) * to_float(weight[c]));
        }
        key[i] = k;
        value[i] = v;
    }
    const int tail = width - turned - latent;
    for (int i = threadIdx.x; i < heads * (turned + tail); i += blockDim.x) {
        const int head = i / (turned + tail);
        const int j = i - head * (turned + tail);
        T* q = dst + static_cast<size_t>(head) * width;
        if (j < turned)
            q[j] = src[static_cast<size_t>(head) * (plain + turned) + plain + j];
        else
            q[turned + latent + (j - turned)] = zero;
    }
}

CIE_API int cie_latent_rows(void* stream, int dtype, int wdtype, const void* proj, long ldp, const void* weight,
                            void* rows, int tokens, int heads, int plain, int turned, int latent, int width, float eps) {
    if (tokens < 0 || heads <= 0 || plain <= 0 || turned < 0 || latent <= 0 || width < turned + latent || !(eps > 0.f) ||
        ldp < static_cast<long>(heads) * (plain + turned) + latent + turned)
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == CIE_F32 && wdtype == CIE_F32)
        latent_rows_kernel<float, float><<<tokens, 256, 0, s>>>(
            static_cast<const float*>(proj), ldp, static_cast<const float*>(weight), static_cast<float*>(rows), heads, plain,
            turned, latent, width, eps);
    else if (dtype == CIE_BF16 && wdtype == CIE_BF16)
        latent_rows_kernel<bf16_t, bf16_t><<<tokens, 256, 0, s>>>(
            static_cast<const bf16_t*>(proj), ldp, static_cast<const bf16_t*>(weight), static_cast<bf16_t*>(rows), heads,
            plain, turned, latent, width, eps);
    else if (dtype == CIE_BF16 && wdtype == CIE_F32)
        latent_rows_kernel<bf16_t, float><<<tokens, 256, 0, s>>>(
            static_cast<const bf16_t*>(proj), ldp, static_cast<const float*>(weight), static_cast<bf16_t*>(rows), heads,
            plain, turned, latent, width, eps);
    else
        return CIE_BAD_ARGUMENT;
    return cie_after_launch();
}

// ---------------------------------------------------------------------------------------------- with a query latent
// The same layer in a form whose cache keeps an entry [turned part (R) | normed latent (C) | zeros], D numbers wide, and
// as its value the normed latent alone (DV numbers wide), and whose queries may come from a latent of their own.
//
// `latent_down_kernel`, one workgroup per token, stands behind the down projections: it norms the query latent
// (RMS, weight) into `q_latent`, norms the key latent (RMS, weight), turns the first `rot` numbers of the shared key part
// by the token's position, and writes both into the token's place in the cache.  `latent_queries_kernel` stands behind
// the queries' projection [heads x (plain (P) | turned (R))]: it turns each head's turned part and lays it out, with the
// zeros behind the latent's room, in rows [tokens, heads * D]; the room itself is filled by the block-diagonal product
// with the key expansion.  Norms, angles and products with them are float32; one rounding to the activation type.
struct Turn {
    const float* cos_table;  // [positions, rot / 2]
    const float* sin_table;
    int rot;
    int neighbours;
};

// number d of a part that starts at p, turned by the position
template <typename T>
__device__ __forceinline__ float turned_number(const T* p, int d, int pos, const Turn& turn) {
    const float x = to_float(p[d]);
    if (d >= turn.rot) return x;
    const int half = turn.rot / 2;
    const int i = turn.neighbours ? d >> 1 : (d < half ? d : d - half);
    const bool is_u = turn.neighbours ? !(d & 1) : d < half;
    const int mate = turn.neighbours ? d ^ 1 : (is_u ? d + half : d - half);
    const float y = to_float(p[mate]);
    const float c = turn.cos_table[static_cast<size_t>(pos) * half + i];
    const float s = turn.sin_table[static_cast<size_t>(pos) * half + i];
    return is_u ? x * c - y * s : x * c + y * s;
}

template <typename T>
__global__ void __launch_bounds__(256)
latent_down_kernel(const T* __restrict__ proj, long ldp, int q_off, int q_rank, int c_off, const float* __restrict__ q_weight,
                   const float* __restrict__ c_weight, T* __restrict__ q_latent, Turn turn, const int* __restrict__ positions,
                   const int* __restrict__ seq_of_token, const int* __restrict__ seq_slot,
                   const int* __restrict__ block_table, int table_width, T* __restrict__ k_pool, T* __restrict__ v_pool,
                   int latent, int turned, int D, int DV, int page_shift, float eps, int write_kv) {
    __shared__ float scratch[16];
    const int token = blockIdx.x;
    const T* row = proj + static_cast<size_t>(token) * ldp;
    const T* down = row + c_off;
    const int pos = positions[token];
    const int page = write_kv ? block_table[static_cast<size_t>(seq_slot[seq_of_token[token]]) * table_width + (pos >> page_shift)] : 0;
    float q_sq = 0.f, c_sq = 0.f;
    for (int i = threadIdx.x; i < q_rank; i += blockDim.x) {
        const float x = to_float(row[q_off + i]);
        q_sq += x * x;
    }
    for (int i = threadIdx.x; i < latent; i += blockDim.x) {
        const float x = to_float(down[i]);
        c_sq += x * x;
    }
    if (q_rank > 0) {
        const float inv = 1.0f / sqrtf(block_sum(q_sq, scratch) / static_cast<float>(q_rank) + eps);
        for (int i = threadIdx.x; i < q_rank; i += blockDim.x)
            q_latent[static_cast<size_t>(token) * q_rank + i] = from_float<T>(to_float(row[q_off + i]) * inv * q_weight[i]);
    }
    if (!write_kv) return;
    const float inv = 1.0f / sqrtf(block_sum(c_sq, scratch) / static_cast<float>(latent) + eps);
    const int in_page = pos & ((1 << page_shift) - 1);
    T* key = k_pool + ((static_cast<size_t>(page) << page_shift) + in_page) * D;
    T* value = v_pool + ((static_cast<size_t>(page) * DV) << page_shift) + in_page;
    for (int i = threadIdx.x; i < D; i += blockDim.x) {
        float x = 0.f;
        if (i < turned)
            x = turned_number(down + latent, i, pos, turn);
        else if (i < turned + latent)
            x = to_float(down[i - turned]) * inv * c_weight[i - turned];
        key[i] = from_float<T>(x);
    }
    for (int i = threadIdx.x; i < DV; i += blockDim.x)
        value[static_cast<size_t>(i) << page_shift] = from_float<T>(i < latent ? to_float(down[i]) * inv * c_weight[i] : 0.f);
}

template <typename T>
__global__ void __launch_bounds__(256)
latent_queries_kernel(const T* __restrict__ q, long ldq, Turn turn, const int* __restrict__ positions, T* __restrict__ rows,
                      int heads, int plain, int turned, int latent, int D) {
    const int token = blockIdx.x;
    const int pos = positions[token];
    const int tail = D - turned - latent;
    const T* src = q + static_cast<size_t>(token) * ldq;
    T* dst = rows + static_cast<size_t>(token) * heads * D;
    for (int i = blockIdx.y * blockDim.x + threadIdx.x; i < heads * (turned + tail); i += blockDim.x * gridDim.y) {
        const int head = i / (turned + tail);
        const int j = i - head * (turned + tail);
        if (j < turned)
            dst[static_cast<size_t>(head) * D + j] =
                from_float<T>(turned_number(src + static_cast<size_t>(head) * (plain + turned) + plain, j, pos, turn));
        else
            dst[static_cast<size_t>(head) * D + latent + j] = from_float<T>(0.f);
    }
}

CIE_API int cie_latent_down(void* stream, int dtype, const void* proj, long ldp, int q_off, int q_rank, int c_off,
                            const float* q_weight, const float* c_weight, void* q_latent, const float* cos_table,
                            const float* sin_table, int rot, int neighbours, const int* positions, const int* seq_of_token,
                            const int* seq_slot, const int* block_table, int table_width, void* k_pool, void* v_pool,
                            int tokens, int latent, int turned, int D, int DV, int page_size, float eps, int write_kv) {
    if (tokens < 0 || q_rank < 0 || q_off < 0 || c_off < 0 || latent <= 0 || turned < 0 || D < latent + turned || DV < latent ||
        rot < 0 || rot % 2 || rot > turned || (rot > 0 && (!cos_table || !sin_table)) || page_size <= 0 ||
        (page_size & (page_size - 1)) || table_width <= 0 || !(eps > 0.f) || ldp < q_off + q_rank ||
        ldp < c_off + latent + turned || (q_rank > 0 && (!q_weight || !q_latent)) || !c_weight)
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    int page_shift = 0;
    while ((1 << page_shift) < page_size) ++page_shift;
    const Turn turn{cos_table, sin_table, rot, neighbours};
    hipStream_t s = static_cast<hipStream_t>(stream);
#define CIE_LATENT_DOWN(T)                                                                                              \
    latent_down_kernel<T><<<tokens, 256, 0, s>>>(static_cast<const T*>(proj), ldp, q_off, q_rank, c_off, q_weight, c_weight, \
                                                 static_cast<T*>(q_latent), turn, positions, seq_of_token, seq_slot,       \
                                                 block_table, table_width, static_cast<T*>(k_pool), static_cast<T*>(v_pool), \
                                                 latent, turned, D, DV, page_shift, eps, write_kv)
    if (dtype == CIE_F32) CIE_LATENT_DOWN(float);
    else if (dtype == CIE_BF16) CIE_LATENT_DOWN(bf16_t);
    else return CIE_BAD_ARGUMENT;
#undef CIE_LATENT_DOWN
    return cie_after_launch();
}

CIE_API int cie_latent_queries(void* stream, int dtype, const void* q, long ldq, const float* cos_table,
                               const float* sin_table, int rot, int neighbours, const int* positions, void* rows, int tokens,
                               int heads, int plain, int turned, int latent, int D) {
    if (tokens < 0 || heads <= 0 || plain < 0 || turned < 0 || latent <= 0 || D < turned + latent || rot < 0 || rot % 2 ||
        rot > turned || (rot > 0 && (!cos_table || !sin_table)) || ldq < static_cast<long>(heads) * (plain + turned))
        return CIE_BAD_ARGUMENT;
    const int numbers = heads * (D - latent);
    if (tokens == 0 || numbers == 0) return CIE_OK;
    const Turn turn{cos_table, sin_table, rot, neighbours};
    const int blocks = (numbers + 255) / 256;
    const dim3 grid(tokens, tokens >= 512 ? 1 : blocks < 32 ? blocks : 32);
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == CIE_F32)
        latent_queries_kernel<float><<<grid, 256, 0, s>>>(static_cast<const float*>(q), ldq, turn, positions,
                                                          static_cast<float*>(rows), heads, plain, turned, latent, D);
    else if (dtype == CIE_BF16)
        latent_queries_kernel<bf16_t><<<grid, 256, 0, s>>>(static_cast<const bf16_t*>(q), ldq, turn, positions,
                                                           static_cast<bf16_t*>(rows), heads, plain, turned, latent, D);
    else
        return CIE_BAD_ARGUMENT;
    return cie_after_launch();
}
