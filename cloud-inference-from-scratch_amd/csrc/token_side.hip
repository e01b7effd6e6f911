// What a layer adds to the stream from an embedding of the tokens that is the layer's own:
//
//   g = gelu_tanh(W_gate x) * e,   e = the token's row of the layer's columns of a table
//   x <- x + (W_proj g) / sqrt(mean((W_proj g)^2) + eps) * weight
//
// with x the float32 stream behind the layer's other branches.  Three ways to it.  Any sizes and float32: products of their
// own with small kernels around them (`stream_rows`, `gated_token_rows`; the norm and the add are the branch norm's kernel).
// bfloat16, few rows: one kernel makes g from the stream itself (the product, the gate and the lookup), many workgroups to a
// row.  bfloat16, many rows: one kernel does all of it, from the add of the other branches to the norm that the next layer
// reads, a workgroup to sixteen rows: a row is read and written once, and both weights come from the L2 caches.
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

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float floatx4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ floatx4 mfma16(uint4 a, uint4 b, floatx4 c) {  // 16 rows of a, 16 columns of b, 32 numbers of k
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}

__device__ __forceinline__ uint4 pack8(float4 lo, float4 hi) {
    return uint4{pack_bf16(lo.x, lo.y), pack_bf16(lo.z, lo.w), pack_bf16(hi.x, hi.y), pack_bf16(hi.z, hi.w)};
}

// Both kernels below read their weights as the matrix cores take them: [N, K] cut into pieces of 16 rows and 32 columns
// (zeros past either end), a piece's 64 lanes lying in a row of 1,024 bytes, lane (r, g) holding row r, columns 8 g .. 8 g + 7.
// A load of a piece is then one stretch of memory; from the plain layout it is sixteen half-used cache lines, and what a
// compute unit takes in a second, not the caches behind it, bounds the kernel (86 us for 2,048 rows of 2,048 instead of 41).
__device__ __forceinline__ const uint4* piece(const bf16_t* w, int n_tile, int k_slices, int k_slice, int lane) {
    return reinterpret_cast<const uint4*>(w) + (static_cast<size_t>(n_tile) * k_slices + k_slice) * kWave + lane;
}

// ---------------------------------------------------------------------------------------------- few rows
// g for 16 rows and 16 of the layer's columns a workgroup; its waves share K (the width) in slices of 32 and meet in LDS.
// The stream is read as it is and rounded on the way into the product.
constexpr int kGateWaves = 8;

__global__ void __launch_bounds__(64 * kGateWaves)
token_gate_kernel(const float* __restrict__ stream, const bf16_t* __restrict__ gate, const bf16_t* __restrict__ table, long ld,
                  int column, const int* __restrict__ ids, bf16_t* __restrict__ out, int tokens, int hidden, int dim, int vocab) {
    __shared__ float part[kGateWaves][256];
    constexpr int U = 4;  // slices of a wave that are on their way together
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int r = lane & 15, g = lane >> 4;
    const int n0 = blockIdx.x * 16, m0 = blockIdx.y * 16;
    const int slices = (hidden + 31) / 32;
    // (the thread that stores a number fetches the table's before the product starts)
    const int my_row = m0 + static_cast<int>(threadIdx.x) / 16, my_col = n0 + (threadIdx.x & 15);
    const bool stores = threadIdx.x < 256 && my_row < tokens && my_col < dim;
    float e = 0.f;
    if (stores) e = to_float(table[static_cast<size_t>(min(max(ids[my_row], 0), vocab - 1)) * ld + column + my_col]);
    const float* a = stream + static_cast<size_t>(min(m0 + r, tokens - 1)) * hidden;
    floatx4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = wave; s0 < slices; s0 += U * kGateWaves) {
        float4 x[U][2];
        uint4 w[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int slice = min(s0 + u * kGateWaves, slices - 1);
            const int k = min(slice * 32 + g * 8, hidden - 8);  // (past the last number the weights are zero)
            w[u] = *piece(gate, blockIdx.x, slices, slice, lane);
            x[u][0] = *reinterpret_cast<const float4*>(a + k);
            x[u][1] = *reinterpret_cast<const float4*>(a + k + 4);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const uint4 rows = pack8(x[u][0], x[u][1]);
            acc = mfma16(s0 + u * kGateWaves < slices ? rows : uint4{0u, 0u, 0u, 0u}, w[u], acc);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave][(g * 4 + i) * 16 + r] = acc[i];
    __syncthreads();
    if (!stores) return;
    float z = 0.f;
#pragma unroll
    for (int w = 0; w < kGateWaves; ++w) z += part[w][threadIdx.x];
    out[static_cast<size_t>(my_row) * dim + my_col] = from_float<bf16_t>(gelu_tanh(z) * e);
}

// ---------------------------------------------------------------------------------------------- many rows
constexpr int kSideWaves = 16;
constexpr int kSideRows = 16;

struct SideArgs {
    float* stream;             // [tokens, hidden], in place
    const bf16_t* branch;      // [tokens, hidden] still to be added, or null
    const bf16_t* gate;        // [dim, hidden] in pieces
    const bf16_t* proj;        // [hidden, dim] in pieces
    const bf16_t* table;
    long ld;
    int column;
    const int* ids;
    const float* weight;       // [hidden]
    const float* next_weight;  // [hidden] or null
    bf16_t* normed;            // [tokens, hidden]
    int tokens, hidden, dim, vocab;
    float eps;
    int k_shares;              // shares of the width that the first product is cut into, so that all waves have a tile
};

// The workgroup's LDS: the rows in the activation type, and later y, [16][hidden to 32 + 8]; the first product's shares
// [shares][16][dim to 16]; g [16][dim to 32 + 8].
struct SideLds {
    int hidden32, dim16, dim32, z, g, bytes;
    __host__ __device__ SideLds(int hidden, int dim, int k_shares) {
        hidden32 = (hidden + 31) / 32 * 32;
        dim16 = (dim + 15) / 16 * 16;
        dim32 = (dim + 31) / 32 * 32;
        z = kSideRows * (hidden32 + 8) * 2;
        g = z + k_shares * kSideRows * dim16 * 4;
        bytes = g + kSideRows * (dim32 + 8) * 2;
    }
};

__device__ __forceinline__ void load8f(const float* p, float (&v)[8]) {
    const float4 lo = *reinterpret_cast<const float4*>(p), hi = *reinterpret_cast<const float4*>(p + 4);
    v[0] = lo.x; v[1] = lo.y; v[2] = lo.z; v[3] = lo.w;
    v[4] = hi.x; v[5] = hi.y; v[6] = hi.z; v[7] = hi.w;
}
__device__ __forceinline__ void store8f(float* p, const float (&v)[8]) {
    *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<float4*>(p + 4) = float4{v[4], v[5], v[6], v[7]};
}
__device__ __forceinline__ void load8b(const bf16_t* p, float (&v)[8]) {
    const uint4 raw = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[2 * i] = __uint_as_float(w[i] << 16);
        v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}
__device__ __forceinline__ uint4 pack8v(const float (&v)[8]) {
    return uint4{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]), pack_bf16(v[4], v[5]), pack_bf16(v[6], v[7])};
}

// TURNS: turns of 512 numbers that a wave takes to go through a row.  (Fetching the next pieces of a weight while the last
// ones are multiplied changes nothing: a compute unit takes the two weights at some 75 GB/s either way.)
template <int TURNS>
__global__ void __launch_bounds__(64 * kSideWaves) token_side_kernel(SideArgs a) {
    extern __shared__ __attribute__((aligned(16))) char lds[];
    const SideLds at(a.hidden, a.dim, a.k_shares);
    bf16_t* rows_s = reinterpret_cast<bf16_t*>(lds);
    float* z_s = reinterpret_cast<float*>(lds + at.z);
    bf16_t* g_s = reinterpret_cast<bf16_t*>(lds + at.g);
    const int row_stride = at.hidden32 + 8, g_stride = at.dim32 + 8;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int r = lane & 15, g = lane >> 4;
    const int m0 = blockIdx.x * kSideRows;
    const bool real = m0 + wave < a.tokens;  // (the wave's own row, at the start and at the end)
    const size_t row = static_cast<size_t>(min(m0 + wave, a.tokens - 1));
    float* stream = a.stream + row * a.hidden;

    // a row a wave: the table's numbers, the stream with what is still to be added
    {
        const bf16_t* e = a.table + static_cast<size_t>(min(max(a.ids[row], 0), a.vocab - 1)) * a.ld + a.column;
        const bf16_t* add = a.branch ? a.branch + row * a.hidden : nullptr;
#pragma unroll
        for (int i = 0; i < TURNS; ++i) {
            const int h = (i * kWave + lane) * 8;
            if (h >= at.hidden32) break;
            float x[8] = {};
            if (h < a.hidden) {
                load8f(stream + h, x);
                if (add) {
                    float y[8];
                    load8b(add + h, y);
#pragma unroll
                    for (int v = 0; v < 8; ++v) x[v] += y[v];
                    if (real) store8f(stream + h, x);
                }
            }
            *reinterpret_cast<uint4*>(rows_s + wave * row_stride + h) = pack8v(x);
        }
        for (int i = lane; i < at.dim32; i += kWave) g_s[wave * g_stride + i] = i < a.dim ? e[i] : bf16_t{0};
    }
    __syncthreads();

    // z = rows * gate^T: a wave takes one tile of 16 columns over one share of the width (several, for a wide table part)
    // (The workgroups of an XCD go through the same weights at the same time: each begins at a place of its own, so that most
    // pieces have been brought into the XCD's L2 by another one when they are asked for.)
    const int column_tiles = at.dim16 / 16, slices = at.hidden32 / 32;
    const int first_slice = static_cast<int>((blockIdx.x / 8) * 8 % slices);
    for (int item = wave; item < column_tiles * a.k_shares; item += kSideWaves) {
        const int tile = item % column_tiles, share = item / column_tiles;
        floatx4 acc = {0.f, 0.f, 0.f, 0.f};
        constexpr int U = 8;
        for (int s0 = share; s0 < slices; s0 += U * a.k_shares) {
            uint4 w[U];
            int slice[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                slice[u] = min(s0 + u * a.k_shares, slices - 1) + first_slice;
                if (slice[u] >= slices) slice[u] -= slices;
                w[u] = *piece(a.gate, tile, slices, slice[u], lane);
            }
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const uint4 x = *reinterpret_cast<const uint4*>(rows_s + r * row_stride + slice[u] * 32 + g * 8);
                acc = mfma16(s0 + u * a.k_shares < slices ? x : uint4{0u, 0u, 0u, 0u}, w[u], acc);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) z_s[(share * kSideRows + g * 4 + i) * at.dim16 + tile * 16 + r] = acc[i];
    }
    __syncthreads();
    for (int i = threadIdx.x; i < kSideRows * a.dim; i += 64 * kSideWaves) {
        const int m = i / a.dim, n = i - m * a.dim;
        float z = 0.f;
        for (int s = 0; s < a.k_shares; ++s) z += z_s[(s * kSideRows + m) * at.dim16 + n];
        g_s[m * g_stride + n] = from_float<bf16_t>(gelu_tanh(z) * to_float(g_s[m * g_stride + n]));
    }
    __syncthreads();

    // y = g * proj^T, in the rows' place: a wave takes eight tiles of 16 columns at a time over all of the table part
    constexpr int kTiles = 8;
    const int y_tiles = (a.hidden + 15) / 16, y_slices = at.dim32 / 32;
    for (int t0 = wave * kTiles; t0 < y_tiles; t0 += kSideWaves * kTiles) {
        floatx4 y[kTiles];
#pragma unroll
        for (int t = 0; t < kTiles; ++t) y[t] = floatx4{0.f, 0.f, 0.f, 0.f};
        for (int s0 = 0, s = static_cast<int>((blockIdx.x / 8) % y_slices); s0 < y_slices; ++s0, s = s + 1 < y_slices ? s + 1 : 0) {
            uint4 w[kTiles];
#pragma unroll
            for (int t = 0; t < kTiles; ++t) w[t] = *piece(a.proj, min(t0 + t, y_tiles - 1), y_slices, s, lane);
            const uint4 x = *reinterpret_cast<const uint4*>(g_s + r * g_stride + s * 32 + g * 8);  // (zeros past the table part)
#pragma unroll
            for (int t = 0; t < kTiles; ++t) y[t] = mfma16(x, w[t], y[t]);
        }
#pragma unroll
        for (int t = 0; t < kTiles; ++t) {
            if (t0 + t >= y_tiles) break;  // wave-uniform
#pragma unroll
            for (int i = 0; i < 4; ++i) rows_s[(g * 4 + i) * row_stride + (t0 + t) * 16 + r] = from_float<bf16_t>(y[t][i]);
        }
    }
    __syncthreads();
    if (!real) return;

    // a row a wave again: its norm, the add, the next norm
    float x[TURNS][8];
    float sum_sq = 0.f;
#pragma unroll
    for (int i = 0; i < TURNS; ++i) {
        const int h = (i * kWave + lane) * 8;
        if (h >= a.hidden) break;
        float y[8];
        load8b(rows_s + wave * row_stride + h, y);
#pragma unroll
        for (int v = 0; v < 8; ++v) sum_sq += y[v] * y[v];
        load8f(stream + h, x[i]);
    }
    float inv = 1.0f / sqrtf(wave_sum(sum_sq) / static_cast<float>(a.hidden) + a.eps);
    sum_sq = 0.f;
#pragma unroll
    for (int i = 0; i < TURNS; ++i) {
        const int h = (i * kWave + lane) * 8;
        if (h >= a.hidden) break;
        float y[8], by[8];
        load8b(rows_s + wave * row_stride + h, y);
        load8f(a.weight + h, by);
#pragma unroll
        for (int v = 0; v < 8; ++v) {
            x[i][v] += (y[v] * inv) * by[v];
            sum_sq += x[i][v] * x[i][v];
        }
        store8f(stream + h, x[i]);
    }
    if (!a.next_weight) return;
    inv = 1.0f / sqrtf(wave_sum(sum_sq) / static_cast<float>(a.hidden) + a.eps);
#pragma unroll
    for (int i = 0; i < TURNS; ++i) {
        const int h = (i * kWave + lane) * 8;
        if (h >= a.hidden) break;
        float by[8];
        load8f(a.next_weight + h, by);
#pragma unroll
        for (int v = 0; v < 8; ++v) by[v] *= x[i][v] * inv;
        *reinterpret_cast<uint4*>(a.normed + row * a.hidden + h) = pack8v(by);
    }
}

template <int TURNS>
int launch_token_side(hipStream_t s, const SideArgs& a, int bytes) {
    static bool asked = false;  // (more LDS than a kernel gets without asking: once, and again is harmless)
    if (!asked) {
        if (hipFuncSetAttribute(reinterpret_cast<const void*>(&token_side_kernel<TURNS>), hipFuncAttributeMaxDynamicSharedMemorySize,
                                160 * 1024) != hipSuccess) {
            (void)hipGetLastError();
            return CIE_LAUNCH_FAILED;
        }
        asked = true;
    }
    token_side_kernel<TURNS><<<(a.tokens + kSideRows - 1) / kSideRows, 64 * kSideWaves, bytes, s>>>(a);
    return cie_after_launch();
}

}  // namespace

// g for few rows: bfloat16; hidden a multiple of 8; `gate` in pieces.
CIE_API int cie_token_gate(void* stream, const float* x, const void* gate, const void* table, long ld, int column,
                           const int* ids, void* out, int tokens, int hidden, int dim, int vocab) {
    if (tokens < 0 || hidden < 8 || hidden % 8 || dim <= 0 || column < 0 || ld < static_cast<long>(column) + dim || vocab <= 0 ||
        (tokens + 15) / 16 > 65535)
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    token_gate_kernel<<<dim3((dim + 15) / 16, (tokens + 15) / 16), 64 * kGateWaves, 0, static_cast<hipStream_t>(stream)>>>(
        x, static_cast<const bf16_t*>(gate), static_cast<const bf16_t*>(table), ld, column, ids, static_cast<bf16_t*>(out), tokens,
        hidden, dim, vocab);
    return cie_after_launch();
}

// All of it for many rows: bfloat16; hidden a multiple of 8 up to 4,096, and what the workgroup's LDS holds (`k_shares` as
// the caller planned it); `gate` and `proj` in pieces.
CIE_API int cie_token_side(void* stream, float* x, const void* branch, const void* gate, const void* proj, const void* table,
                           long ld, int column, const int* ids, const float* weight, const float* next_weight, void* normed,
                           int tokens, int hidden, int dim, int vocab, float eps, int k_shares) {
    if (tokens < 0 || hidden < 8 || hidden % 8 || hidden > 4096 || dim < 1 || column < 0 ||
        ld < static_cast<long>(column) + dim || vocab <= 0 || !(eps > 0.f) || !weight || (next_weight && !normed) || k_shares < 1 ||
        k_shares > kSideWaves)
        return CIE_BAD_ARGUMENT;
    const SideLds need(hidden, dim, k_shares);
    if (need.bytes > 160 * 1024) return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    const SideArgs a{x, static_cast<const bf16_t*>(branch), static_cast<const bf16_t*>(gate), static_cast<const bf16_t*>(proj),
                     static_cast<const bf16_t*>(table), ld, column, ids, weight, next_weight, static_cast<bf16_t*>(normed), tokens,
                     hidden, dim, vocab, eps, k_shares};
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (hidden <= 1024) return launch_token_side<2>(s, a, need.bytes);
    if (hidden <= 2048) return launch_token_side<4>(s, a, need.bytes);
    return launch_token_side<8>(s, a, need.bytes);
}

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
