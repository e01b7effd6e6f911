// The gated delta rule: per head a float32 memory S [dim, vdim] that every token fades, corrects and reads,
//
//     S' = g S + k u^T  with the correction  u = beta (v - g S^T k),   read as  S'^T q
//
// where g (the decay, the exponential of -exp(a_log) times a softplus of its logit and bias) and beta (the step size, a
// sigmoid) are one number per head and token.  In front of it stand a causal convolution over each channel's last `taps`
// inputs with silu, for queries and keys a scaling to length one (1e-6 beside the sum of squares) and for queries a
// factor; neighbouring heads share a query and key head.  Behind it a head's read-out is RMS-normed under a weight that
// the heads share and gated by silu.  What enters is the projections' rows; everything behind them is float32.
//
// State per request slot: the memory, kept as [heads, vdim, dim] (a column of S lies in one piece), and the
// convolutions' last taps - 1 inputs, kept per head as [heads, taps - 1, 2 dim + vdim] (a head's query, key and value
// channels, oldest input first; heads that share a key head hold the same query and key inputs, so that each workgroup
// owns what it moves on).
//
// Two forms.  Steps of few tokens a sequence: one kernel does all of it, a workgroup per (sequence, head), the memory
// in registers (`delta_walk_kernel`); where the head's columns are cut into several workgroups the read-out goes out
// as float32 rows for a norm kernel behind it.  Prompts' portions: blocks of 32 tokens on the matrix cores (below).
#include "common.h"

namespace {

__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
__device__ __forceinline__ float softplus_f(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }

// Sum over the 16 lanes of a row of the wave; every lane gets it (rotations inside the row, no LDS).
template <int N>
__device__ __forceinline__ float row_rotated(float v) {
    return __uint_as_float(static_cast<unsigned>(
        __builtin_amdgcn_update_dpp(0, static_cast<int>(__float_as_uint(v)), 0x120 + N, 0xf, 0xf, true)));
}
__device__ __forceinline__ float row16_sum(float v) {
    v += row_rotated<8>(v);
    v += row_rotated<4>(v);
    v += row_rotated<2>(v);
    v += row_rotated<1>(v);
    return v;
}

template <typename T>
struct DeltaArgs {
    const T* proj;        // [tokens, ldp]: queries and keys (kv_heads x dim), values and gates (heads x vdim), b and a (heads)
    long ldp;
    int q_off, k_off, v_off, g_off, b_off, a_off;
    const T* taps_w;      // [2 kv_heads dim + heads vdim, taps]: the query, key and value channels' taps
    int taps;
    const float* a_log;   // [heads]
    const float* dt_bias; // [heads]
    float q_scale;
    float* state;         // [slots, heads, vdim, dim]
    float* past;          // [slots, heads, max(taps - 1, 1), 2 dim + vdim]
    const int* seq_slot;
    const int* q_start_loc;
    int heads, kv_heads, dim, vdim;
};

// which channel of a head (query, key, value numbers in a row) is column `col` of the projection and row `channel` of the taps
template <typename T>
__device__ __forceinline__ void head_channel(const DeltaArgs<T>& a, int head, int c, int& col, int& channel) {
    const int shared = head / (a.heads / a.kv_heads);
    if (c < a.dim) {
        channel = shared * a.dim + c;
        col = a.q_off + channel;
    } else if (c < 2 * a.dim) {
        const int at = shared * a.dim + c - a.dim;
        channel = a.kv_heads * a.dim + at;
        col = a.k_off + at;
    } else {
        const int at = head * a.vdim + c - 2 * a.dim;
        channel = 2 * a.kv_heads * a.dim + at;
        col = a.v_off + at;
    }
}

// channel c of `head` at token `t` of a sequence that starts at flat row `first`, convolved and activated
template <typename T>
__device__ __forceinline__ float convolved(const DeltaArgs<T>& a, int head, int c, int first, int t, const float* past) {
    int col, channel;
    head_channel(a, head, c, col, channel);
    const int width = 2 * a.dim + a.vdim;
    const T* w = a.taps_w + static_cast<size_t>(channel) * a.taps;
    float acc = 0.f;
    for (int j = 0; j < a.taps; ++j) {
        const int src = t - (a.taps - 1) + j;
        const float in = src >= 0 ? to_float(a.proj[static_cast<size_t>(first + src) * a.ldp + col])
                                  : past[static_cast<size_t>(a.taps - 1 + src) * width + c];
        acc = fmaf(to_float(w[j]), in, acc);
    }
    return silu_f(acc);
}

template <typename T>
__device__ __forceinline__ void steps_of(const DeltaArgs<T>& a, int head, int token, float& beta, float& log_decay) {
    const T* row = a.proj + static_cast<size_t>(token) * a.ldp;
    beta = sigmoid_f(to_float(row[a.b_off + head]));
    log_decay = -expf(a.a_log[head]) * softplus_f(to_float(row[a.a_off + head]) + a.dt_bias[head]);
}

// of [what the state held, the step's inputs] the last taps - 1 inputs of a head stay
template <typename T>
__device__ __forceinline__ void keep_inputs(const DeltaArgs<T>& a, int head, int first, int count, float* past) {
    const int width = 2 * a.dim + a.vdim;
    const int keep_n = a.taps - 1;
    for (int c = threadIdx.x; c < width; c += blockDim.x) {
        int col, channel;
        head_channel(a, head, c, col, channel);
        for (int j = 0; j < keep_n; ++j) {  // (row j is written from row j + count, which lies behind it)
            const int src = count + j;
            past[static_cast<size_t>(j) * width + c] =
                src < keep_n ? past[static_cast<size_t>(src) * width + c]
                             : to_float(a.proj[static_cast<size_t>(first + src - keep_n) * a.ldp + col]);
        }
    }
}

// ---------------------------------------------------------------------------------------------- the walk
// A workgroup per (sequence, head, slice of columns); 16 lanes to a column of S, each with R of its rows in registers
// (pieces of four neighbouring rows, 64 apart), CPT columns a thread.  Tokens go in chunks: the chunk's convolutions,
// norms and step sizes are made by the whole workgroup into LDS, then every group of 16 lanes walks its columns through
// the chunk without a barrier: S^T k and S^T q are summed across the 16 lanes by rotations, and the read-out behind the
// update is g S^T q + (k . q) u.  The order of every sum depends on the sizes alone.
template <typename T>
struct WalkOut {
    const float* norm_weight;  // [vdim]
    float eps;
    T* out;                    // [tokens, heads * vdim]: normed and gated, where one workgroup has all columns
    float* y;                  // ... else the raw read-out, float32
    int slice, chunk;
};

template <typename T, int R, int CPT, bool WHOLE>
__global__ void __launch_bounds__(512) delta_walk_kernel(DeltaArgs<T> a, WalkOut<T> w) {
    extern __shared__ float4 lds4[];
    constexpr int ROWS = 16 * R;
    constexpr int Q = R / 4;
    const int seq = blockIdx.x;
    const int head = blockIdx.y;
    const int slice0 = blockIdx.z * w.slice;
    const int cols = min(w.slice, a.vdim - slice0);
    const int lane16 = threadIdx.x & 15;
    const int group = threadIdx.x >> 4;
    const int groups = blockDim.x >> 4;
    const int lane = threadIdx.x % kWave;
    const int wave = threadIdx.x / kWave;
    const int waves = blockDim.x / kWave;
    const int first = a.q_start_loc[seq];
    const int count = a.q_start_loc[seq + 1] - first;
    if (count <= 0) return;
    float* q_s = reinterpret_cast<float*>(lds4);  // [chunk][ROWS]
    float* k_s = q_s + w.chunk * ROWS;            // [chunk][ROWS]
    float* v_s = k_s + w.chunk * ROWS;            // [chunk][slice]
    float* o_s = v_s + w.chunk * w.slice;         // [chunk][slice]
    float* kq_s = o_s + w.chunk * w.slice;        // [chunk]
    float* beta_s = kq_s + w.chunk;               // [chunk]
    float* decay_s = beta_s + w.chunk;            // [chunk]
    const size_t slot = a.seq_slot[seq];
    float* mem = a.state + (slot * a.heads + head) * a.vdim * a.dim;
    float* past = a.past + (slot * a.heads + head) * max(a.taps - 1, 1) * (2 * a.dim + a.vdim);
    const bool wide = a.dim % 4 == 0;  // (a column's pieces start at multiples of 16 bytes)
    float S[CPT][R];
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
        const int c = group + i * groups;
        const float* column = mem + static_cast<size_t>(slice0 + min(c, cols - 1)) * a.dim;
#pragma unroll
        for (int p = 0; p < Q; ++p) {
            const int n = 64 * p + 4 * lane16;
            if (wide) {
                const float4 x = *reinterpret_cast<const float4*>(column + min(n, a.dim - 4));
                const bool real = n < a.dim;
                S[i][4 * p] = real ? x.x : 0.f;
                S[i][4 * p + 1] = real ? x.y : 0.f;
                S[i][4 * p + 2] = real ? x.z : 0.f;
                S[i][4 * p + 3] = real ? x.w : 0.f;
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) S[i][4 * p + e] = n + e < a.dim ? column[n + e] : 0.f;
            }
        }
    }
    for (int from = 0; from < count; from += w.chunk) {
        const int n_tok = min(w.chunk, count - from);
        __syncthreads();  // (the chunk before has been read)
        for (int idx = threadIdx.x; idx < n_tok * ROWS; idx += blockDim.x) {
            const int t = idx / ROWS;
            const int n = idx - t * ROWS;
            q_s[idx] = n < a.dim ? convolved(a, head, n, first, from + t, past) : 0.f;
            k_s[idx] = n < a.dim ? convolved(a, head, a.dim + n, first, from + t, past) : 0.f;
        }
        for (int idx = threadIdx.x; idx < n_tok * w.slice; idx += blockDim.x) {
            const int t = idx / w.slice;
            const int c = idx - t * w.slice;
            v_s[idx] = c < cols ? convolved(a, head, 2 * a.dim + slice0 + c, first, from + t, past) : 0.f;
        }
        for (int t = threadIdx.x; t < n_tok; t += blockDim.x) {
            float beta, log_decay;
            steps_of(a, head, first + from + t, beta, log_decay);
            beta_s[t] = beta;
            decay_s[t] = expf(log_decay);
        }
        __syncthreads();
        for (int t = wave; t < n_tok; t += waves) {  // lengths of one, and k . q
            float qq = 0.f, kk = 0.f, kq = 0.f;
            for (int n = lane; n < ROWS; n += kWave) {
                const float q = q_s[t * ROWS + n], k = k_s[t * ROWS + n];
                qq += q * q;
                kk += k * k;
                kq += k * q;
            }
            const float q_by = a.q_scale / sqrtf(wave_sum(qq) + 1e-6f);
            const float k_by = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
            kq = wave_sum(kq);
            for (int n = lane; n < ROWS; n += kWave) {
                q_s[t * ROWS + n] *= q_by;
                k_s[t * ROWS + n] *= k_by;
            }
            if (lane == 0) kq_s[t] = kq * q_by * k_by;
        }
        __syncthreads();
        for (int t = 0; t < n_tok; ++t) {
            float4 k4[Q], q4[Q];
#pragma unroll
            for (int p = 0; p < Q; ++p) {
                k4[p] = *reinterpret_cast<const float4*>(k_s + t * ROWS + 64 * p + 4 * lane16);
                q4[p] = *reinterpret_cast<const float4*>(q_s + t * ROWS + 64 * p + 4 * lane16);
            }
            const float g = decay_s[t], beta = beta_s[t], kq = kq_s[t];
#pragma unroll
            for (int i = 0; i < CPT; ++i) {
                const int c = group + i * groups;
                float dk0 = 0.f, dk1 = 0.f, dq0 = 0.f, dq1 = 0.f;
#pragma unroll
                for (int p = 0; p < Q; ++p) {
                    dk0 = fmaf(S[i][4 * p], k4[p].x, dk0);
                    dk1 = fmaf(S[i][4 * p + 1], k4[p].y, dk1);
                    dk0 = fmaf(S[i][4 * p + 2], k4[p].z, dk0);
                    dk1 = fmaf(S[i][4 * p + 3], k4[p].w, dk1);
                    dq0 = fmaf(S[i][4 * p], q4[p].x, dq0);
                    dq1 = fmaf(S[i][4 * p + 1], q4[p].y, dq1);
                    dq0 = fmaf(S[i][4 * p + 2], q4[p].z, dq0);
                    dq1 = fmaf(S[i][4 * p + 3], q4[p].w, dq1);
                }
                const float dk = row16_sum(dk0 + dk1);
                const float dq = row16_sum(dq0 + dq1);
                const float u = beta * (v_s[t * w.slice + min(c, w.slice - 1)] - g * dk);
#pragma unroll
                for (int p = 0; p < Q; ++p) {
                    S[i][4 * p] = fmaf(k4[p].x, u, g * S[i][4 * p]);
                    S[i][4 * p + 1] = fmaf(k4[p].y, u, g * S[i][4 * p + 1]);
                    S[i][4 * p + 2] = fmaf(k4[p].z, u, g * S[i][4 * p + 2]);
                    S[i][4 * p + 3] = fmaf(k4[p].w, u, g * S[i][4 * p + 3]);
                }
                if (lane16 == 0 && c < cols) o_s[t * w.slice + c] = fmaf(kq, u, g * dq);
            }
        }
        __syncthreads();
        if (WHOLE) {
            for (int t = wave; t < n_tok; t += waves) {
                float sum = 0.f;
                for (int c = lane; c < cols; c += kWave) {
                    const float o = o_s[t * w.slice + c];
                    sum += o * o;
                }
                const float inv = 1.0f / sqrtf(wave_sum(sum) / static_cast<float>(a.vdim) + w.eps);
                const size_t token = first + from + t;
                const T* gate = a.proj + token * a.ldp + a.g_off + static_cast<size_t>(head) * a.vdim;
                T* dst = w.out + token * a.heads * a.vdim + static_cast<size_t>(head) * a.vdim;
                for (int c = lane; c < cols; c += kWave)
                    dst[c] = from_float<T>(o_s[t * w.slice + c] * inv * w.norm_weight[c] * silu_f(to_float(gate[c])));
            }
        } else {
            for (int idx = threadIdx.x; idx < n_tok * w.slice; idx += blockDim.x) {
                const int t = idx / w.slice;
                const int c = idx - t * w.slice;
                if (c < cols)
                    w.y[static_cast<size_t>(first + from + t) * a.heads * a.vdim + static_cast<size_t>(head) * a.vdim +
                        slice0 + c] = o_s[idx];
            }
        }
    }
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
        const int c = group + i * groups;
        if (c >= cols) continue;
        float* column = mem + static_cast<size_t>(slice0 + c) * a.dim;
#pragma unroll
        for (int p = 0; p < Q; ++p) {
            const int n = 64 * p + 4 * lane16;
            if (wide) {
                if (n < a.dim)
                    *reinterpret_cast<float4*>(column + n) = float4{S[i][4 * p], S[i][4 * p + 1], S[i][4 * p + 2], S[i][4 * p + 3]};
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < a.dim) column[n + e] = S[i][4 * p + e];
            }
        }
    }
    if (WHOLE) keep_inputs(a, head, first, count, past);  // (every read of the old inputs lies in front of the last barriers)
}

template <typename T>
__global__ void __launch_bounds__(256) delta_keep_kernel(DeltaArgs<T> a) {
    const int seq = blockIdx.x;
    const int head = blockIdx.y;
    const int first = a.q_start_loc[seq];
    const int count = a.q_start_loc[seq + 1] - first;
    if (count <= 0) return;
    float* past = a.past + (static_cast<size_t>(a.seq_slot[seq]) * a.heads + head) * max(a.taps - 1, 1) * (2 * a.dim + a.vdim);
    keep_inputs(a, head, first, count, past);
}

// ---------------------------------------------------------------------------------------------- blocks
// Blocks of 32 tokens, float32 on the matrix cores (`v_mfma_f32_16x16x4_f32`).  With S the memory in front of a block,
// L_i the sum of the logarithms of the decays of the block's tokens 0 .. i,
//     A_ij = beta_i exp(L_i - L_j) (k_i . k_j)  for j < i,       T = (I + A)^-1        (unit lower triangular)
//     U = T diag(beta) V - T diag(beta exp(L)) K S                                      (row i is the token's u)
//     o_i = exp(L_i) S^T q_i + sum_{j <= i} exp(L_i - L_j) (q_i . k_j) u_j
//     S' = exp(L_31) S + sum_j exp(L_31 - L_j) k_j u_j^T
// (every exponent is at most zero; tokens past a block's end have beta = 0 and so u = 0, and repeat the last L).
// `delta_prepare_kernel`: every token at once makes its q, k (rows padded with zeros to `padded` numbers), v, beta, log g.
// `delta_block_kernel`: every block at once makes T diag(beta) V, -T diag(beta exp(L)) K, the 32 x 32 weights of the
// read-out's second term and the powers of the decays.  `delta_scan_kernel`: a workgroup per (sequence, head, 16 columns)
// goes over the blocks in order with its 16 columns of S in registers; it is a chain of steps, so what it reads lies as
// its lanes take it (a float4 a lane, 64 lanes in a row: an "operand tile").
// Block b of sequence s has place first_token(s) / 32 + s + b.
// Operand layout of the product: lane (l16 = lane % 16, g = lane / 16) gives A[l16][g] and B[g][l16] and gets rows
// 4 g .. 4 g + 3 of column l16; which four numbers of a sum one product takes does not matter as long as both operands
// agree, so four products take the numbers 4 g .. 4 g + 3 of a run of 16: a result tile is then an operand as it is.
typedef float acc4_t __attribute__((ext_vector_type(4)));
constexpr int kBlock = 32;
constexpr int kTri = kBlock + 4;  // row stride of a 32 x 32 matrix in LDS

struct BlockArgs {
    float* rows;    // [tokens, 2 * kv_heads * padded]: q then k heads
    float* values;  // [tokens, heads * vdim]
    float* beta;    // [tokens, heads]
    float* logs;    // [tokens, heads]
    // operand tiles, of 16 tokens (half of a block) and 16 channels or columns each; lane (l16, g) has of
    float4* w;      // [places, heads, tiles, 2, 64]: -T diag(beta exp(L)) K: token l16, channels 4 g ..
    float4* q;      // [places, kv_heads, tiles, 2, 64]: token l16, channels 4 g ..
    float4* k;      // [places, kv_heads, tiles, 2, 64]: tokens 4 g .., channel l16
    float4* u;      // [places, heads, cols16 / 16, 2, 64]: T diag(beta) V: tokens 4 g .., column l16
    float4* p;      // [places, heads, 2, 2, 64]: the read-out's weights: row l16 of the first half index, 4 g .. of the second
    float* fade;    // [places, heads, 2, 32]: exp(L_i), exp(L_31 - L_i)
    float* state;   // [slots, heads, vdim, dim]
    const int* seq_slot;
    const int* q_start_loc;
    float* y;       // [tokens, heads * vdim]
    int heads, kv_heads, dim, vdim, padded, cols16;
    int tiles;      // of 16 channels: a multiple of 4, the ones past `padded` hold zeros
};

// One wave per (run of kRun neighbouring tokens, query or key head or piece of a value head): a lane has NC channels, 64
// apart, with their taps and last inputs in registers, so that a token's input is read once and not once a tap.  With more
// than kWindow taps every tap reads its input.
constexpr int kRun = 16;
constexpr int kWindow = 4;

template <typename T, int NC>
__global__ void __launch_bounds__(256)
delta_prepare_kernel(DeltaArgs<T> a, BlockArgs b, const int* __restrict__ seq_of_token, int tokens, int pieces) {
    const int lane = threadIdx.x % kWave;
    const int slots = 2 * a.kv_heads + a.heads * pieces;
    const long unit = static_cast<long>(blockIdx.x) * (blockDim.x / kWave) + threadIdx.x / kWave;
    const int run = static_cast<int>(unit / slots);
    if (run * kRun >= tokens) return;
    const int what = static_cast<int>(unit - static_cast<long>(run) * slots);
    const int per = a.heads / a.kv_heads;
    const bool is_value = what >= 2 * a.kv_heads;
    const bool is_q = what < a.kv_heads;
    const int piece = is_value ? (what - 2 * a.kv_heads) % pieces : 0;
    const int head = is_value ? (what - 2 * a.kv_heads) / pieces : (what % a.kv_heads) * per;
    const int size = is_value ? a.vdim : a.dim;
    const int from_channel = is_value ? 2 * a.dim : is_q ? 0 : a.dim;
    const int width = 2 * a.dim + a.vdim;
    const bool windowed = a.taps <= kWindow;
    int col[NC], at[NC];         // the lane's columns of the projection, and their numbers in the head
    bool real[NC];
    float tap[NC][kWindow], window[NC][kWindow - 1];
#pragma unroll
    for (int i = 0; i < NC; ++i) {
        at[i] = piece * NC * kWave + lane + i * kWave;
        real[i] = at[i] < size;
        int channel;
        head_channel(a, head, from_channel + (real[i] ? at[i] : 0), col[i], channel);
        const T* w = a.taps_w + static_cast<size_t>(channel) * a.taps;
#pragma unroll
        for (int j = 0; j < kWindow; ++j) {  // (fewer taps than the window: leading zeros)
            const int from = j - (kWindow - a.taps);
            tap[i][j] = windowed && from >= 0 ? to_float(w[from]) : 0.f;
        }
    }
    int seq = -1, first = 0;
    const float* past = nullptr;
    const int end = min(tokens, (run + 1) * kRun);
    for (int token = run * kRun; token < end; ++token) {
        const int now = seq_of_token[token];
        if (now != seq) {  // (uniform in the wave)
            seq = now;
            first = a.q_start_loc[seq];
            past = a.past + (static_cast<size_t>(a.seq_slot[seq]) * a.heads + head) * max(a.taps - 1, 1) * width + from_channel;
            if (windowed) {
#pragma unroll
                for (int i = 0; i < NC; ++i)
#pragma unroll
                    for (int j = 0; j < kWindow - 1; ++j) {
                        const int src = token - first - (kWindow - 1) + j;
                        const int kept = a.taps - 1 + src;  // its row of the state, if it lies in front of the step
                        window[i][j] = !real[i] ? 0.f
                                       : src >= 0 ? to_float(a.proj[static_cast<size_t>(first + src) * a.ldp + col[i]])
                                       : kept >= 0 ? past[static_cast<size_t>(kept) * width + at[i]] : 0.f;
                    }
            }
        }
        float x[NC];
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
            float acc = 0.f;
            if (windowed) {
                const float in = real[i] ? to_float(a.proj[static_cast<size_t>(token) * a.ldp + col[i]]) : 0.f;
#pragma unroll
                for (int j = 0; j < kWindow - 1; ++j) acc = fmaf(tap[i][j], window[i][j], acc);
                acc = fmaf(tap[i][kWindow - 1], in, acc);
#pragma unroll
                for (int j = 0; j + 1 < kWindow - 1; ++j) window[i][j] = window[i][j + 1];
                window[i][kWindow - 2] = in;
                x[i] = silu_f(acc);
            } else {
                x[i] = real[i] ? convolved(a, head, from_channel + at[i], first, token - first, past - from_channel) : 0.f;
            }
            sum += x[i] * x[i];
        }
        if (is_value) {
            float* dst = b.values + static_cast<size_t>(token) * a.heads * a.vdim + static_cast<size_t>(head) * a.vdim;
#pragma unroll
            for (int i = 0; i < NC; ++i)
                if (real[i]) dst[at[i]] = x[i];
        } else {
            const float by = (is_q ? a.q_scale : 1.0f) / sqrtf(wave_sum(sum) + 1e-6f);
            float* dst = b.rows + (static_cast<size_t>(token) * 2 * a.kv_heads + what) * b.padded;
#pragma unroll
            for (int i = 0; i < NC; ++i)
                if (at[i] < b.padded) dst[at[i]] = x[i] * by;
        }
    }
    if (is_value && piece == 0 && run * kRun + lane < end) {  // step sizes and decays, a token a lane
        const size_t token = static_cast<size_t>(run) * kRun + lane;
        if (lane < kRun) {
            float beta, log_decay;
            steps_of(a, head, static_cast<int>(token), beta, log_decay);
            b.beta[token * a.heads + head] = beta;
            b.logs[token * a.heads + head] = log_decay;
        }
    }
}

// Inverse of a unit lower triangular 16 x 16 matrix I + A, one column per lane of 16: x_i = [i = c] - sum_{j<i} A_ij x_j.
__device__ __forceinline__ void invert16(const float* a_rows, int stride, int c, float (&x)[16]) {
#pragma unroll
    for (int i = 0; i < 16; ++i) {
        float sum = i == c ? 1.f : 0.f;
#pragma unroll
        for (int j = 0; j < i; ++j) sum = fmaf(-a_rows[i * stride + j], x[j], sum);
        x[i] = sum;
    }
}

__global__ void __launch_bounds__(256) delta_block_kernel(BlockArgs a) {
    const int seq = blockIdx.x / a.heads;
    const int head = blockIdx.x - seq * a.heads;
    const int first = a.q_start_loc[seq];
    const int count = a.q_start_loc[seq + 1] - first;
    const int c0 = blockIdx.y * kBlock;
    if (c0 >= count) return;  // (the whole workgroup: the grid is sized for the longest sequence)
    const int cn = min(kBlock, count - c0);
    const int padded = a.padded;
    const int stride = padded + 4;
    extern __shared__ float4 lds4[];
    float* k_s = reinterpret_cast<float*>(lds4);  // [32][stride]
    float* a_s = k_s + kBlock * stride;           // [32][kTri]: A, strictly lower
    float* t_s = a_s + kBlock * kTri;             // [32][kTri]: T
    float* z_s = t_s + kBlock * kTri;             // [16][20]
    float* log_s = z_s + 16 * 20;                 // [32]: L
    float* beta_s = log_s + kBlock;               // [32]
    const int lane = threadIdx.x % kWave;
    const int wave = threadIdx.x / kWave;
    const int l16 = lane % 16;
    const int g = lane / 16;
    const int shared = head / (a.heads / a.kv_heads);
    const size_t ld = static_cast<size_t>(2) * a.kv_heads * padded;
    const float* q_rows = a.rows + static_cast<size_t>(first + c0) * ld + static_cast<size_t>(shared) * padded;
    const float* k_rows = q_rows + static_cast<size_t>(a.kv_heads) * padded;
    for (int idx = threadIdx.x; idx < kBlock * (padded / 4); idx += blockDim.x) {
        const int t = idx / (padded / 4);
        const int n = 4 * (idx - t * (padded / 4));
        *reinterpret_cast<float4*>(k_s + t * stride + n) =
            *reinterpret_cast<const float4*>(k_rows + static_cast<size_t>(min(t, cn - 1)) * ld + n);
    }
    if (wave == 0) {
        const size_t token = static_cast<size_t>(first + c0 + min(lane, cn - 1));
        float log = lane < cn ? a.logs[token * a.heads + head] : 0.f;
#pragma unroll
        for (int d = 1; d < kBlock; d <<= 1) {
            const float before = __shfl_up(log, d, kWave);
            if (lane >= d) log += before;
        }
        if (lane < kBlock) {
            log_s[lane] = log;
            beta_s[lane] = lane < cn ? a.beta[token * a.heads + head] : 0.f;
        }
    }
    for (int idx = threadIdx.x; idx < kBlock * kTri; idx += blockDim.x) a_s[idx] = t_s[idx] = 0.f;
    __syncthreads();
    const int place = first / kBlock + seq + blockIdx.y;
    const size_t unit = static_cast<size_t>(place) * a.heads + head;
    const size_t unit_kv = static_cast<size_t>(place) * a.kv_heads + shared;
    const bool leads = head % (a.heads / a.kv_heads) == 0;  // writes what the heads of a key head share
    {   // this wave's tile of k k^T and of (q k^T)^T (the tile above the diagonal is zero)
        const int ti = wave >> 1, tj = wave & 1;
        acc4_t kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
        if (tj <= ti) {
            const float* ka = k_s + (16 * ti + l16) * stride + 4 * g;
            const float* kb = k_s + (16 * tj + l16) * stride + 4 * g;
            const float* qa = q_rows + static_cast<size_t>(min(16 * ti + l16, cn - 1)) * ld + 4 * g;
            float4* q_out = leads && tj == 0 ? a.q + unit_kv * a.tiles * 2 * kWave + ti * kWave + lane : nullptr;
            for (int m = 0; m < padded / 16; ++m) {
                const float4 x = *reinterpret_cast<const float4*>(ka + 16 * m);
                const float4 y = *reinterpret_cast<const float4*>(kb + 16 * m);
                const float4 z = *reinterpret_cast<const float4*>(qa + 16 * m);
                if (q_out) q_out[m * 2 * kWave] = z;
                kk = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, kk, 0, 0, 0);
                qk = __builtin_amdgcn_mfma_f32_16x16x4f32(y.x, z.x, qk, 0, 0, 0);
                kk = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, kk, 0, 0, 0);
                qk = __builtin_amdgcn_mfma_f32_16x16x4f32(y.y, z.y, qk, 0, 0, 0);
                kk = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, kk, 0, 0, 0);
                qk = __builtin_amdgcn_mfma_f32_16x16x4f32(y.z, z.z, qk, 0, 0, 0);
                kk = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, kk, 0, 0, 0);
                qk = __builtin_amdgcn_mfma_f32_16x16x4f32(y.w, z.w, qk, 0, 0, 0);
            }
            if (q_out)
                for (int m = padded / 16; m < a.tiles; ++m) q_out[m * 2 * kWave] = float4{0.f, 0.f, 0.f, 0.f};
        }
        acc4_t p;  // (queries along the lanes: as the scan takes it)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = 16 * ti + 4 * g + r, j = 16 * tj + l16;
            if (i > j) a_s[i * kTri + j] = beta_s[i] * expf(log_s[i] - log_s[j]) * kk[r];
            const int row = 16 * ti + l16, key = 16 * tj + 4 * g + r;
            p[r] = row >= key ? expf(log_s[row] - log_s[key]) * qk[r] : 0.f;
        }
        a.p[((unit * 2 + ti) * 2 + tj) * kWave + lane] = __builtin_bit_cast(float4, p);
    }
    __syncthreads();
    if (wave == 0 && lane < 32) {  // the two 16 x 16 inverses on the diagonal, a column per lane
        const int d = lane / 16;
        float x[16];
        invert16(a_s + 16 * d * kTri + 16 * d, kTri, l16, x);
#pragma unroll
        for (int i = 0; i < 16; ++i) t_s[(16 * d + i) * kTri + 16 * d + l16] = x[i];
    }
    __syncthreads();
    if (wave == 0) {  // below the diagonal: -T22 A21 T11
        acc4_t z = {0.f, 0.f, 0.f, 0.f};
        const float4 x = *reinterpret_cast<const float4*>(a_s + (16 + l16) * kTri + 4 * g);
        z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, t_s[(4 * g) * kTri + l16], z, 0, 0, 0);
        z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, t_s[(4 * g + 1) * kTri + l16], z, 0, 0, 0);
        z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, t_s[(4 * g + 2) * kTri + l16], z, 0, 0, 0);
        z = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, t_s[(4 * g + 3) * kTri + l16], z, 0, 0, 0);
        // (a result tile is the second operand of the next product as it is)
        const float4 y = *reinterpret_cast<const float4*>(t_s + (16 + l16) * kTri + 16 + 4 * g);
        acc4_t t21 = {0.f, 0.f, 0.f, 0.f};
        t21 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.x, z[0], t21, 0, 0, 0);
        t21 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.y, z[1], t21, 0, 0, 0);
        t21 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.z, z[2], t21, 0, 0, 0);
        t21 = __builtin_amdgcn_mfma_f32_16x16x4f32(y.w, z[3], t21, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) t_s[(16 + 4 * g + r) * kTri + l16] = -t21[r];
        const int i = lane % kBlock;
        a.fade[unit * 2 * kBlock + lane] = expf(lane < kBlock ? log_s[i] : log_s[kBlock - 1] - log_s[i]);
    }
    __syncthreads();
    float4 t_a[2][2];         // T's rows as operands: [row tile][run of 16 tokens]
    float k_by[2][4], v_by[2][4];
#pragma unroll
    for (int h = 0; h < 2; ++h) {
#pragma unroll
        for (int ti = 0; ti < 2; ++ti) t_a[ti][h] = *reinterpret_cast<const float4*>(t_s + (16 * ti + l16) * kTri + 16 * h + 4 * g);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int j = 16 * h + 4 * g + e;
            v_by[h][e] = beta_s[j];
            k_by[h][e] = -beta_s[j] * expf(log_s[j]);
        }
    }
    const int k_tiles = padded / 16, v_tiles = a.cols16 / 16;
    for (int ct = wave; ct < a.tiles + v_tiles; ct += 4) {
        const bool is_k = ct < a.tiles;
        const int tile = is_k ? ct : ct - a.tiles;
        const int col = 16 * tile + l16;
        float4* dst = (is_k ? a.w + (unit * a.tiles + tile) * 2 * kWave : a.u + (unit * v_tiles + tile) * 2 * kWave) + lane;
        float b[2][4];
#pragma unroll
        for (int h = 0; h < 2; ++h) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = 16 * h + 4 * g + e;
                if (is_k)
                    b[h][e] = tile < k_tiles ? k_s[j * stride + col] : 0.f;
                else
                    b[h][e] = col < a.vdim ? a.values[(static_cast<size_t>(first + c0) + min(j, cn - 1)) * a.heads * a.vdim +
                                                      static_cast<size_t>(head) * a.vdim + col] : 0.f;
            }
            if (is_k && leads)
                a.k[((unit_kv * a.tiles + tile) * 2 + h) * kWave + lane] = float4{b[h][0], b[h][1], b[h][2], b[h][3]};
#pragma unroll
            for (int e = 0; e < 4; ++e) b[h][e] *= is_k ? k_by[h][e] : v_by[h][e];
        }
        acc4_t r0 = {0.f, 0.f, 0.f, 0.f}, r1 = {0.f, 0.f, 0.f, 0.f};
        // (the upper tile has nothing right of the diagonal; the product's sides as the scan takes the result)
#define CIE_DELTA_TILE(r, t, h, c, e)                                                        \
    r = is_k ? __builtin_amdgcn_mfma_f32_16x16x4f32(b[h][e], t_a[t][h].c, r, 0, 0, 0)        \
             : __builtin_amdgcn_mfma_f32_16x16x4f32(t_a[t][h].c, b[h][e], r, 0, 0, 0)
        CIE_DELTA_TILE(r0, 0, 0, x, 0); CIE_DELTA_TILE(r1, 1, 0, x, 0); CIE_DELTA_TILE(r0, 0, 0, y, 1); CIE_DELTA_TILE(r1, 1, 0, y, 1);
        CIE_DELTA_TILE(r0, 0, 0, z, 2); CIE_DELTA_TILE(r1, 1, 0, z, 2); CIE_DELTA_TILE(r0, 0, 0, w, 3); CIE_DELTA_TILE(r1, 1, 0, w, 3);
        CIE_DELTA_TILE(r1, 1, 1, x, 0); CIE_DELTA_TILE(r1, 1, 1, y, 1); CIE_DELTA_TILE(r1, 1, 1, z, 2); CIE_DELTA_TILE(r1, 1, 1, w, 3);
#undef CIE_DELTA_TILE
        dst[0] = __builtin_bit_cast(float4, r0);
        dst[kWave] = __builtin_bit_cast(float4, r1);
    }
}

// A barrier for what waves exchange through LDS alone: loads from memory that are under way (the next block's operands)
// stay so, where __syncthreads() would wait for them.
__device__ __forceinline__ void lds_barrier() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "workgroup", "local");
    __builtin_amdgcn_s_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "workgroup", "local");
}

// What one block brings to a wave of the scan, in registers.
template <int MT>
struct ScanStage {
    float4 w[MT][2], q[MT][2], k[MT][2], p[2], u[2], grown[2], left[2];
    float whole;
};

// MT tiles of 16 channels a wave (tiles = 4 * MT): wave w has the tiles w, w + 4, ...
template <int MT>
__global__ void __launch_bounds__(256) delta_scan_kernel(BlockArgs a) {
    const int seq = blockIdx.x / a.heads;
    const int head = blockIdx.x - seq * a.heads;
    const int first = a.q_start_loc[seq];
    const int count = a.q_start_loc[seq + 1] - first;
    if (count <= 0) return;
    const int lane = threadIdx.x % kWave;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWave);
    const int l16 = lane % 16;
    const int g = lane / 16;
    const int col = 16 * blockIdx.y + l16;
    const int shared = head / (a.heads / a.kv_heads);
    __shared__ float4 part_s[2][4][4][kWave];  // [buffer][wave][u tile 0, 1, o tile 0, 1][lane]
    float* column = a.state + ((static_cast<size_t>(a.seq_slot[seq]) * a.heads + head) * a.vdim + min(col, a.vdim - 1)) * a.dim;
    acc4_t S[MT];
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = 16 * (wave + 4 * m) + 4 * g + e;
            S[m][e] = (n < a.dim && col < a.vdim) ? column[n] : 0.f;
        }
    const int blocks = (count + kBlock - 1) / kBlock;
    const size_t place0 = static_cast<size_t>(first / kBlock + seq);
    const size_t ldy = static_cast<size_t>(a.heads) * a.vdim;
    float* y = a.y + static_cast<size_t>(first + 16 * (wave & 1) + 4 * g) * ldy + static_cast<size_t>(head) * a.vdim + col;
    auto fetch = [&](ScanStage<MT>& to, int block) {
        const size_t place = place0 + min(block, blocks - 1);  // (past the end: the last one again, and nobody looks at it)
        const size_t unit = place * a.heads + head;
        const float4* w = a.w + (unit * (4 * MT) + wave) * 2 * kWave + lane;
        const size_t kv = ((place * a.kv_heads + shared) * (4 * MT) + wave) * 2 * kWave;
        const float4* q = a.q + kv + lane;
        const float4* k = a.k + kv + lane;
        const float4* u = a.u + (unit * (a.cols16 / 16) + blockIdx.y) * 2 * kWave + lane;
        const float4* p = a.p + (unit * 2 + (wave & 1)) * 2 * kWave + lane;
        const float* fade = a.fade + unit * 2 * kBlock;
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                to.w[m][t] = w[(8 * m + t) * kWave];
                to.q[m][t] = q[(8 * m + t) * kWave];
            }
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            to.u[t] = u[t * kWave];
            to.p[t] = p[t * kWave];
            to.grown[t] = *reinterpret_cast<const float4*>(fade + 16 * t + 4 * g);
            to.left[t] = *reinterpret_cast<const float4*>(fade + kBlock + 16 * t + 4 * g);
        }
        to.whole = fade[kBlock - 1];
#pragma unroll
        for (int m = 0; m < MT; ++m)
#pragma unroll
            for (int t = 0; t < 2; ++t) to.k[m][t] = k[(8 * m + t) * kWave];
    };
    auto step = [&](const ScanStage<MT>& in, int b) {
        // this wave's rows' share of -W S and of S^T q, for both tiles of tokens
        acc4_t us[2], os[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) us[t] = os[t] = acc4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int m = 0; m < MT; ++m) {
#define CIE_DELTA_SHARE(c, e)                                                                          \
    us[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(in.w[m][0].c, S[m][e], us[0], 0, 0, 0);               \
    us[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(in.w[m][1].c, S[m][e], us[1], 0, 0, 0);               \
    os[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(in.q[m][0].c, S[m][e], os[0], 0, 0, 0);               \
    os[1] = __builtin_amdgcn_mfma_f32_16x16x4f32(in.q[m][1].c, S[m][e], os[1], 0, 0, 0)
            CIE_DELTA_SHARE(x, 0); CIE_DELTA_SHARE(y, 1); CIE_DELTA_SHARE(z, 2); CIE_DELTA_SHARE(w, 3);
#undef CIE_DELTA_SHARE
        }
        auto& part = part_s[b & 1];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            part[wave][t][lane] = __builtin_bit_cast(float4, us[t]);
            part[wave][2 + t][lane] = __builtin_bit_cast(float4, os[t]);
        }
        lds_barrier();
        acc4_t u[2], faded[2];
#pragma unroll
        for (int t = 0; t < 2; ++t) {
            u[t] = __builtin_bit_cast(acc4_t, in.u[t]);
#pragma unroll
            for (int s = 0; s < 4; ++s) u[t] += __builtin_bit_cast(acc4_t, part[s][t][lane]);
            faded[t] = u[t] * __builtin_bit_cast(acc4_t, in.left[t]);
        }
#pragma unroll
        for (int m = 0; m < MT; ++m) S[m] *= in.whole;
#pragma unroll
        for (int t = 0; t < 2; ++t) {
#define CIE_DELTA_KEEP(c, e)                                                                           \
    _Pragma("unroll") for (int m = 0; m < MT; ++m)                                                     \
        S[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(in.k[m][t].c, faded[t][e], S[m], 0, 0, 0)
            CIE_DELTA_KEEP(x, 0); CIE_DELTA_KEEP(y, 1); CIE_DELTA_KEEP(z, 2); CIE_DELTA_KEEP(w, 3);
#undef CIE_DELTA_KEEP
        }
        if (wave < 2) {  // the read-out of tile `wave`
            acc4_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int s = 0; s < 4; ++s) o += __builtin_bit_cast(acc4_t, part[s][2 + wave][lane]);
            o *= __builtin_bit_cast(acc4_t, wave == 0 ? in.grown[0] : in.grown[1]);
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(in.p[t].x, u[t][0], o, 0, 0, 0);
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(in.p[t].y, u[t][1], o, 0, 0, 0);
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(in.p[t].z, u[t][2], o, 0, 0, 0);
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(in.p[t].w, u[t][3], o, 0, 0, 0);
            }
            float* row = y + static_cast<size_t>(b * kBlock) * ldy;
            if ((b + 1) * kBlock <= count) {
                if (col < a.vdim) {
#pragma unroll
                    for (int r = 0; r < 4; ++r) row[r * ldy] = o[r];
                }
            } else {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (col < a.vdim && b * kBlock + 16 * wave + 4 * g + r < count) row[r * ldy] = o[r];
            }
        }
    };
    // two blocks are under way while one is worked on
    ScanStage<MT> s0, s1, s2;
    fetch(s0, 0);
    fetch(s1, 1);
    for (int b = 0;; b += 3) {
        fetch(s2, b + 2);
        step(s0, b);
        if (b + 1 >= blocks) break;
        fetch(s0, b + 3);
        step(s1, b + 1);
        if (b + 2 >= blocks) break;
        fetch(s1, b + 4);
        step(s2, b + 2);
        if (b + 3 >= blocks) break;
    }
    if (col >= a.vdim) return;
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = 16 * (wave + 4 * m) + 4 * g + e;
            if (n < a.dim) column[n] = S[m][e];
        }
}

template <typename T>
DeltaArgs<T> delta_args(const void* proj, long ldp, int q_off, int k_off, int v_off, int g_off, int b_off, int a_off,
                        const void* taps_w, int taps, const float* a_log, const float* dt_bias, float q_scale, float* state,
                        float* past, const int* seq_slot, const int* q_start_loc, int heads, int kv_heads, int dim, int vdim) {
    return DeltaArgs<T>{static_cast<const T*>(proj), ldp, q_off, k_off, v_off, g_off, b_off, a_off,
                        static_cast<const T*>(taps_w), taps, a_log, dt_bias, q_scale, state, past, seq_slot, q_start_loc,
                        heads, kv_heads, dim, vdim};
}

template <typename T, int R, int CPT>
int launch_walk(hipStream_t s, const DeltaArgs<T>& a, const WalkOut<T>& w, int sequences, int threads, size_t lds) {
    const int slices = (a.vdim + w.slice - 1) / w.slice;
    const dim3 grid(sequences, a.heads, slices);
    if (slices == 1) {
        delta_walk_kernel<T, R, CPT, true><<<grid, threads, lds, s>>>(a, w);
        return cie_after_launch();
    }
    delta_walk_kernel<T, R, CPT, false><<<grid, threads, lds, s>>>(a, w);
    if (hipGetLastError() != hipSuccess) return CIE_LAUNCH_FAILED;
    delta_keep_kernel<T><<<dim3(sequences, a.heads), 256, 0, s>>>(a);
    return cie_after_launch();
}

template <typename T>
int walk(hipStream_t s, const DeltaArgs<T>& a, const WalkOut<T>& w, int sequences, int rows_per_thread, int columns_per_thread,
         int threads) {
    const size_t lds = sizeof(float) * static_cast<size_t>(w.chunk) * (32 * rows_per_thread + 2 * w.slice + 3);
    if (lds > 64 * 1024) return CIE_BAD_ARGUMENT;
#define CIE_DELTA_WALK(R, C) \
    if (rows_per_thread == R && columns_per_thread == C) return launch_walk<T, R, C>(s, a, w, sequences, threads, lds)
    CIE_DELTA_WALK(4, 1); CIE_DELTA_WALK(4, 2); CIE_DELTA_WALK(4, 4); CIE_DELTA_WALK(4, 8);
    CIE_DELTA_WALK(8, 1); CIE_DELTA_WALK(8, 2); CIE_DELTA_WALK(8, 4); CIE_DELTA_WALK(8, 8);
    CIE_DELTA_WALK(16, 1); CIE_DELTA_WALK(16, 2); CIE_DELTA_WALK(16, 4); CIE_DELTA_WALK(16, 8);
    CIE_DELTA_WALK(32, 1); CIE_DELTA_WALK(32, 2);
#undef CIE_DELTA_WALK
    return CIE_BAD_ARGUMENT;
}

bool bad_delta(int sequences, int heads, int kv_heads, int dim, int vdim, int taps, long ldp, int q_off, int k_off, int v_off,
               int g_off, int b_off, int a_off) {
    const long qk = static_cast<long>(kv_heads) * dim, vg = static_cast<long>(heads) * vdim;
    return sequences < 0 || sequences > 65535 || heads <= 0 || heads > 65535 || kv_heads <= 0 || heads % kv_heads ||
           dim <= 0 || dim > 512 || vdim <= 0 || taps < 1 || taps > 64 || q_off < 0 || k_off < 0 || v_off < 0 || g_off < 0 ||
           b_off < 0 || a_off < 0 || q_off + qk > ldp || k_off + qk > ldp || v_off + vg > ldp || g_off + vg > ldp ||
           b_off + heads > ldp || a_off + heads > ldp;
}

}  // namespace

// The walk, token by token.  16 * rows_per_thread >= dim; threads a multiple of 64 up to 512; threads / 16 *
// columns_per_thread >= slice.  One slice (slice >= vdim): `out` gets the normed, gated rows; else `y` the raw read-out.
CIE_API int cie_delta_walk(void* stream, int dtype, const void* proj, long ldp, int q_off, int k_off, int v_off, int g_off,
                           int b_off, int a_off, const void* taps_w, int taps, const float* a_log, const float* dt_bias,
                           float q_scale, const float* norm_weight, float eps, float* state, float* past, const int* seq_slot,
                           const int* q_start_loc, void* out, float* y, int sequences, int heads, int kv_heads, int dim,
                           int vdim, int rows_per_thread, int columns_per_thread, int threads, int slice, int chunk) {
    if (bad_delta(sequences, heads, kv_heads, dim, vdim, taps, ldp, q_off, k_off, v_off, g_off, b_off, a_off) ||
        16 * rows_per_thread < dim || threads < 64 || threads > 512 || threads % 64 || slice <= 0 ||
        (threads / 16) * columns_per_thread < slice || chunk <= 0 || (vdim + slice - 1) / slice > 65535 || !proj || !taps_w ||
        !a_log || !dt_bias || !state || !past || (slice >= vdim ? !out || !norm_weight || !(eps > 0.f) : !y))
        return CIE_BAD_ARGUMENT;
    if (sequences == 0) return CIE_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == CIE_F32)
        return walk<float>(s, delta_args<float>(proj, ldp, q_off, k_off, v_off, g_off, b_off, a_off, taps_w, taps, a_log, dt_bias,
                                                q_scale, state, past, seq_slot, q_start_loc, heads, kv_heads, dim, vdim),
                           WalkOut<float>{norm_weight, eps, static_cast<float*>(out), y, slice, chunk}, sequences,
                           rows_per_thread, columns_per_thread, threads);
    if (dtype == CIE_BF16)
        return walk<bf16_t>(s, delta_args<bf16_t>(proj, ldp, q_off, k_off, v_off, g_off, b_off, a_off, taps_w, taps, a_log, dt_bias,
                                                  q_scale, state, past, seq_slot, q_start_loc, heads, kv_heads, dim, vdim),
                            WalkOut<bf16_t>{norm_weight, eps, static_cast<bf16_t*>(out), y, slice, chunk}, sequences,
                            rows_per_thread, columns_per_thread, threads);
    return CIE_BAD_ARGUMENT;
}

// The same in blocks of 32 tokens on the matrix cores; `y` gets the raw read-out.  Scratch, float32: `rows`
// [tokens, 2 kv_heads padded], `values` [tokens, heads vdim], `steps` [2, tokens, heads], and for
// tokens / 32 + sequences + 1 blocks `blocks` with heads * (32 * wide + 32 * cols16 + 32 * 32 + 64) + kv_heads * 64 * wide
// numbers each; padded and cols16 are dim and vdim rounded up to multiples of 16, wide is dim rounded up to one of 64.
CIE_API int cie_delta_blocks(void* stream, int dtype, const void* proj, long ldp, int q_off, int k_off, int v_off, int g_off,
                             int b_off, int a_off, const void* taps_w, int taps, const float* a_log, const float* dt_bias,
                             float q_scale, float* state, float* past, const int* seq_of_token, const int* seq_slot,
                             const int* q_start_loc, float* y, float* rows, float* values, float* steps, float* blocks,
                             int tokens, int sequences, int heads, int kv_heads, int dim, int vdim) {
    if (bad_delta(sequences, heads, kv_heads, dim, vdim, taps, ldp, q_off, k_off, v_off, g_off, b_off, a_off) || dim > 256 ||
        tokens < 0 || !proj || !taps_w || !a_log || !dt_bias || !state || !past || !y || !rows || !values || !steps || !blocks)
        return CIE_BAD_ARGUMENT;
    const int padded = (dim + 15) / 16 * 16;
    const int cols16 = (vdim + 15) / 16 * 16;
    const int most_blocks = (tokens + kBlock - 1) / kBlock;  // (of one sequence)
    const size_t lds = sizeof(float) * (static_cast<size_t>(kBlock) * (padded + 4) + 2 * kBlock * kTri + 16 * 20 + 2 * kBlock);
    const int channels = dim <= kWave ? 1 : dim <= 2 * kWave ? 2 : 4;  // of a head that a lane takes
    const int pieces = (vdim + channels * kWave - 1) / (channels * kWave);
    const long prepare = (static_cast<long>((tokens + kRun - 1) / kRun) * (2 * kv_heads + static_cast<long>(heads) * pieces) + 3) / 4;
    if (lds > 64 * 1024 || most_blocks > 65535 || cols16 / 16 > 65535 || static_cast<long>(sequences) * heads > 0x7fffffffL ||
        prepare > 0x7fffffffL)
        return CIE_BAD_ARGUMENT;
    if (sequences == 0 || tokens == 0) return CIE_OK;
    const size_t places = static_cast<size_t>(tokens) / kBlock + sequences + 1;
    const size_t units = places * heads;
    const size_t pair = 2 * kWave;  // the two operand tiles of a block
    BlockArgs b;
    b.rows = rows;
    b.values = values;
    b.beta = steps;
    b.logs = steps + static_cast<size_t>(tokens) * heads;
    b.tiles = (dim + 63) / 64 * 4;
    b.w = reinterpret_cast<float4*>(blocks);
    b.q = b.w + units * b.tiles * pair;
    b.k = b.q + places * kv_heads * b.tiles * pair;
    b.u = b.k + places * kv_heads * b.tiles * pair;
    b.p = b.u + units * (cols16 / 16) * pair;
    b.fade = reinterpret_cast<float*>(b.p + units * 2 * pair);
    b.state = state;
    b.seq_slot = seq_slot;
    b.q_start_loc = q_start_loc;
    b.y = y;
    b.heads = heads;
    b.kv_heads = kv_heads;
    b.dim = dim;
    b.vdim = vdim;
    b.padded = padded;
    b.cols16 = cols16;
    hipStream_t s = static_cast<hipStream_t>(stream);
#define CIE_DELTA_ARGS(T)                                                                                              \
    delta_args<T>(proj, ldp, q_off, k_off, v_off, g_off, b_off, a_off, taps_w, taps, a_log, dt_bias, q_scale, state, past, \
                  seq_slot, q_start_loc, heads, kv_heads, dim, vdim)
#define CIE_DELTA_PREPARE(T, NC) \
    delta_prepare_kernel<T, NC><<<static_cast<unsigned>(prepare), 256, 0, s>>>(CIE_DELTA_ARGS(T), b, seq_of_token, tokens, pieces)
    if (dtype == CIE_F32 && channels == 1) CIE_DELTA_PREPARE(float, 1);
    else if (dtype == CIE_F32 && channels == 2) CIE_DELTA_PREPARE(float, 2);
    else if (dtype == CIE_F32) CIE_DELTA_PREPARE(float, 4);
    else if (dtype == CIE_BF16 && channels == 1) CIE_DELTA_PREPARE(bf16_t, 1);
    else if (dtype == CIE_BF16 && channels == 2) CIE_DELTA_PREPARE(bf16_t, 2);
    else if (dtype == CIE_BF16) CIE_DELTA_PREPARE(bf16_t, 4);
    else return CIE_BAD_ARGUMENT;
#undef CIE_DELTA_PREPARE
    if (hipGetLastError() != hipSuccess) return CIE_LAUNCH_FAILED;
    delta_block_kernel<<<dim3(sequences * heads, most_blocks), 256, lds, s>>>(b);
    if (hipGetLastError() != hipSuccess) return CIE_LAUNCH_FAILED;
    const dim3 scan_grid(sequences * heads, cols16 / 16);
    if (b.tiles == 4)
        delta_scan_kernel<1><<<scan_grid, 256, 0, s>>>(b);
    else if (b.tiles == 8)
        delta_scan_kernel<2><<<scan_grid, 256, 0, s>>>(b);
    else if (b.tiles == 12)
        delta_scan_kernel<3><<<scan_grid, 256, 0, s>>>(b);
    else
        delta_scan_kernel<4><<<scan_grid, 256, 0, s>>>(b);
    if (hipGetLastError() != hipSuccess) return CIE_LAUNCH_FAILED;
    if (dtype == CIE_F32)
        delta_keep_kernel<float><<<dim3(sequences, heads), 256, 0, s>>>(CIE_DELTA_ARGS(float));
    else
        delta_keep_kernel<bf16_t><<<dim3(sequences, heads), 256, 0, s>>>(CIE_DELTA_ARGS(bf16_t));
#undef CIE_DELTA_ARGS
    return cie_after_launch();
}
