// Paged grouped-query attention whose scores are shaped before the softmax, and the kernel that prepares its
// heads.  Every shaping step is a parameter and may be left out:
//
//   s_ij = (q_i . k_j) * scale
//   s_ij <- cap * tanh(s_ij / cap)                       cap > 0
//   s_ij <- s_ij - slope[head] * (i - j)                 slopes given (a bias on the distance itself)
//   j is seen by i when 0 <= i - j < window              window > 0 (else every j <= i)
//   ... or, beside the window, when j < keep <= ...       keep > 0: the first `keep` keys of the sequence stay visible
//                                                        to every later token, at their own positions
//   ... or when j <= i and floor(i / chunk) = floor(j / chunk)   chunk > 0: chunks counted from position 0
//   p_ij = exp(s_ij) / (sum_j exp(s_ij) + exp(sink[head]))   sinks given: one more term in the denominator, which
//                                                        has no key and no value, no scale and no bias
//   o_i  = sum_j p_ij v_j,  o_i <- o_i * sigmoid(gate[i, head])   gate given; or, with a gate per number of the head,
//                                                        o_i[d] <- o_i[d] * sigmoid(gate[i, head * vdim + d])
//
// Differential heads (two maps): queries and keys come in pairs, every map is a softmax of its own over the same values,
// and  o_i = (a1_i - lambda a2_i) / sqrt(mean((a1_i - lambda a2_i)^2) + eps) * factor  over the head's vdim numbers.  A
// query or key row then holds its two maps one after the other (D numbers in all).
//
// Keys have D numbers per head, values DV (the two may differ).  Cache layout as everywhere in this library:
// keys [pages, kv_heads, page_size, D], values transposed [pages, kv_heads, DV, page_size].  Scores, the softmax,
// the value sums and the gate are float32 in both storage types.
//
// `cie_heads_prepare` is what stands between the projection and this attention: a per-head RMS norm of queries
// and keys (with a weight, without one, or none; or one RMS norm over all query heads of a token together and one
// over all its key heads, with a weight per number of the projection), the queries' factor that grows with the position,
//   q <- q * (1 + coef * ln(floor((p + 1) / every) + 1)),
// then a rotation of the first `rot` numbers of every query and key head by the position (pairs of neighbours or of
// the two halves; cos and sin from float32 tables [positions, rot / 2]),
// queries laid out [tokens, heads, D] (zero-padded from the projection's head size up to D) and keys and values
// written to the cache (padded likewise).  Statistics, the logarithm and the scaling are float32.
#include "attention_args.h"
#include "common.h"

using namespace cie_attention;

namespace {

// ------------------------------------------------------------------------------------------------ prepare
// A wave's sum of the squares of n numbers: sixteen bytes a lane and load where the numbers start at a multiple of
// sixteen bytes (every wave of a token sums the whole projection again under the norm over all heads: the loads
// are what that costs).
__device__ __forceinline__ float wave_sum_squares(const float* p, int n, int lane) {
    float sum = 0.f;
    int done = 0;
    if ((reinterpret_cast<uintptr_t>(p) & 15) == 0) {
        for (int d = 4 * lane; d + 3 < n; d += 4 * kWave) {
            const float4 v = *reinterpret_cast<const float4*>(p + d);
            sum += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
        }
        done = n & ~3;
    }
    for (int d = done + lane; d < n; d += kWave) sum += p[d] * p[d];
    return wave_sum(sum);
}
__device__ __forceinline__ float wave_sum_squares(const bf16_t* p, int n, int lane) {
    float sum = 0.f;
    int done = 0;
    if ((reinterpret_cast<uintptr_t>(p) & 15) == 0) {
        for (int d = 8 * lane; d + 7 < n; d += 8 * kWave) {
            const uint4 raw = *reinterpret_cast<const uint4*>(p + d);
            const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const float lo = __uint_as_float(w[i] << 16), hi = __uint_as_float(w[i] & 0xffff0000u);
                sum += lo * lo + hi * hi;
            }
        }
        done = n & ~7;
    }
    for (int d = done + lane; d < n; d += kWave) {
        const float x = to_float(p[d]);
        sum += x * x;
    }
    return wave_sum(sum);
}

// One wave per (token, head slot): slots 0..H-1 queries, H..H+G-1 keys, H+G..H+G+V-1 values.  With `maps` > 1 the query and
// key heads come in runs of that many (the maps of one head), laid side by side in the rows and in the cache; there are
// V = kv_heads value heads, and H = maps * q_heads, G = maps * kv_heads.
template <typename T>
__global__ void __launch_bounds__(256)
heads_prepare_kernel(const T* __restrict__ proj, int proj_stride, int q_off, int k_off, int v_off,
                     const float* __restrict__ q_weight, const float* __restrict__ k_weight, int norm_mode,
                     float eps, float temp_coef, int temp_every, const int* __restrict__ positions,
                     const int* __restrict__ seq_of_token, const int* __restrict__ seq_slot,
                     const int* __restrict__ block_table, int table_width, T* __restrict__ q_out,
                     T* __restrict__ k_pool, T* __restrict__ v_pool, int tokens, int q_heads, int kv_heads,
                     int dim, int vdim, int D, int DV, int page_shift, int write_kv,
                     const float* __restrict__ cos_table, const float* __restrict__ sin_table, int rot, int neighbours,
                     int maps) {
    const int lane = threadIdx.x % kWave;
    const int value_heads = kv_heads;
    q_heads *= maps;
    kv_heads *= maps;
    const int slots = q_heads + kv_heads + value_heads;
    const long unit = static_cast<long>(blockIdx.x) * (blockDim.x / kWave) + threadIdx.x / kWave;
    if (unit >= static_cast<long>(tokens) * slots) return;
    const int token = static_cast<int>(unit / slots);
    const int slot = static_cast<int>(unit - static_cast<long>(token) * slots);
    const int pos = positions[token];
    const T* row = proj + static_cast<size_t>(token) * proj_stride;
    const int page_size = 1 << page_shift;
    size_t page = 0;
    if (slot >= q_heads) {
        if (!write_kv) return;
        const int* table = block_table + static_cast<size_t>(seq_slot[seq_of_token[token]]) * table_width;
        page = static_cast<size_t>(table[pos >> page_shift]);
    }
    if (slot >= q_heads + kv_heads) {  // a value head: copied, padded, into the transposed pool
        const int head = slot - q_heads - kv_heads;
        const T* src = row + v_off + head * vdim;
        T* dst = v_pool + ((page * value_heads + head) * DV << page_shift) + (pos & (page_size - 1));
        for (int d = lane; d < DV; d += kWave)
            dst[static_cast<size_t>(d) << page_shift] = d < vdim ? src[d] : from_float<T>(0.f);
        return;
    }
    const bool is_q = slot < q_heads;
    const int head = is_q ? slot : slot - q_heads;
    const T* src = row + (is_q ? q_off : k_off) + head * dim;
    const float* weight = is_q ? q_weight : k_weight;
    float factor = 1.f;
    if (norm_mode == 3) {  // one root mean square over all heads of the projection; the weight has a number for each
        const int all = (is_q ? q_heads : kv_heads) * dim;
        const T* whole = row + (is_q ? q_off : k_off);
        factor = 1.0f / sqrtf(wave_sum_squares(whole, all, lane) / static_cast<float>(all) + eps);
        weight += head * dim;
    } else if (norm_mode != 0) {
        float sum_sq = 0.f;
        for (int d = lane; d < dim; d += kWave) {
            const float x = to_float(src[d]);
            sum_sq += x * x;
        }
        factor = 1.0f / sqrtf(wave_sum(sum_sq) / static_cast<float>(dim) + eps);
    }
    const bool weighted = norm_mode >= 2;
    float after = 1.f;  // the queries' factor of the position
    if (is_q && temp_every > 0)
        after = 1.0f + temp_coef * logf(static_cast<float>((pos + 1) / temp_every) + 1.0f);
    T* dst = is_q ? q_out + (static_cast<size_t>(token) * q_heads + head) * D
                  : k_pool + ((((page * value_heads + head / maps) << page_shift) + (pos & (page_size - 1))) * maps + head % maps) * D;
    const int half = rot / 2;
    const float* cos_row = rot > 0 ? cos_table + static_cast<size_t>(pos) * half : nullptr;
    const float* sin_row = rot > 0 ? sin_table + static_cast<size_t>(pos) * half : nullptr;
    for (int d = lane; d < D; d += kWave) {
        float x = 0.f;
        if (d < dim) {
            x = to_float(src[d]) * factor;
            if (weighted) x *= weight[d];
            if (d < rot) {
                // the pair (u, v) of the angle's index i turns to (u cos - v sin, v cos + u sin): neighbours
                // (2i, 2i + 1) or the halves (i, i + rot / 2)
                const int i = neighbours ? d >> 1 : (d < half ? d : d - half);
                const bool is_u = neighbours ? !(d & 1) : d < half;
                const int mate = neighbours ? d ^ 1 : (is_u ? d + half : d - half);
                float y = to_float(src[mate]) * factor;
                if (weighted) y *= weight[mate];
                const float c = cos_row[i], sn = sin_row[i];
                x = is_u ? x * c - y * sn : x * c + y * sn;
            }
            x *= after;
        }
        dst[d] = from_float<T>(x);
    }
}

// The same preparation for heads whose projections first pass a causal convolution over the tokens, channel by channel:
//   y_t = sum_j taps[j, c] u_(t - n + 1 + j)   (the last tap meets the token itself),
// with the inputs of the tokens before the step in `past` [slots, max(n - 1, 1), channels] (float32, oldest first; the
// channels are those of the queries, the keys and the values in that order), and for values that are mixed with those
// that an earlier layer of the same step made of the same tokens:
//   v <- (1 - mix) v + mix * v_first,   the mixed v being what is cached.
// A layer that is the first of those leaves its convolved values in `first_out`.
template <typename T>
struct ConvHeads {
    const T* taps;         // [n, channels]; null: the projection as it is (n = 1)
    int n;
    float* past;
    const int* q_start_loc;
    int single;            // every sequence of the step brings one token: the kernel also moves `past` on
    T* first_out;          // [tokens, kv_heads * vdim] or null
    const T* first_in;     // likewise
    float mix;
};
constexpr int kMaxConvTaps = 16;  // inputs that `past` keeps, at most, and one

// Numbers d and d + 1 of a row; as one load where every row's start allows it.
__device__ __forceinline__ float2 load_pair(const float* p, int d, int n, bool paired) {
    if (paired) return *reinterpret_cast<const float2*>(p + d);
    return float2{p[d], d + 1 < n ? p[d + 1] : 0.f};
}
__device__ __forceinline__ float2 load_pair(const bf16_t* p, int d, int n, bool paired) {
    if (paired) {
        const uint32_t raw = *reinterpret_cast<const uint32_t*>(p + d);
        return float2{__uint_as_float(raw << 16), __uint_as_float(raw & 0xffff0000u)};
    }
    return float2{to_float(p[d]), d + 1 < n ? to_float(p[d + 1]) : 0.f};
}
__device__ __forceinline__ void store_pair(float* p, float2 v) { *reinterpret_cast<float2*>(p) = v; }
__device__ __forceinline__ void store_pair(bf16_t* p, float2 v) { *reinterpret_cast<uint32_t*>(p) = pack_bf16(v.x, v.y); }

// One wave per (run of RUN tokens of the step, head slot); slots as above.  A lane holds neighbours 2l, 2l + 1 of the head
// (CHUNKS = 2: and those 128 further on) for all of the run's tokens: a projected row is read once for all taps, the taps and
// what a token's place leads to (sequence, slot, page) once a run, and eight values of a channel are stored together where
// they lie side by side in the transposed pool.  TAPS: the convolution's taps where the kernel knows them, 0 (runs of one
// token only): c.n of them.
template <typename T, int TAPS, int RUN, int CHUNKS>
__global__ void __launch_bounds__(256)
heads_conv_prepare_kernel(const T* __restrict__ proj, int proj_stride, int q_off, int k_off, int v_off, ConvHeads<T> c,
                          const float* __restrict__ q_weight, const float* __restrict__ k_weight, int norm_mode, float eps,
                          float temp_coef, int temp_every, const int* __restrict__ positions,
                          const int* __restrict__ seq_of_token, const int* __restrict__ seq_slot,
                          const int* __restrict__ block_table, int table_width, T* __restrict__ q_out,
                          T* __restrict__ k_pool, T* __restrict__ v_pool, int tokens, int q_heads, int kv_heads, int dim,
                          int vdim, int D, int DV, int page_shift, const float* __restrict__ cos_table,
                          const float* __restrict__ sin_table, int rot, int neighbours) {
    static_assert(TAPS > 0 || RUN == 1, "runs of several tokens know their taps");
    constexpr int kTaps = TAPS > 0 ? TAPS : kMaxConvTaps;
    constexpr int kRows = RUN + kTaps - 1;
    __shared__ float staged[4][128 * CHUNKS];  // a head of each wave, for partners that another lane holds
    const int lane = threadIdx.x % kWave;
    const int wave = threadIdx.x / kWave;
    const int slots = q_heads + 2 * kv_heads;
    const long unit = static_cast<long>(blockIdx.x) * 4 + wave;
    if (unit >= static_cast<long>((tokens + RUN - 1) / RUN) * slots) return;
    const int token0 = static_cast<int>(unit / slots) * RUN;
    const int slot = static_cast<int>(unit - static_cast<long>(token0 / RUN) * slots);
    const int count = min(RUN, tokens - token0);
    const bool is_q = slot < q_heads, is_v = slot >= q_heads + kv_heads;
    const int head = is_q ? slot : is_v ? slot - q_heads - kv_heads : slot - q_heads;
    const int n = is_v ? vdim : dim;
    const int padded = is_v ? DV : D;
    const int column = (is_q ? q_off : is_v ? v_off : k_off) + head * n;
    const int channels = (q_heads + kv_heads) * dim + kv_heads * vdim;
    const int channel = is_v ? (q_heads + kv_heads) * dim + head * vdim : (is_q ? 0 : q_heads * dim) + head * dim;
    const int taps = TAPS > 0 ? TAPS : c.n;
    const bool paired = (((proj_stride | column | n) & 1) == 0);  // (the base of `proj` is aligned to a pair)
    const bool paired_channels = (((channels | channel | n) & 1) == 0);
    // lane i knows the place of the run's token i
    const int mine = token0 + min(lane, count - 1);
    const int my_pos = positions[mine];
    const int my_seq = seq_of_token[mine];
    const int my_slot = seq_slot[my_seq];
    const int my_first = c.q_start_loc[my_seq];
    const int my_page = is_q ? 0 : block_table[static_cast<size_t>(my_slot) * table_width + (my_pos >> page_shift)];
    auto of = [&](int value, int tt) { return __builtin_amdgcn_readlane(value, tt); };

    // what the steps behind the convolution need from memory is asked for in front of it: single tokens wait for one round
    // of loads instead of three
    const float* weight = norm_mode == 2 && !is_v ? (is_q ? q_weight : k_weight) : nullptr;
    const int half = rot / 2;
    float2 scale[CHUNKS], turn[CHUNKS];  // (`turn`: runs of one token only)
#pragma unroll
    for (int i = 0; i < CHUNKS; ++i) {
        const int d = 2 * lane + 128 * i;
        scale[i] = float2{weight && d < n ? weight[d] : 1.f, weight && d + 1 < n ? weight[d + 1] : 1.f};
        turn[i] = float2{1.f, 0.f};
        if (RUN == 1 && neighbours && !is_v && d < rot) {
            const size_t at = static_cast<size_t>(of(my_pos, 0)) * half + (d >> 1);
            turn[i] = float2{cos_table[at], sin_table[at]};
        }
    }

    float2 y[RUN][CHUNKS];
    float sum_sq[RUN];
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) sum_sq[tt] = 0.f;
#pragma unroll
    for (int i = 0; i < CHUNKS; ++i) {
        const int d = 2 * lane + 128 * i;
#pragma unroll
        for (int tt = 0; tt < RUN; ++tt) y[tt][i] = float2{0.f, 0.f};
        if (d >= n) continue;
        const bool two = d + 1 < n;
        float2 u[kRows];  // the projected rows token0 - (taps - 1) and on (a place in front of the step's first row: not used)
        float2 w[kTaps];
#pragma unroll
        for (int r = 0; r < kRows; ++r) {
            if (TAPS == 0 && r >= taps) break;
            const int row = min(max(token0 - (taps - 1) + r, 0), tokens - 1);
            u[r] = load_pair(proj + static_cast<size_t>(row) * proj_stride + column, d, n, paired);
        }
#pragma unroll
        for (int j = 0; j < kTaps; ++j) {
            if (TAPS == 0 && j >= taps) break;
            w[j] = c.taps ? load_pair(c.taps + static_cast<size_t>(j) * channels + channel, d, n, paired_channels) : float2{1.f, 1.f};
        }
#pragma unroll
        for (int tt = 0; tt < RUN; ++tt) {
            if (tt >= count) break;
            const int t = token0 + tt - of(my_first, tt);  // the token's place in the step's portion of its sequence
            float* before = c.past + static_cast<size_t>(of(my_slot, tt)) * max(taps - 1, 1) * channels + channel;
#pragma unroll
            for (int j = 0; j < kTaps; ++j) {
                if (TAPS == 0 && j >= taps) break;
                float2 in = u[tt + j];
                if (t - (taps - 1) + j < 0) {  // (in front of the portion: what earlier steps left)
                    in = load_pair(before + static_cast<size_t>(t + j) * channels, d, n, paired_channels);
                    if (RUN == 1) u[j] = in;
                }
                y[tt][i].x = fmaf(w[j].x, in.x, y[tt][i].x);
                y[tt][i].y = fmaf(w[j].y, in.y, y[tt][i].y);
            }
            if (RUN == 1 && c.single) {  // (t = 0: u[j] is what the state held at j, and the last is the token's own)
#pragma unroll
                for (int j = 1; j < kTaps; ++j) {
                    if (TAPS == 0 && j >= taps) break;
                    float* now = before + static_cast<size_t>(j - 1) * channels + d;
                    if (paired_channels) {
                        store_pair(now, u[j]);
                    } else {
                        now[0] = u[j].x;
                        if (two) now[1] = u[j].y;
                    }
                }
            }
            sum_sq[tt] += y[tt][i].x * y[tt][i].x + y[tt][i].y * y[tt][i].y;
        }
    }
    const int page_mask = (1 << page_shift) - 1;
    if (is_v) {
        // a run of one sequence that lies in one page from a place that is a multiple of eight on
        const bool together = RUN == 8 && sizeof(T) == 2 && count == RUN && of(my_seq, 0) == of(my_seq, RUN - 1) &&
                              page_shift >= 3 && (of(my_pos, 0) & 7) == 0;
#pragma unroll
        for (int i = 0; i < CHUNKS; ++i) {
            const int d = 2 * lane + 128 * i;
            if (d >= padded) continue;
#pragma unroll
            for (int tt = 0; tt < RUN; ++tt) {
                if (tt >= count) break;
                const size_t at = (static_cast<size_t>(token0 + tt) * kv_heads + head) * vdim + d;
                if (c.first_out) {
                    if (d < n) c.first_out[at] = from_float<T>(y[tt][i].x);
                    if (d + 1 < n) c.first_out[at + 1] = from_float<T>(y[tt][i].y);
                }
                if (c.first_in) {
                    if (d < n) y[tt][i].x = (1.0f - c.mix) * y[tt][i].x + c.mix * to_float(c.first_in[at]);
                    if (d + 1 < n) y[tt][i].y = (1.0f - c.mix) * y[tt][i].y + c.mix * to_float(c.first_in[at + 1]);
                }
            }
            if constexpr (RUN == 8 && sizeof(T) == 2) {
                if (together) {
                    T* dst = v_pool + (((static_cast<size_t>(of(my_page, 0)) * kv_heads + head) * DV + d) << page_shift) + (of(my_pos, 0) & page_mask);
                    *reinterpret_cast<uint4*>(dst) = uint4{pack_bf16(y[0][i].x, y[1 % RUN][i].x), pack_bf16(y[2 % RUN][i].x, y[3 % RUN][i].x),
                                                           pack_bf16(y[4 % RUN][i].x, y[5 % RUN][i].x), pack_bf16(y[6 % RUN][i].x, y[7 % RUN][i].x)};
                    *reinterpret_cast<uint4*>(dst + (static_cast<size_t>(1) << page_shift)) =
                        uint4{pack_bf16(y[0][i].y, y[1 % RUN][i].y), pack_bf16(y[2 % RUN][i].y, y[3 % RUN][i].y),
                              pack_bf16(y[4 % RUN][i].y, y[5 % RUN][i].y), pack_bf16(y[6 % RUN][i].y, y[7 % RUN][i].y)};
                    continue;
                }
            }
#pragma unroll
            for (int tt = 0; tt < RUN; ++tt) {
                if (tt >= count) break;
                T* dst = v_pool + (((static_cast<size_t>(of(my_page, tt)) * kv_heads + head) * DV + d) << page_shift) + (of(my_pos, tt) & page_mask);
                dst[0] = from_float<T>(y[tt][i].x);
                dst[static_cast<size_t>(1) << page_shift] = from_float<T>(y[tt][i].y);
            }
        }
        return;
    }
    if (norm_mode != 0) {  // (the tokens' sums side by side: their steps across the lanes do not wait for one another)
#pragma unroll
        for (int offset = kWave / 2; offset > 0; offset >>= 1)
#pragma unroll
            for (int tt = 0; tt < RUN; ++tt) sum_sq[tt] += __shfl_xor(sum_sq[tt], offset, kWave);
    }
#pragma unroll
    for (int tt = 0; tt < RUN; ++tt) {
        if (tt >= count) break;
        const int token = token0 + tt;
        const int pos = of(my_pos, tt);
        float factor = 1.f;
        if (norm_mode != 0) factor = 1.0f / sqrtf(sum_sq[tt] / static_cast<float>(dim) + eps);
        float after = 1.f;  // the queries' factor of the position
        if (is_q && temp_every > 0) after = 1.0f + temp_coef * logf(static_cast<float>((pos + 1) / temp_every) + 1.0f);
#pragma unroll
        for (int i = 0; i < CHUNKS; ++i) {
            const int d = 2 * lane + 128 * i;
            y[tt][i].x *= factor * scale[i].x;
            y[tt][i].y *= factor * scale[i].y;
            if (rot > 0 && !neighbours) {
                if (d < n) staged[wave][d] = y[tt][i].x;
                if (d + 1 < n) staged[wave][d + 1] = y[tt][i].y;
            }
        }
        __builtin_amdgcn_wave_barrier();  // (a wave's LDS operations keep their order; the compiler is held to it too)
        T* dst = is_q ? q_out + (static_cast<size_t>(token) * q_heads + head) * D
                      : k_pool + (((static_cast<size_t>(of(my_page, tt)) * kv_heads + head) << page_shift) + (pos & page_mask)) * D;
        const float* cos_row = rot > 0 ? cos_table + static_cast<size_t>(pos) * half : nullptr;
        const float* sin_row = rot > 0 ? sin_table + static_cast<size_t>(pos) * half : nullptr;
#pragma unroll
        for (int i = 0; i < CHUNKS; ++i) {
            const int d = 2 * lane + 128 * i;
            if (d >= padded) continue;
            float2 x = y[tt][i];
            if (d < rot && neighbours) {  // (rot is even: a pair turns or stays as one)
                const float cs = RUN == 1 ? turn[i].x : cos_row[d >> 1], sn = RUN == 1 ? turn[i].y : sin_row[d >> 1];
                x = float2{y[tt][i].x * cs - y[tt][i].y * sn, y[tt][i].y * cs + y[tt][i].x * sn};
            } else if (d < rot) {
                float turned[2] = {x.x, x.y};
#pragma unroll
                for (int e = 0; e < 2; ++e) {
                    const int at = d + e;
                    const bool is_u = at < half;
                    const float mate = staged[wave][is_u ? at + half : at - half];
                    const int angle = is_u ? at : at - half;
                    turned[e] = is_u ? turned[e] * cos_row[angle] - mate * sin_row[angle] : turned[e] * cos_row[angle] + mate * sin_row[angle];
                }
                x = float2{turned[0], turned[1]};
            }
            x.x *= after;
            x.y *= after;
            store_pair(dst + d, x);
        }
        __builtin_amdgcn_wave_barrier();
    }
}

// ------------------------------------------------------------------------------------------------ generic
// One workgroup (4 waves) per (query token, query head); each wave takes 64-key chunks in turn, one key per
// lane for the scores, then one slice of the value head per lane; the four running (max, sum, accumulator)
// triples meet in LDS.  Any D, DV that are multiples of 8 up to 256; float32 or bfloat16 storage.
// With `maps` = 2 a query or key row holds two maps of D numbers each; they are walked one after the other.
constexpr int kMaxSlices = 4;       // pieces of 64 numbers of a value head that a lane keeps ...
constexpr int kMaxWideSlices = 16;  // ... and in the form for wide values

template <typename T>
__device__ __forceinline__ void load8(const T* p, float (&v)[8]);
template <>
__device__ __forceinline__ void load8<float>(const float* p, float (&v)[8]) {
    const float4 a = *reinterpret_cast<const float4*>(p);
    const float4 b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
    v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
template <>
__device__ __forceinline__ void load8<bf16_t>(const bf16_t* p, float (&v)[8]) {
    const uint4 raw = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[2 * i] = __uint_as_float(w[i] << 16);
        v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}

struct ScoreShape {
    float scale;
    float softcap;        // <= 0: none
    const float* slopes;  // [q_heads] or null
    const float* sinks;   // [q_heads] or null
    int window;           // <= 0: all keys
    int chunk;            // > 0: i sees j <= i only inside its own chunk, floor(i / chunk) == floor(j / chunk)
    int keep;             // > 0 (with a window): keys 0 .. keep - 1 are seen from behind the window too
    int gate_wide;        // the gate has a number for every number of the head (head * vdim + d), not one per head
    int vdim;             // numbers of a value head that are not padding
    float lambda;         // two maps: the second one's weight ...
    float factor;         // ... the factor behind the norm of their difference ...
    float eps;            // ... and that norm's eps
};

// The first key that the query at position `pos` sees.
__device__ __forceinline__ int first_seen(int pos, int window, int chunk) {
    if (chunk > 0) return pos < 0 ? 0 : pos - pos % chunk;
    return window > 0 ? max(0, pos + 1 - window) : 0;
}

template <typename T, int SLICES>
__global__ void __launch_bounds__(256)
scored_attention_generic_kernel(const T* __restrict__ q, const T* __restrict__ k_pool, const T* __restrict__ v_pool,
                                const int* __restrict__ block_table, int table_width,
                                const int* __restrict__ positions, const int* __restrict__ seq_of_token,
                                const int* __restrict__ seq_slot, const T* __restrict__ gate, int gate_stride,
                                T* __restrict__ out, long out_stride, int q_heads, int kv_heads, int D, int DV, int page_size,
                                int maps, ScoreShape shape) {
    extern __shared__ float lds[];
    float* q_s = lds;            // [D]
    float* acc_s = lds + D;      // [4][DV]
    float* done_s = acc_s + 4 * DV;  // [maps][DV]
    __shared__ float m_s[4];
    __shared__ float l_s[4];
    __shared__ float scratch[16];

    const int token = blockIdx.x;
    const int head = blockIdx.y;
    const int lane = threadIdx.x % kWave;
    const int wave = threadIdx.x / kWave;
    const int kv_head = head / (q_heads / kv_heads);
    const int pos = positions[token];
    const int len = pos + 1;
    const int lo = first_seen(pos, shape.window, shape.chunk);
    const int* table = block_table + static_cast<size_t>(seq_slot[seq_of_token[token]]) * table_width;
    const float slope = shape.slopes ? shape.slopes[head] : 0.f;

    // the keys in the order they are walked: the kept first ones that lie in front of the window, then the window's
    const int kept = (shape.window > 0 && shape.keep > 0) ? min(shape.keep, lo) : 0;
    const int walk = kept + len - lo;
    for (int map = 0; map < maps; ++map) {
        __syncthreads();  // (the map before has been read out)
        const T* q_row = q + ((static_cast<size_t>(token) * q_heads + head) * maps + map) * D;
        for (int d = threadIdx.x; d < D; d += blockDim.x) q_s[d] = to_float(q_row[d]);
        __syncthreads();

        float m = -INFINITY;
        float l = 0.f;
        float acc[SLICES];
#pragma unroll
        for (int i = 0; i < SLICES; ++i) acc[i] = 0.f;
        for (int base = wave * kWave; base < walk; base += 4 * kWave) {
            const int at = base + lane;
            const int key = at < kept ? at : at - kept + lo;
            const bool valid = at < walk;
            float s = -INFINITY;
            uint32_t head_block = 0;
            uint32_t in_page = 0;
            if (valid) {
                const int page = table[key / page_size];
                head_block = static_cast<uint32_t>(page) * kv_heads + kv_head;
                in_page = key % page_size;
                const T* k_row = k_pool + ((static_cast<size_t>(head_block) * page_size + in_page) * maps + map) * D;
                float dot = 0.f;
                for (int d = 0; d < D; d += 8) {
                    float kk[8];
                    load8<T>(k_row + d, kk);
#pragma unroll
                    for (int j = 0; j < 8; ++j) dot = fmaf(q_s[d + j], kk[j], dot);
                }
                s = dot * shape.scale;
                if (shape.softcap > 0.f) s = shape.softcap * tanhf(s / shape.softcap);
                s -= slope * static_cast<float>(pos - key);
            }
            const float m_new = fmaxf(m, wave_max(s));  // finite: lane 0 of every chunk is valid
            const float alpha = expf(m - m_new);
            const float p = valid ? expf(s - m_new) : 0.f;
            l = l * alpha + wave_sum(p);
#pragma unroll
            for (int i = 0; i < SLICES; ++i) acc[i] *= alpha;
            const int count = min(kWave, walk - base);
            for (int j = 0; j < count; ++j) {
                const float pj = __shfl(p, j, kWave);
                const uint32_t block_j = __shfl(head_block, j, kWave);
                const uint32_t in_page_j = __shfl(in_page, j, kWave);
                const T* v_column = v_pool + static_cast<size_t>(block_j) * page_size * DV + in_page_j;
#pragma unroll
                for (int i = 0; i < SLICES; ++i) {
                    const int d = lane + kWave * i;
                    if (d < DV) acc[i] = fmaf(pj, to_float(v_column[static_cast<size_t>(d) * page_size]), acc[i]);
                }
            }
            m = m_new;
        }
        if (lane == 0) {
            m_s[wave] = m;
            l_s[wave] = l;
        }
#pragma unroll
        for (int i = 0; i < SLICES; ++i) {
            const int d = lane + kWave * i;
            if (d < DV) acc_s[wave * DV + d] = acc[i];
        }
        __syncthreads();
        float m_all = m_s[0];
        for (int w = 1; w < 4; ++w) m_all = fmaxf(m_all, m_s[w]);
        const float sink = shape.sinks ? shape.sinks[head] : -INFINITY;
        m_all = fmaxf(m_all, sink);
        float den = shape.sinks ? expf(sink - m_all) : 0.f;
        float e[4];
        for (int w = 0; w < 4; ++w) {
            e[w] = expf(m_s[w] - m_all);  // a wave that saw no key has m = -inf: weight 0
            den += l_s[w] * e[w];
        }
        for (int d = threadIdx.x; d < DV; d += blockDim.x) {
            float num = 0.f;
            for (int w = 0; w < 4; ++w) num += acc_s[w * DV + d] * e[w];
            done_s[map * DV + d] = num / den;
        }
    }
    // (a thread reads the numbers of `done_s` that it wrote itself)
    float by = 1.f;
    if (maps > 1) {
        float sum = 0.f;
        for (int d = threadIdx.x; d < shape.vdim; d += blockDim.x) {
            const float x = done_s[d] - shape.lambda * done_s[DV + d];
            done_s[d] = x;
            sum += x * x;
        }
        by = shape.factor / sqrtf(block_sum(sum, scratch) / static_cast<float>(shape.vdim) + shape.eps);
    }
    const T* gates = gate ? gate + static_cast<size_t>(token) * gate_stride : nullptr;
    T* out_row = out + static_cast<size_t>(token) * out_stride + head * DV;
    for (int d = threadIdx.x; d < DV; d += blockDim.x) {
        float x = d < shape.vdim ? done_s[d] * by : 0.f;
        if (gates && d < shape.vdim)
            x *= 1.0f / (1.0f + expf(-to_float(gates[shape.gate_wide ? head * shape.vdim + d : head])));
        out_row[d] = from_float<T>(x);
    }
}

// ------------------------------------------------------------------------------------------------ matrix cores
// bfloat16.  A workgroup of four waves per (tile, kv head); a tile is up to `tokens_per_tile` consecutive query
// tokens of one sequence, its rows the (token, head of the group) pairs: row = token * G + head, at most 16 * RT.
// Wave w takes every fourth block of 32 keys of the range the tile can see, so each key and value is read once
// per workgroup.  Per block, as in the other matrix-core attention kernels of this library:
//   S^T[key, row] = K[key, :] . Q[row, :]   v_mfma_f32_16x16x32_bf16, A = K, B = Q; lane (r = lane % 16,
//   g = lane / 16) then holds, for row r, the scores of keys g*4 .. g*4+3 of each 16-key tile, which is the A-operand
//   layout of P in  O[row, d] += P[row, key] * V[key, d]  (B = rows of the transposed values).
// The softmax runs in base 2 (scores, cap, bias and sink are brought there once).  The four waves' running
// (max, sum, accumulator) meet in LDS, one wave after the other, and all threads write the tile's rows.  Few tiles
// over many keys (single tokens behind long windows) have their keys cut into shares, a workgroup each, whose
// (max, sum, accumulator) a second kernel joins; sink and gate are then applied there.  The accumulator is rescaled
// only in blocks where some row's maximum moved, and keys are masked only in blocks that reach an edge of some row.
struct ScoredArgs {
    const bf16_t* q;          // [tokens, q_heads, D]
    const bf16_t* k_pool;
    const bf16_t* v_pool;
    const int* block_table;
    int table_width;
    const int* tile_seq;      // null: tile i is the first tile of sequence i
    const int* tile_q0;
    const int* seq_slot;
    const int* seq_start;
    const int* seq_q_len;
    const int* q_start_loc;
    const bf16_t* gate;       // [tokens, gate_stride], column = head; or null
    int gate_stride;
    bf16_t* out;              // [tokens, q_heads, DV], rows out_stride numbers apart
    long out_stride;
    int q_heads;
    int kv_heads;
    int page_shift;
    int tokens_per_tile;
    int n_tiles;
    int n_splits;        // > 1: the keys of a tile in that many shares of keys_per_split (a multiple of 128), one
    int keys_per_split;  // workgroup each (blockIdx.z); the shares' sums meet in scored_attention_merge_kernel
    float* part_o;       // [tiles, kv_heads, splits, rows, DV]
    float* part_ml;      // [tiles, kv_heads, splits, rows, 2]
    ScoreShape shape;
};

constexpr int kScoredWaves = 4;
constexpr float kLog2e = 1.44269504088896341f;

__device__ __forceinline__ float fast_tanh(float y) {
    // tanh(y) = 1 - 2 / (exp(2y) + 1); exp through the hardware's base-2 exponential
    const float e = __builtin_amdgcn_exp2f(fminf(y * (2.f * kLog2e), 126.f));
    return 1.f - 2.f * __builtin_amdgcn_rcpf(e + 1.f);
}

// A head's read-out (number d in x[d / 64] of lane d % 64), normed where it is a difference of two maps, gated, stored.
template <int MAPS, int DV, int N>
__device__ __forceinline__ void write_head(const ScoredArgs& a, const float (&x)[N], size_t token, int head, int lane) {
    float factor = 1.f;
    if (MAPS == 2) {
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < N; ++i) sum += x[i] * x[i];  // (padding is zero)
        factor = a.shape.factor / sqrtf(wave_sum(sum) / static_cast<float>(a.shape.vdim) + a.shape.eps);
    }
    const bf16_t* gates = a.gate ? a.gate + token * a.gate_stride : nullptr;
    if (gates && !a.shape.gate_wide) factor *= 1.0f / (1.0f + __expf(-to_float(gates[head])));
    bf16_t* dst = a.out + token * a.out_stride + head * DV;
#pragma unroll
    for (int i = 0; i < N; ++i) {
        const int d = lane + i * kWave;
        if (d >= DV) continue;
        float y = x[i] * factor;
        if (gates && a.shape.gate_wide && d < a.shape.vdim)
            y *= 1.0f / (1.0f + __expf(-to_float(gates[head * a.shape.vdim + d])));
        dst[d] = from_float<bf16_t>(y);
    }
}

// MAPS = 2: rows of the first map fill the first RT / 2 tiles of 16, the same rows of the second map the others; the two
// maps of a query or key row lie side by side, D / 2 numbers each.
template <int D, int DV, int RT, int MAPS>
__global__ void __launch_bounds__(64 * kScoredWaves, RT * (D / 4 + DV) <= 2 * (32 + 128) ? 2 : 1)
scored_attention_mfma_kernel(ScoredArgs a) {
    constexpr int MD = D / MAPS;      // numbers of a map
    constexpr int NK = MD / 32;
    constexpr int ND = DV / 16;
    constexpr int ROWS = 16 * RT;
    constexpr int RTM = RT / MAPS;    // tiles of a map
    constexpr int MROWS = 16 * RTM;   // rows of a map
    constexpr int STEP = kKeysPerBlock * kScoredWaves;
    __shared__ float m_s[kScoredWaves][ROWS];
    __shared__ float l_s[kScoredWaves][ROWS];
    __shared__ float o_s[ROWS][DV + 1];
    const int lane = threadIdx.x & (kWave - 1);
    const int wave = threadIdx.x / kWave;
    const int r = lane & 15;
    const int g = lane >> 4;
    const int tile = a.n_tiles - 1 - static_cast<int>(blockIdx.x);  // the last tiles of a prompt see the most keys
    const int kv_head = blockIdx.y;
    const int group = a.q_heads / a.kv_heads;
    const int seq = a.tile_seq ? a.tile_seq[tile] : tile;
    const int q0 = a.tile_seq ? a.tile_q0[tile] : 0;
    const int start = a.seq_start[seq];
    const int n_tok = min(a.tokens_per_tile, a.seq_q_len[seq] - q0);
    const int n_rows = n_tok * group;
    const int first_row_token = a.q_start_loc[seq] + q0;
    const int page_mask = (1 << a.page_shift) - 1;
    const int* table = a.block_table + static_cast<size_t>(a.seq_slot[seq]) * a.table_width;
    const float scale = a.shape.scale;
    const float cap = a.shape.softcap;
    const float inv_cap = cap > 0.f ? 1.0f / cap : 0.f;
    const int window = a.shape.window;

    const int hi = start + q0 + n_tok;
    const int chunk = a.shape.chunk;
    const int lo = first_seen(start + q0, window, chunk);
    // The blocks of keys are walked in an order of their own: with kept first keys that lie wholly in front of the
    // window's first block, blocks 0 .. kept_span - 1 come first and the window's blocks follow them; a walked index at
    // or beyond kept_span is `gap` keys short of the key it stands for.  Otherwise walked index and key are the same.
    const int keep = (window > 0 && a.shape.keep > 0) ? a.shape.keep : 0;
    int range_begin = lo & ~(kKeysPerBlock - 1);
    int kept_span = 0, gap = 0;
    if (keep > 0) {
        const int kept_blocks = (min(keep, hi) + kKeysPerBlock - 1) & ~(kKeysPerBlock - 1);
        if (kept_blocks < range_begin) {
            kept_span = kept_blocks;
            gap = range_begin - kept_blocks;
        }
        range_begin = 0;
    }
    int range_end = hi - gap;
    const int split = blockIdx.z;
    if (a.n_splits > 1) {
        range_begin += split * a.keys_per_split;
        range_end = min(hi - gap, range_begin + a.keys_per_split);
    }
    const int first_pos = start + q0;            // position of the tile's first token (its window reaches back furthest)
    const int last_lo = first_seen(start + q0 + n_tok - 1, window, chunk);  // the first key the tile's last token sees

    if (a.n_splits > 1 && range_begin >= range_end) {  // a share without keys: its statistics say so, its sums are never read
        float* pml = a.part_ml + ((static_cast<size_t>(tile) * a.kv_heads + kv_head) * a.n_splits + split) * ROWS * 2;
        if (threadIdx.x < ROWS) {
            pml[threadIdx.x * 2] = -INFINITY;
            pml[threadIdx.x * 2 + 1] = 0.f;
        }
        return;
    }

    uint4 qf[RT][NK];
    int row_pos[RT];      // position of the lane's row r of tile rt; -1 for a row that does not exist
    float row_slope[RT];  // its head's slope, in base-2 units
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int row = (rt % RTM) * 16 + r;
        const bool valid = row < n_rows;
        const int tok = valid ? row / group : 0;
        const int head = kv_head * group + (valid ? row - tok * group : 0);
        row_pos[rt] = valid ? start + q0 + tok : -1;
        row_slope[rt] = a.shape.slopes ? a.shape.slopes[head] * kLog2e : 0.f;
        const bf16_t* q_row = a.q + (static_cast<size_t>(first_row_token + tok) * a.q_heads + head) * D + (rt / RTM) * MD +
                              g * (MD / 4);
#pragma unroll
        for (int j = 0; j < NK; ++j)
            qf[rt][j] = valid ? *reinterpret_cast<const uint4*>(q_row + j * 8) : uint4{0, 0, 0, 0};
    }

    float m_run[RT], l_run[RT];
    floatx4 o[RT][ND];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        m_run[rt] = -INFINITY;
        l_run[rt] = 0.f;
#pragma unroll
        for (int dt = 0; dt < ND; ++dt) o[rt][dt] = floatx4{0.f, 0.f, 0.f, 0.f};
    }

    for (int at = range_begin + wave * kKeysPerBlock; at < range_end; at += STEP) {
        const int kb = at < kept_span ? at : at + gap;  // the block's first key
        const int block_end = range_end + (kb - at);    // where this share's keys end, counted in keys of this block's stretch
        // every row sees every key of the block: none lies behind the first token, none before the last one's window
        // (or all are kept first keys)
        const bool inner = kb + kKeysPerBlock - 1 <= first_pos && (kb >= last_lo || kb + kKeysPerBlock <= keep) &&
                           kb + kKeysPerBlock <= block_end;
        floatx4 s[RT][2];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            const int key = min(kb + kt * 16 + r, hi - 1);  // keys past the end are masked below
            const int page = table[key >> a.page_shift];
            const bf16_t* k_row = a.k_pool +
                (((static_cast<size_t>(page) * a.kv_heads + kv_head) << a.page_shift) + (key & page_mask)) * D +
                g * (MD / 4);
            uint4 kf[MAPS * NK];
#pragma unroll
            for (int j = 0; j < MAPS * NK; ++j)
                kf[j] = *reinterpret_cast<const uint4*>(k_row + (j / NK) * MD + (j % NK) * 8);
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) {
                floatx4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int j = 0; j < NK; ++j)
                    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kf[(rt / RTM) * NK + j]),
                                                                  __builtin_bit_cast(bf16x8, qf[rt][j]), acc, 0, 0, 0);
                s[rt][kt] = acc;
            }
        }
        uint2 vf[ND][2];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            const int key = min(kb + kt * 16 + g * 4, (hi - 1) & ~3);
            const int page = table[key >> a.page_shift];
            const bf16_t* v_base = a.v_pool +
                ((static_cast<size_t>(page) * a.kv_heads + kv_head) * DV << a.page_shift) + (key & page_mask);
#pragma unroll
            for (int dt = 0; dt < ND; ++dt)
                vf[dt][kt] = *reinterpret_cast<const uint2*>(v_base + (static_cast<size_t>(dt * 16 + r) << a.page_shift));
        }
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) {
            const int pos = row_pos[rt];
            const int row_lo = first_seen(pos, window, chunk);
            float block_max = -INFINITY;
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int key = kb + kt * 16 + g * 4 + i;
                    const bool seen = inner || (key <= pos && (key >= row_lo || key < keep) && key < block_end);
                    float x = s[rt][kt][i] * scale;
                    if (cap > 0.f) x = cap * fast_tanh(x * inv_cap);
                    x = x * kLog2e - row_slope[rt] * static_cast<float>(pos - key);
                    x = seen ? x : -INFINITY;
                    s[rt][kt][i] = x;
                    block_max = fmaxf(block_max, x);
                }
            }
            block_max = fmaxf(block_max, __shfl_xor(block_max, 16, kWave));
            block_max = fmaxf(block_max, __shfl_xor(block_max, 32, kWave));
            const float m_new = fmaxf(m_run[rt], block_max);
            const float m_safe = (m_new == -INFINITY) ? 0.f : m_new;
            const float alpha = __builtin_amdgcn_exp2f(m_run[rt] - m_safe);  // m_run = -inf: 0, and l, O are 0 anyway
            const bool moved = m_new != m_run[rt];
            m_run[rt] = m_new;
            float p_sum = 0.f;
            uint32_t pw[4];
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
                const float p0 = __builtin_amdgcn_exp2f(s[rt][kt][0] - m_safe);
                const float p1 = __builtin_amdgcn_exp2f(s[rt][kt][1] - m_safe);
                const float p2 = __builtin_amdgcn_exp2f(s[rt][kt][2] - m_safe);
                const float p3 = __builtin_amdgcn_exp2f(s[rt][kt][3] - m_safe);
                p_sum += (p0 + p1) + (p2 + p3);
                pw[kt * 2] = pack_bf16(p0, p1);
                pw[kt * 2 + 1] = pack_bf16(p2, p3);
            }
            l_run[rt] = l_run[rt] * alpha + p_sum;
            if (__any(moved)) {
                // the accumulator's rows are g*4+i, the statistics' row is r: fetch alpha of those rows
                float alpha_o[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) alpha_o[i] = __shfl(alpha, g * 4 + i, kWave);
#pragma unroll
                for (int dt = 0; dt < ND; ++dt)
#pragma unroll
                    for (int i = 0; i < 4; ++i) o[rt][dt][i] *= alpha_o[i];
            }
            const bf16x8 p_frag = __builtin_bit_cast(bf16x8, (uint4{pw[0], pw[1], pw[2], pw[3]}));
#pragma unroll
            for (int dt = 0; dt < ND; ++dt) {
                const uint4 v = uint4{vf[dt][0].x, vf[dt][0].y, vf[dt][1].x, vf[dt][1].y};
                o[rt][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p_frag, __builtin_bit_cast(bf16x8, v), o[rt][dt], 0, 0, 0);
            }
        }
    }

    // ---- the waves' statistics, then the common reference of every row and the whole denominator
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        float l = l_run[rt];
        l += __shfl_xor(l, 16, kWave);
        l += __shfl_xor(l, 32, kWave);
        if (g == 0) {
            m_s[wave][rt * 16 + r] = m_run[rt];
            l_s[wave][rt * 16 + r] = l;
        }
    }
    __syncthreads();
    float own[RT][4];  // this wave's factor for the accumulator rows g*4+i of tile rt
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = rt * 16 + g * 4 + i;
            float m_all = m_s[0][row];
#pragma unroll
            for (int w = 1; w < kScoredWaves; ++w) m_all = fmaxf(m_all, m_s[w][row]);
            if (a.shape.sinks && row < n_rows && a.n_splits == 1)
                m_all = fmaxf(m_all, a.shape.sinks[kv_head * group + row % group] * kLog2e);
            const float mine = m_s[wave][row];
            own[rt][i] = (mine == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(mine - m_all);
        }
    }
    for (int w = 0; w < kScoredWaves; ++w) {
        if (wave == w) {
#pragma unroll
            for (int rt = 0; rt < RT; ++rt)
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int dt = 0; dt < ND; ++dt) {
                        float* cell = &o_s[rt * 16 + g * 4 + i][dt * 16 + r];
                        const float mine = o[rt][dt][i] * own[rt][i];
                        *cell = (w == 0) ? mine : *cell + mine;
                    }
        }
        __syncthreads();
    }
    if (a.n_splits > 1) {
        // this share's (max, sum, accumulator) of every row, for the merge
        const size_t unit = (static_cast<size_t>(tile) * a.kv_heads + kv_head) * a.n_splits + split;
        float* po = a.part_o + unit * ROWS * DV;
        float* pml = a.part_ml + unit * ROWS * 2;
        for (int at = wave; at < n_rows * MAPS; at += kScoredWaves) {
            const int row = MAPS == 1 ? at : at < n_rows ? at : MROWS + at - n_rows;
            float m_all = m_s[0][row];
#pragma unroll
            for (int w = 1; w < kScoredWaves; ++w) m_all = fmaxf(m_all, m_s[w][row]);
            float sum = 0.f;
#pragma unroll
            for (int w = 0; w < kScoredWaves; ++w) {
                const float mine = m_s[w][row];
                sum += (mine == -INFINITY) ? 0.f : l_s[w][row] * __builtin_amdgcn_exp2f(mine - m_all);
            }
            if (lane == 0) {
                pml[row * 2] = m_all;
                pml[row * 2 + 1] = sum;
            }
            for (int d = lane; d < DV; d += kWave) po[static_cast<size_t>(row) * DV + d] = o_s[row][d];
        }
        return;
    }
    for (int row = wave; row < n_rows; row += kScoredWaves) {
        const int tok = row / group;
        const int head = kv_head * group + (row - tok * group);
        float inverse[MAPS];  // 1 / the denominator of each map
#pragma unroll
        for (int map = 0; map < MAPS; ++map) {
            const int at = map * MROWS + row;
            float m_all = m_s[0][at];
#pragma unroll
            for (int w = 1; w < kScoredWaves; ++w) m_all = fmaxf(m_all, m_s[w][at]);
            float den = 0.f;
            if (a.shape.sinks) {
                const float sink = a.shape.sinks[head] * kLog2e;
                m_all = fmaxf(m_all, sink);
                den = __builtin_amdgcn_exp2f(sink - m_all);
            }
#pragma unroll
            for (int w = 0; w < kScoredWaves; ++w) {
                const float mine = m_s[w][at];
                den += (mine == -INFINITY) ? 0.f : l_s[w][at] * __builtin_amdgcn_exp2f(mine - m_all);
            }
            inverse[map] = 1.0f / den;
        }
        float x[(DV + kWave - 1) / kWave];
#pragma unroll
        for (int i = 0; i < (DV + kWave - 1) / kWave; ++i) {
            const int d = lane + i * kWave;
            x[i] = d < DV ? o_s[row][d] * inverse[0] : 0.f;
            if (MAPS == 2 && d < DV) x[i] -= a.shape.lambda * (o_s[MROWS + row][d] * inverse[MAPS - 1]);
        }
        write_head<MAPS, DV>(a, x, static_cast<size_t>(first_row_token + tok), head, lane);
    }
}

// Joins the shares of a tile's keys: one wave per row (four rows a workgroup).  Lane s fetches the statistics of share
// s (and s + 64, ...), so the common reference and every share's factor are known after one round of loads; the shares'
// sums are then fetched without waiting on one another.
constexpr int kMergeShares = 64;  // shares whose factors one pass keeps in a lane each
constexpr int kMergeAhead = 8;    // shares whose sums are on their way at once

template <int DV, int MAPS>
__global__ void __launch_bounds__(256) scored_attention_merge_kernel(ScoredArgs a, int rows_per_tile) {
    constexpr int N = (DV + kWave - 1) / kWave;
    const int lane = threadIdx.x & (kWave - 1);
    const int wave = threadIdx.x / kWave;
    const int tile = blockIdx.x;
    const int kv_head = blockIdx.y;
    const int group = a.q_heads / a.kv_heads;
    const int seq = a.tile_seq ? a.tile_seq[tile] : tile;
    const int q0 = a.tile_seq ? a.tile_q0[tile] : 0;
    const int n_tok = min(a.tokens_per_tile, a.seq_q_len[seq] - q0);
    const int n_rows = n_tok * group;
    const int row = blockIdx.z * 4 + wave;
    if (row >= n_rows) return;
    const int first_row_token = a.q_start_loc[seq] + q0;
    const size_t unit0 = (static_cast<size_t>(tile) * a.kv_heads + kv_head) * a.n_splits;
    const int tok = row / group;
    const int head = kv_head * group + (row - tok * group);
    float x[N];
#pragma unroll
    for (int map = 0; map < MAPS; ++map) {
        const int at = map * (rows_per_tile / MAPS) + row;
        float m_all = -INFINITY;
        for (int sp = lane; sp < a.n_splits; sp += kWave)
            m_all = fmaxf(m_all, a.part_ml[((unit0 + sp) * rows_per_tile + at) * 2]);
        m_all = wave_max(m_all);
        float sink_term = 0.f;  // the sink's share of the denominator, counted once
        if (a.shape.sinks) {
            const float sink = a.shape.sinks[head] * kLog2e;
            m_all = fmaxf(m_all, sink);
            sink_term = __builtin_amdgcn_exp2f(sink - m_all);
        }
        float den = 0.f;        // this lane's shares of it
        float acc[N];
#pragma unroll
        for (int i = 0; i < N; ++i) acc[i] = 0.f;
        for (int base = 0; base < a.n_splits; base += kMergeShares) {
            float mine = 0.f;  // the factor of share base + lane; 0 for a share without keys
            if (base + lane < a.n_splits) {
                const float* ml = a.part_ml + ((unit0 + base + lane) * rows_per_tile + at) * 2;
                mine = (ml[0] == -INFINITY) ? 0.f : __builtin_amdgcn_exp2f(ml[0] - m_all);
                den += ml[1] * mine;
            }
            const int count = min(kMergeShares, a.n_splits - base);
            for (int sp0 = 0; sp0 < count; sp0 += kMergeAhead) {  // (the loads of that many shares travel together)
                float v[kMergeAhead][N];
#pragma unroll
                for (int s = 0; s < kMergeAhead; ++s) {
                    const float* po = a.part_o + ((unit0 + base + min(sp0 + s, count - 1)) * rows_per_tile + at) * DV;
#pragma unroll
                    for (int i = 0; i < N; ++i) v[s][i] = lane + i * kWave < DV ? po[lane + i * kWave] : 0.f;
                }
#pragma unroll
                for (int s = 0; s < kMergeAhead; ++s) {
                    // (0 past the last share, and for a share without keys, whose sums nobody wrote)
                    const float f = sp0 + s < count ? __shfl(mine, sp0 + s, kWave) : 0.f;
#pragma unroll
                    for (int i = 0; i < N; ++i) acc[i] = fmaf(f == 0.f ? 0.f : v[s][i], f, acc[i]);
                }
            }
        }
        const float inverse = 1.0f / (wave_sum(den) + sink_term);
#pragma unroll
        for (int i = 0; i < N; ++i)
            x[i] = map == 0 ? acc[i] * inverse : x[i] - a.shape.lambda * (acc[i] * inverse);
    }
    write_head<MAPS, DV>(a, x, static_cast<size_t>(first_row_token + tok), head, lane);
}

// MOST: the most tiles of 16 rows a workgroup of these sizes takes
template <int D, int DV, int MAPS = 1, int MOST = 4>
int launch_scored(hipStream_t s, const ScoredArgs& a, int row_tiles) {
    dim3 grid(a.n_tiles, a.kv_heads, a.n_splits);
    if (row_tiles > MOST || row_tiles < MAPS) return CIE_BAD_ARGUMENT;
    if constexpr (MAPS == 1) {
        if (row_tiles == 1) scored_attention_mfma_kernel<D, DV, 1, 1><<<grid, 64 * kScoredWaves, 0, s>>>(a);
    }
    if constexpr (MOST >= 2) {
        if (row_tiles == 2) scored_attention_mfma_kernel<D, DV, 2, MAPS><<<grid, 64 * kScoredWaves, 0, s>>>(a);
    }
    if constexpr (MOST >= 4) {
        if (row_tiles == 4) scored_attention_mfma_kernel<D, DV, 4, MAPS><<<grid, 64 * kScoredWaves, 0, s>>>(a);
    }
    if (row_tiles != 1 && row_tiles != 2 && row_tiles != 4) return CIE_BAD_ARGUMENT;
    if (hipGetLastError() != hipSuccess) return CIE_LAUNCH_FAILED;
    if (a.n_splits > 1)
        scored_attention_merge_kernel<DV, MAPS><<<dim3(a.n_tiles, a.kv_heads, 4 * row_tiles / MAPS), 256, 0, s>>>(a, 16 * row_tiles);
    return cie_after_launch();
}

}  // namespace

CIE_API int cie_heads_prepare(void* stream, int dtype, const void* proj, int proj_stride, int q_off, int k_off,
                              int v_off, const float* q_weight, const float* k_weight, int norm_mode, float eps,
                              float temp_coef, int temp_every, const int* positions, const int* seq_of_token,
                              const int* seq_slot, const int* block_table, int table_width, void* q_out,
                              void* k_pool, void* v_pool, int tokens, int q_heads, int kv_heads, int dim, int vdim,
                              int D, int DV, int page_size, int write_kv, const float* cos_table,
                              const float* sin_table, int rot, int neighbours, int maps) {
    if (rot < 0 || rot % 2 || rot > dim || (rot > 0 && (!cos_table || !sin_table))) return CIE_BAD_ARGUMENT;
    if (maps < 1 || maps > 2 || (maps > 1 && norm_mode == 3)) return CIE_BAD_ARGUMENT;
    if (tokens < 0 || q_heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || D < dim || DV < vdim ||
        page_size <= 0 || (page_size & (page_size - 1)) || table_width <= 0 || norm_mode < 0 || norm_mode > 3 ||
        (norm_mode >= 2 && (!q_weight || (write_kv && !k_weight))) || (norm_mode != 0 && !(eps > 0.f)) || temp_every < 0 ||
        q_off < 0 || k_off < 0 || v_off < 0 || proj_stride <= 0)
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    int page_shift = 0;
    while ((1 << page_shift) < page_size) ++page_shift;
    const long units = static_cast<long>(tokens) * (maps * (q_heads + kv_heads) + kv_heads);
    const long blocks = (units + 3) / 4;
    if (blocks > 0x7fffffffL) return CIE_BAD_ARGUMENT;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == CIE_F32)
        heads_prepare_kernel<float><<<static_cast<unsigned>(blocks), 256, 0, s>>>(
            static_cast<const float*>(proj), proj_stride, q_off, k_off, v_off, q_weight, k_weight, norm_mode, eps,
            temp_coef, temp_every, positions, seq_of_token, seq_slot, block_table, table_width,
            static_cast<float*>(q_out), static_cast<float*>(k_pool), static_cast<float*>(v_pool), tokens, q_heads,
            kv_heads, dim, vdim, D, DV, page_shift, write_kv, cos_table, sin_table, rot, neighbours, maps);
    else if (dtype == CIE_BF16)
        heads_prepare_kernel<bf16_t><<<static_cast<unsigned>(blocks), 256, 0, s>>>(
            static_cast<const bf16_t*>(proj), proj_stride, q_off, k_off, v_off, q_weight, k_weight, norm_mode, eps,
            temp_coef, temp_every, positions, seq_of_token, seq_slot, block_table, table_width,
            static_cast<bf16_t*>(q_out), static_cast<bf16_t*>(k_pool), static_cast<bf16_t*>(v_pool), tokens, q_heads,
            kv_heads, dim, vdim, D, DV, page_shift, write_kv, cos_table, sin_table, rot, neighbours, maps);
    else
        return CIE_BAD_ARGUMENT;
    return cie_after_launch();
}

// The preparation behind a convolution (see heads_conv_prepare_kernel).  norm_mode 0, 1 or 2; heads of up to 256 numbers;
// `run` 1, or 8 (2 to 4 taps): tokens that a wave takes.
CIE_API int cie_heads_conv_prepare(void* stream, int dtype, const void* proj, int proj_stride, int q_off, int k_off,
                                   int v_off, const void* taps, int n_taps, float* past, const int* q_start_loc, int single,
                                   void* first_out, const void* first_in, float mix, const float* q_weight,
                                   const float* k_weight, int norm_mode, float eps, float temp_coef, int temp_every,
                                   const int* positions, const int* seq_of_token, const int* seq_slot,
                                   const int* block_table, int table_width, void* q_out, void* k_pool, void* v_pool,
                                   int tokens, int q_heads, int kv_heads, int dim, int vdim, int D, int DV, int page_size,
                                   const float* cos_table, const float* sin_table, int rot, int neighbours, int run) {
    if (rot < 0 || rot % 2 || rot > dim || (rot > 0 && (!cos_table || !sin_table))) return CIE_BAD_ARGUMENT;
    if (tokens < 0 || q_heads <= 0 || kv_heads <= 0 || dim <= 0 || vdim <= 0 || D < dim || DV < vdim || D > 256 || DV > 256 ||
        D % 2 || DV % 2 || page_size <= 0 || (page_size & (page_size - 1)) || table_width <= 0 || norm_mode < 0 ||
        norm_mode > 2 || (norm_mode == 2 && (!q_weight || !k_weight)) || (norm_mode != 0 && !(eps > 0.f)) || temp_every < 0 ||
        q_off < 0 || k_off < 0 || v_off < 0 || proj_stride <= 0 || n_taps < 1 || n_taps > kMaxConvTaps || !q_start_loc ||
        (!taps && n_taps != 1) || (n_taps > 1 && !past))
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    int page_shift = 0;
    while ((1 << page_shift) < page_size) ++page_shift;
    if (single && run != 1) return CIE_BAD_ARGUMENT;
    if (run != 1 && (run != 8 || n_taps < 2 || n_taps > 4)) return CIE_BAD_ARGUMENT;
    const long blocks = (static_cast<long>((tokens + run - 1) / run) * (q_heads + 2 * kv_heads) + 3) / 4;
    if (blocks > 0x7fffffffL) return CIE_BAD_ARGUMENT;
    const int chunks = (D > 128 || DV > 128) ? 2 : 1;
    hipStream_t s = static_cast<hipStream_t>(stream);
#define CIE_CONV_HEADS(T, TAPS, RUN, CHUNKS)                                                                             \
    heads_conv_prepare_kernel<T, TAPS, RUN, CHUNKS><<<static_cast<unsigned>(blocks), 256, 0, s>>>(                       \
        static_cast<const T*>(proj), proj_stride, q_off, k_off, v_off,                                                   \
        ConvHeads<T>{static_cast<const T*>(taps), n_taps, past, q_start_loc, single, static_cast<T*>(first_out),         \
                     static_cast<const T*>(first_in), mix},                                                              \
        q_weight, k_weight, norm_mode, eps, temp_coef, temp_every, positions, seq_of_token, seq_slot, block_table,       \
        table_width, static_cast<T*>(q_out), static_cast<T*>(k_pool), static_cast<T*>(v_pool), tokens, q_heads, kv_heads, \
        dim, vdim, D, DV, page_shift, cos_table, sin_table, rot, neighbours)
#define CIE_CONV_HEADS_CHUNKS(T, TAPS, RUN)                \
    do {                                                   \
        if (chunks == 1) CIE_CONV_HEADS(T, TAPS, RUN, 1);  \
        else CIE_CONV_HEADS(T, TAPS, RUN, 2);              \
    } while (0)
#define CIE_CONV_HEADS_TYPE(T)                                     \
    do {                                                           \
        if (n_taps == 2 && run == 1) CIE_CONV_HEADS_CHUNKS(T, 2, 1);      \
        else if (n_taps == 3 && run == 1) CIE_CONV_HEADS_CHUNKS(T, 3, 1); \
        else if (n_taps == 4 && run == 1) CIE_CONV_HEADS_CHUNKS(T, 4, 1); \
        else if (n_taps == 2 && run == 8) CIE_CONV_HEADS_CHUNKS(T, 2, 8); \
        else if (n_taps == 3 && run == 8) CIE_CONV_HEADS_CHUNKS(T, 3, 8); \
        else if (n_taps == 4 && run == 8) CIE_CONV_HEADS_CHUNKS(T, 4, 8); \
        else CIE_CONV_HEADS_CHUNKS(T, 0, 1);                              \
    } while (0)
    if (dtype == CIE_F32) CIE_CONV_HEADS_TYPE(float);
    else if (dtype == CIE_BF16) CIE_CONV_HEADS_TYPE(bf16_t);
    else return CIE_BAD_ARGUMENT;
#undef CIE_CONV_HEADS_CHUNKS
#undef CIE_CONV_HEADS_TYPE
#undef CIE_CONV_HEADS
    return cie_after_launch();
}

CIE_API int cie_scored_attention_generic(void* stream, int dtype, const void* q, const void* k_pool,
                                         const void* v_pool, const int* block_table, int table_width,
                                         const int* positions, const int* seq_of_token, const int* seq_slot,
                                         const void* gate, int gate_stride, void* out, int tokens, int q_heads,
                                         int kv_heads, int D, int DV, int page_size, int window, float scale,
                                         float softcap, const float* slopes, const float* sinks, int chunk,
                                         int keep, int gate_wide, int real_vdim, int maps, float lambda, float factor,
                                         float eps, long out_stride) {
    if (tokens < 0 || q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads || D <= 0 || D % 8 || DV <= 0 || DV % 8 ||
        DV > kWave * kMaxWideSlices || page_size <= 0 || table_width <= 0 || q_heads > 65535 || real_vdim <= 0 ||
        real_vdim > DV || maps < 1 || maps > 2 || (maps == 2 && !(eps > 0.f)) || out_stride < static_cast<long>(q_heads) * DV ||
        (gate && gate_stride < (gate_wide ? q_heads * real_vdim : q_heads)))
        return CIE_BAD_ARGUMENT;
    if (tokens == 0) return CIE_OK;
    hipStream_t s = static_cast<hipStream_t>(stream);
    dim3 grid(tokens, q_heads);
    const size_t lds = (static_cast<size_t>(D) + (4 + maps) * DV) * sizeof(float);
    if (lds > 60 * 1024) return CIE_BAD_ARGUMENT;
    if (chunk < 0 || (chunk > 0 && window > 0) || keep < 0 || (keep > 0 && window <= 0)) return CIE_BAD_ARGUMENT;
    const ScoreShape shape{scale, softcap, slopes, sinks, window, chunk, keep, gate_wide, real_vdim, lambda, factor, eps};
#define CIE_GENERIC(T, SLICES)                                                                                          \
    scored_attention_generic_kernel<T, SLICES><<<grid, 256, lds, s>>>(                                                  \
        static_cast<const T*>(q), static_cast<const T*>(k_pool), static_cast<const T*>(v_pool), block_table, table_width, \
        positions, seq_of_token, seq_slot, static_cast<const T*>(gate), gate_stride, static_cast<T*>(out), out_stride, q_heads, kv_heads, \
        D, DV, page_size, maps, shape)
    const bool wide = DV > kWave * kMaxSlices;
    if (dtype == CIE_F32 && !wide) CIE_GENERIC(float, kMaxSlices);
    else if (dtype == CIE_F32) CIE_GENERIC(float, kMaxWideSlices);
    else if (dtype == CIE_BF16 && !wide) CIE_GENERIC(bf16_t, kMaxSlices);
    else if (dtype == CIE_BF16) CIE_GENERIC(bf16_t, kMaxWideSlices);
    else return CIE_BAD_ARGUMENT;
#undef CIE_GENERIC
    return cie_after_launch();
}

// bfloat16 on the matrix cores: (D, DV) as the last lines list them; pages of at least 4 keys; a token's heads of one key
// head fill at most `row_tiles` tiles of 16 rows (of each of the `maps`).
CIE_API int cie_scored_attention_mfma(void* stream, const void* q, const void* k_pool, const void* v_pool,
                                      const int* block_table, int table_width, const int* tile_seq,
                                      const int* tile_q0, int n_tiles, const int* seq_slot, const int* seq_start,
                                      const int* seq_q_len, const int* q_start_loc, const void* gate,
                                      int gate_stride, void* out, int q_heads, int kv_heads, int D, int DV,
                                      int page_size, int tokens_per_tile, int row_tiles, int window, float scale,
                                      float softcap, const float* slopes, const float* sinks, int n_splits,
                                      int keys_per_split, float* part_o, float* part_ml, int chunk, int keep,
                                      int gate_wide, int real_vdim, int maps, float lambda, float factor, float eps,
                                      long out_stride) {
    if (chunk < 0 || (chunk > 0 && window > 0) || keep < 0 || (keep > 0 && window <= 0)) return CIE_BAD_ARGUMENT;
    if (n_tiles < 0 || q_heads <= 0 || kv_heads <= 0 || q_heads % kv_heads || page_size < 4 ||
        (page_size & (page_size - 1)) || table_width <= 0 || tokens_per_tile < 1 || kv_heads > 65535 ||
        (tile_seq == nullptr) != (tile_q0 == nullptr) || maps < 1 || maps > 2 || (maps == 2 && (!(eps > 0.f) || sinks)) ||
        real_vdim <= 0 || real_vdim > DV || (gate && gate_stride < (gate_wide ? q_heads * real_vdim : q_heads)))
        return CIE_BAD_ARGUMENT;
    if (tokens_per_tile * (q_heads / kv_heads) * maps > 16 * row_tiles || out_stride < static_cast<long>(q_heads) * DV) return CIE_BAD_ARGUMENT;
    if (n_splits < 1 || n_splits > 65535 ||
        (n_splits > 1 && (keys_per_split < 128 || keys_per_split % 128 || !part_o || !part_ml)))
        return CIE_BAD_ARGUMENT;
    if (n_tiles == 0) return CIE_OK;
    ScoredArgs a;
    a.n_splits = n_splits;
    a.keys_per_split = keys_per_split;
    a.part_o = part_o;
    a.part_ml = part_ml;
    a.q = static_cast<const bf16_t*>(q);
    a.k_pool = static_cast<const bf16_t*>(k_pool);
    a.v_pool = static_cast<const bf16_t*>(v_pool);
    a.block_table = block_table;
    a.table_width = table_width;
    a.tile_seq = tile_seq;
    a.tile_q0 = tile_q0;
    a.seq_slot = seq_slot;
    a.seq_start = seq_start;
    a.seq_q_len = seq_q_len;
    a.q_start_loc = q_start_loc;
    a.gate = static_cast<const bf16_t*>(gate);
    a.gate_stride = gate_stride;
    a.out = static_cast<bf16_t*>(out);
    a.out_stride = out_stride;
    a.q_heads = q_heads;
    a.kv_heads = kv_heads;
    a.page_shift = 0;
    while ((1 << a.page_shift) < page_size) ++a.page_shift;
    a.tokens_per_tile = tokens_per_tile;
    a.n_tiles = n_tiles;
    a.shape = ScoreShape{scale, softcap, slopes, sinks, window, chunk, keep, gate_wide, real_vdim, lambda, factor, eps};
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (maps == 2) {
        if (D == 64 && DV == 64) return launch_scored<64, 64, 2>(s, a, row_tiles);
        if (D == 64 && DV == 128) return launch_scored<64, 128, 2>(s, a, row_tiles);
        if (D == 128 && DV == 64) return launch_scored<128, 64, 2>(s, a, row_tiles);
        if (D == 128 && DV == 128) return launch_scored<128, 128, 2>(s, a, row_tiles);
        if (D == 128 && DV == 256) return launch_scored<128, 256, 2, 2>(s, a, row_tiles);
        if (D == 256 && DV == 128) return launch_scored<256, 128, 2, 2>(s, a, row_tiles);
        if (D == 256 && DV == 256) return launch_scored<256, 256, 2, 2>(s, a, row_tiles);
        return CIE_BAD_ARGUMENT;
    }
    if (D == 64 && DV == 64) return launch_scored<64, 64>(s, a, row_tiles);
    if (D == 128 && DV == 128) return launch_scored<128, 128>(s, a, row_tiles);
    if (D == 64 && DV == 128) return launch_scored<64, 128>(s, a, row_tiles);
    if (D == 128 && DV == 64) return launch_scored<128, 64>(s, a, row_tiles);
    if (D == 96 && DV == 64) return launch_scored<96, 64>(s, a, row_tiles);
    if (D == 128 && DV == 96) return launch_scored<128, 96>(s, a, row_tiles);
    if (D == 160 && DV == 128) return launch_scored<160, 128, 1, 2>(s, a, row_tiles);
    if (D == 192 && DV == 160) return launch_scored<192, 160, 1, 2>(s, a, row_tiles);
    if (D == 256 && DV == 192) return launch_scored<256, 192, 1, 2>(s, a, row_tiles);
    if (D == 320 && DV == 256) return launch_scored<320, 256, 1, 2>(s, a, row_tiles);
    return CIE_BAD_ARGUMENT;
}
