// Causal attention whose scores carry a bias by distance and whose softmax may have a sink, over keys and values
// of different widths in plain pages.
//
// Pages: keys [page, position, kv_head, key_dim], values [page, position, kv_head, value_dim]. A score is
// (q . k_j) * scale + bias[min(p - j, longest), head]; the bias table has one row per distance up to `longest`,
// which stands for every longer one. A sink is one more term exp(sink[head]) in the softmax's denominator, with
// no key and no value: the running maximum starts at the sink and the running sum at 1.
//
// One wave takes a (token, head). Keys are walked in tiles of 64 at absolute positions: each lane forms the score
// of one key, the tile's maximum and weights follow, and then the lanes turn to the value's channels and add the
// 64 weighted values in key order. The order of every sum depends on the query's position alone, so a row does
// not change with the step's cut, the batch or the pages. Scores, weights and sums are float32.
#include "cache_layout.h"
#include "common.h"
#include "microllm_hip.h"

namespace mll {

constexpr int kBiasKeyTile = 64;
constexpr int kMaxValueChannelsALane = 4;     // value_dim up to 256

template <typename T> __device__ inline float dot_row(const T* key, const float* q, int dim);

template <> __device__ inline float dot_row<float>(const float* key, const float* q, int dim) {
    float sum = 0.0f;
    int c = 0;
    if ((dim & 3) == 0 && (reinterpret_cast<uintptr_t>(key) & 15) == 0) {
        for (; c < dim; c += 4) {
            const float4 k = *reinterpret_cast<const float4*>(key + c);
            sum = fmaf(k.x, q[c], sum);
            sum = fmaf(k.y, q[c + 1], sum);
            sum = fmaf(k.z, q[c + 2], sum);
            sum = fmaf(k.w, q[c + 3], sum);
        }
        return sum;
    }
    for (; c < dim; ++c) sum = fmaf(key[c], q[c], sum);
    return sum;
}

template <> __device__ inline float dot_row<bf16>(const bf16* key, const float* q, int dim) {
    float sum = 0.0f;
    int c = 0;
    if ((dim & 7) == 0 && (reinterpret_cast<uintptr_t>(key) & 15) == 0) {
        for (; c < dim; c += 8) {
            const uint4 raw = *reinterpret_cast<const uint4*>(key + c);
            const uint32_t words[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
            for (int w = 0; w < 4; ++w) {
                const float low = __builtin_bit_cast(float, words[w] << 16);
                const float high = __builtin_bit_cast(float, words[w] & 0xffff0000u);
                sum = fmaf(low, q[c + 2 * w], sum);
                sum = fmaf(high, q[c + 2 * w + 1], sum);
            }
        }
        return sum;
    }
    for (; c < dim; ++c) sum = fmaf(to_float(key[c]), q[c], sum);
    return sum;
}

template <typename T, typename O>
__global__ void __launch_bounds__(kWave)
bias_attention_kernel(const T* __restrict__ q, const T* __restrict__ k_pages, const T* __restrict__ v_pages,
                      const int32_t* __restrict__ block_table, int table_width, const int32_t* __restrict__ seq_of_token,
                      const int32_t* __restrict__ positions, const float* __restrict__ bias, int longest,
                      const float* __restrict__ sink, O* __restrict__ out, int64_t out_stride, int heads, int kv_heads,
                      int key_dim, int value_dim, int page_size, float scale, float out_scale,
                      const float* __restrict__ slopes, int window, int chunk, const float* __restrict__ gate,
                      int64_t gate_stride, float softcap, int gate_channels) {
    extern __shared__ float q_row[];
    const int token = blockIdx.x / heads;
    const int head = blockIdx.x % heads;
    const int seq = seq_of_token[token];
    if (seq < 0) return;       // a row that pads the step
    const int lane = threadIdx.x;
    const int position = positions[token];
    const int kv_head = head / (heads / kv_heads);
    const T* query = q + (static_cast<int64_t>(token) * heads + head) * key_dim;
    for (int c = lane; c < key_dim; c += kWave) q_row[c] = to_float(query[c]);
    __syncthreads();
    const int32_t* table = block_table + static_cast<int64_t>(seq) * table_width;
    float running_max = sink ? sink[head] : -INFINITY;
    float running_sum = sink ? 1.0f : 0.0f;
    float acc[kMaxValueChannelsALane] = {0.0f, 0.0f, 0.0f, 0.0f};
    const int64_t key_row = static_cast<int64_t>(kv_heads) * key_dim;
    const int64_t value_row = static_cast<int64_t>(kv_heads) * value_dim;
    const float slope = slopes ? slopes[head] : 0.0f;
    // the oldest key seen: the first of the query's chunk of positions, or what the window reaches back to
    const int low = chunk > 0 ? position / chunk * chunk : (window > 0 ? max(0, position - window + 1) : 0);
    for (int first = low / kBiasKeyTile * kBiasKeyTile; first <= position; first += kBiasKeyTile) {
        const int j = first + lane;
        float score = -INFINITY;
        int64_t place = 0;
        const bool seen = j >= low && j <= position;
        if (seen) {
            place = static_cast<int64_t>(table[j / page_size]) * page_size + j % page_size;
            const T* key = k_pages + place * key_row + static_cast<int64_t>(kv_head) * key_dim;
            score = dot_row<T>(key, q_row, key_dim) * scale;
            if (softcap > 0.0f) score = softcap * tanhf(score / softcap);
            if (bias) score += bias[static_cast<int64_t>(min(position - j, longest)) * heads + head];
            if (slopes) score -= slope * static_cast<float>(position - j);
        }
        const float tile_max = wave_max(score);
        const float new_max = fmaxf(running_max, tile_max);
        const float keep = running_max == -INFINITY ? 0.0f : expf(running_max - new_max);
        const float weight = seen ? expf(score - new_max) : 0.0f;
        running_sum = running_sum * keep + wave_sum(weight);
        running_max = new_max;
#pragma unroll
        for (int m = 0; m < kMaxValueChannelsALane; ++m) acc[m] *= keep;
        const int in_tile = min(kBiasKeyTile, position - first + 1);
        for (int n = max(0, low - first); n < in_tile; ++n) {
            const float w = __shfl(weight, n, kWave);
            const int64_t at = __shfl(place, n, kWave);
            const T* value = v_pages + at * value_row + static_cast<int64_t>(kv_head) * value_dim;
#pragma unroll
            for (int m = 0; m < kMaxValueChannelsALane; ++m) {
                const int c = lane + m * kWave;
                if (c < value_dim) acc[m] = fmaf(w, to_float(value[c]), acc[m]);
            }
        }
    }
    float factor = out_scale / running_sum;
    const float* gate_row = gate ? gate + static_cast<int64_t>(token) * gate_stride + (gate_channels ? head * value_dim : head) : nullptr;
    if (gate_row && !gate_channels) factor *= 1.0f / (1.0f + expf(-gate_row[0]));
    O* to = out + static_cast<int64_t>(token) * out_stride + static_cast<int64_t>(head) * value_dim;
#pragma unroll
    for (int m = 0; m < kMaxValueChannelsALane; ++m) {
        const int c = lane + m * kWave;
        if (c < value_dim) to[c] = from_float<O>(gate_row && gate_channels ? acc[m] * factor / (1.0f + expf(-gate_row[c])) : acc[m] * factor);
    }
}

constexpr int kNormStoreWaves = 4;

// One wave a (token, head of q, k or v), four to a workgroup: the norm of queries and keys over their head, the queries' factor by
// position, and the write of keys and values into their pages. MORE: with what MllStoreExtras says (a convolution over time
// before everything else, the norm after the turn, heads stored wider than they are, several keys a key head).
template <typename T, bool MORE>
__global__ void __launch_bounds__(kNormStoreWaves * kWave)
qk_norm_store_kernel(const float* __restrict__ qkv, int n_parts, int64_t part_stride, const float* __restrict__ q_weight,
                     const float* __restrict__ k_weight, float eps, const int32_t* __restrict__ positions,
                     const int32_t* __restrict__ slot_mapping, float temp_coef, int temp_every, T* __restrict__ q_out,
                     T* __restrict__ k_pages, T* __restrict__ v_pages, int heads, int kv_heads, int key_dim, int value_dim,
                     int tiled_page_size, const float* __restrict__ bias, int normed, int queries_only, int64_t row_stride,
                     const float* __restrict__ cos_sin, int rot_dims, int values_normed, int total, MllStoreExtras more) {
    extern __shared__ float kept_sums[];        // a wave's vector, as it is before norm and turn: read from memory once
    const int vectors = queries_only ? heads : heads + 2 * kv_heads;
    const int vector = blockIdx.x * kNormStoreWaves + threadIdx.x / kWave;
    float* own = kept_sums + threadIdx.x / kWave * max(key_dim, value_dim);
    if (vector >= total) return;
    const int token = vector / vectors;
    const int which = vector % vectors;
    const int lane = threadIdx.x % kWave;
    const float* row = qkv + static_cast<int64_t>(token) * row_stride;
    const bool is_q = which < heads, is_k = !is_q && which < heads + kv_heads;
    const int head = is_q ? which : (is_k ? which - heads : which - heads - kv_heads);
    const int query_dim = MORE && more.maps > 1 ? key_dim / more.maps : key_dim;
    const int dim = is_q ? query_dim : (is_k ? key_dim : value_dim);
    const int offset = is_q ? head * query_dim
                            : (is_k ? heads * query_dim + head * key_dim : heads * query_dim + kv_heads * key_dim + head * value_dim);
    const int slot = is_q ? 0 : slot_mapping[token];
    if (!is_q && slot < 0) return;
    int tokens_before = 0;              // of the same request in this step
    const float* tail = nullptr;        // the inputs before the step
    if (MORE && more.taps != nullptr) {
        const int seq = more.seq_of_token[token];
        if (seq < 0) return;            // a row that pads the step
        tokens_before = token - more.cu_tokens[seq];
        tail = more.kept + static_cast<int64_t>(more.slots[seq]) * (more.n_taps - 1) * (heads * query_dim + kv_heads * (key_dim + value_dim));
    }
    // what the vector holds at channel c before it is normed or turned: the sums (or their convolution over time), the bias
    auto raw = [&](int c) {
        float value;
        if (MORE && more.taps != nullptr) {
            const int columns = heads * query_dim + kv_heads * (key_dim + value_dim);
            const float* tap = more.taps + static_cast<int64_t>(offset + c) * more.n_taps;
            value = 0.0f;
            for (int j = 0; j < more.n_taps; ++j) {
                const int back = more.n_taps - 1 - j;       // how many tokens before this one
                const float input = back <= tokens_before
                                        ? row[offset + c - static_cast<int64_t>(back) * row_stride]
                                        : tail[static_cast<int64_t>(more.n_taps - 1 - (back - tokens_before)) * columns + offset + c];
                value = fmaf(tap[j], input, value);
            }
        } else {
            value = row[offset + c];
            for (int part = 1; part < n_parts; ++part) value += row[part * part_stride + offset + c];
        }
        if (bias) value += bias[offset + c];
        return value;
    };
    // queries and keys turn by the token's position in their first rot_dims channels, channel i with i + rot_dims / 2
    const bool turns = cos_sin != nullptr && (is_q || is_k);
    const int half = rot_dims / 2;
    const float* angles = cos_sin + static_cast<int64_t>(token) * rot_dims;     // [rot_dims / 2][cos, sin]
    const bool norm_turned = MORE && more.norm_turned && turns;
    float squares = 0.0f;
    for (int c = lane; c < dim; c += kWave) {
        const float value = raw(c);
        own[c] = value;
        float length = 1.0f;
        if (norm_turned && c < rot_dims) {      // a turned pair is as long as before, but for the factor within cos and sin
            const int pair = c < half ? c : c - half;
            length = angles[2 * pair] * angles[2 * pair] + angles[2 * pair + 1] * angles[2 * pair + 1];
        }
        squares += value * value * length;
    }
    const float* weight = is_q ? q_weight : (is_k ? k_weight : nullptr);
    const bool norm = (is_q || is_k) ? normed : values_normed;
    float factor = 1.0f;
    if (norm) factor = 1.0f / sqrtf(wave_sum(squares) / static_cast<float>(dim) + eps);
    if (is_q && temp_coef != 0.0f) {
        const int steps = (positions[token] + 1) / temp_every;
        factor *= 1.0f + temp_coef * static_cast<float>(log(static_cast<double>(steps) + 1.0));
    }
    // how wide the vectors are kept, and where among a key head's keys this query's lies
    const int key_width = MORE && more.stored_dim > 0 ? more.stored_dim : key_dim;
    const int value_width = MORE && more.stored_dim > 0 ? more.stored_dim : value_dim;
    const int place = MORE && is_q && more.maps > 1 ? (head % more.maps) * query_dim : 0;
    T* to = is_q ? q_out + (static_cast<int64_t>(token) * heads + head) * key_width
                 : (is_k ? k_pages + (static_cast<int64_t>(slot) * kv_heads + head) * key_width
                         : v_pages + (static_cast<int64_t>(slot) * kv_heads + head) * value_width);
    // tiled_page_size > 0: the pages are in the order the MFMA kernels read them (cache_layout.h; both widths equal)
    const bool tiled = tiled_page_size > 0 && !is_q;
    const CacheLayout layout(kv_heads, tiled ? tiled_page_size : 16, key_width);
    const int64_t page = tiled ? slot / tiled_page_size : 0;
    const int in_page = tiled ? slot % tiled_page_size : 0;
    auto normed_value = [&](float value, int c) { return norm ? (weight ? value * factor * weight[c] : value * factor) : value; };
    auto prepared = [&](int c) { return norm_turned ? own[c] : normed_value(own[c], c); };      // what is turned
    // the wave's lanes read what its other lanes wrote
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    const int kept_width = MORE ? (is_q || is_k ? key_width : value_width) : dim;
    for (int at = lane; at < kept_width; at += kWave) {
        const int c = at - place;
        float value = 0.0f;
        if (!MORE || (c >= 0 && c < dim)) {
            value = prepared(c);
            if (turns && c < rot_dims) {
                const int pair = c < half ? c : c - half;
                const float other = prepared(c < half ? c + half : c - half);
                const float cosine = angles[2 * pair], sine = angles[2 * pair + 1];
                value = c < half ? value * cosine - other * sine : value * cosine + other * sine;
            }
            if (norm_turned) value = normed_value(value, c);
        }
        const T rounded = from_float<T>(value);
        if (tiled) {
            if (is_k) k_pages[layout.k_at(page, head, in_page, at)] = rounded;
            else v_pages[layout.v_at(page, head, in_page, at)] = rounded;
        } else {
            to[at] = rounded;
        }
    }
}

}  // namespace mll

using namespace mll;

extern "C" {

int mll_qk_norm_store(const float* qkv, int n_parts, int64_t part_stride, const float* q_weight, const float* k_weight,
                      float eps, const int32_t* positions, const int32_t* slot_mapping, float temp_coef, int temp_every,
                      void* q_out, void* k_pages, void* v_pages, int dtype, int n_tokens, int heads, int kv_heads, int key_dim,
                      int value_dim, int tiled_page_size, const float* bias, int normed, int queries_only, int64_t row_stride,
                      const float* cos_sin, int rot_dims, int values_normed, const MllStoreExtras* more, hipStream_t stream) {
    const MllStoreExtras given = more ? *more : MllStoreExtras{};
    const int maps = given.maps > 1 ? given.maps : 1;
    MLL_REQUIRE(tiled_page_size == 0 || (tiled_page_size > 0 && tiled_page_size % 16 == 0 && (key_dim == value_dim || given.stored_dim > 0)),
                "qk_norm_store: tiled pages hold a multiple of 16 positions and keys and values of one width");
    MLL_REQUIRE(n_tokens >= 0 && heads > 0 && kv_heads > 0 && key_dim > 0 && value_dim > 0, "qk_norm_store: sizes must be positive");
    MLL_REQUIRE(n_parts >= 1, "qk_norm_store: at least one part");
    MLL_REQUIRE(key_dim % maps == 0 && heads % maps == 0, "qk_norm_store: a key head holds equal keys, and every map has as many query heads");
    MLL_REQUIRE(row_stride >= (queries_only ? heads * (key_dim / maps) : heads * (key_dim / maps) + kv_heads * (key_dim + value_dim)),
                "qk_norm_store: the rows are narrower than their queries, keys and values");
    MLL_REQUIRE(maps == 1 || (!normed && cos_sin == nullptr), "qk_norm_store: several keys a key head are neither normed nor turned");
    MLL_REQUIRE(given.stored_dim == 0 || (given.stored_dim >= key_dim && given.stored_dim >= value_dim), "qk_norm_store: heads are stored at least as wide as they are");
    MLL_REQUIRE(given.taps == nullptr || (n_parts == 1 && !queries_only && given.n_taps >= 1 && (given.n_taps == 1 || given.kept != nullptr) &&
                                          given.seq_of_token && given.cu_tokens && given.slots),
                "qk_norm_store: a convolution reads whole rows of q, k and v, the request of every token and what requests kept");
    MLL_REQUIRE(!given.norm_turned || (normed && cos_sin != nullptr), "qk_norm_store: a norm of turned vectors needs both");
    MLL_REQUIRE(cos_sin == nullptr || (rot_dims > 0 && rot_dims % 2 == 0 && rot_dims <= key_dim),
                "qk_norm_store: an even number of turned channels, at most the head's");
    MLL_REQUIRE((q_weight == nullptr) == (k_weight == nullptr), "qk_norm_store: norm weights for queries and keys, or for neither");
    MLL_REQUIRE(!(normed || values_normed) || eps > 0.0f, "qk_norm_store: eps must be positive");
    MLL_REQUIRE(normed || q_weight == nullptr, "qk_norm_store: norm weights without a norm");
    MLL_REQUIRE(queries_only || (slot_mapping != nullptr && k_pages != nullptr && v_pages != nullptr), "qk_norm_store: keys and values need pages and slots");
    MLL_REQUIRE(temp_coef == 0.0f || temp_every > 0, "qk_norm_store: the factor by position needs a positive step");
    if (n_tokens == 0) return 0;
    const int64_t total = static_cast<int64_t>(n_tokens) * (queries_only ? heads : heads + 2 * kv_heads);
    MLL_REQUIRE(total < (1ll << 31) - kNormStoreWaves, "qk_norm_store: too many rows for one launch");
    const int64_t blocks = (total + kNormStoreWaves - 1) / kNormStoreWaves;
    const size_t lds = static_cast<size_t>(key_dim > value_dim ? key_dim : value_dim) * kNormStoreWaves * sizeof(float);
    MLL_REQUIRE(lds <= 64 * 1024, "qk_norm_store: heads wider than 4096 are not supported");
#define MLL_NORM_STORE(T, MORE)                                                                                               \
    qk_norm_store_kernel<T, MORE><<<static_cast<unsigned>(blocks), kNormStoreWaves * kWave, lds, stream>>>(                       \
        qkv, n_parts, part_stride, q_weight, k_weight, eps, positions, slot_mapping, temp_coef, temp_every, static_cast<T*>(q_out), \
        static_cast<T*>(k_pages), static_cast<T*>(v_pages), heads, kv_heads, key_dim, value_dim, tiled_page_size, bias, normed,     \
        queries_only, row_stride, cos_sin, rot_dims, values_normed, static_cast<int>(total), given)
    if (dtype == kF32) {
        if (more) MLL_NORM_STORE(float, true); else MLL_NORM_STORE(float, false);
    } else if (dtype == kBF16) {
        if (more) MLL_NORM_STORE(bf16, true); else MLL_NORM_STORE(bf16, false);
    } else {
        return fail("qk_norm_store: unknown dtype");
    }
#undef MLL_NORM_STORE
    return check_launch("qk_norm_store");
}

int mll_bias_attention(const void* q, const void* k_pages, const void* v_pages, const int32_t* block_table, int table_width,
                       const int32_t* seq_of_token, const int32_t* positions, const float* bias, int longest,
                       const float* sink, void* out, int64_t out_stride, int dtype, int n_tokens, int heads, int kv_heads,
                       int key_dim, int value_dim, int page_size, float scale, float out_scale, const float* slopes, int window,
                       int chunk, const float* gate, int64_t gate_stride, float softcap, int gate_channels, int out_f32,
                       hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && heads > 0 && kv_heads > 0 && key_dim > 0 && value_dim > 0 && page_size > 0 && table_width > 0,
                "bias_attention: sizes must be positive");
    MLL_REQUIRE(heads % kv_heads == 0, "bias_attention: heads must divide into kv heads");
    MLL_REQUIRE(value_dim <= kMaxValueChannelsALane * kWave, "bias_attention: value heads wider than 256 are not supported");
    MLL_REQUIRE(bias == nullptr || longest >= 0, "bias_attention: the bias table needs at least one row");
    MLL_REQUIRE(out_stride >= static_cast<int64_t>(heads) * value_dim, "bias_attention: the output rows overlap");
    MLL_REQUIRE(window >= 0 && chunk >= 0 && !(window > 0 && chunk > 0), "bias_attention: a window or chunks of positions, not both");
    MLL_REQUIRE(gate == nullptr || gate_stride >= (gate_channels ? heads * value_dim : heads), "bias_attention: one gate a head, or a channel, in every row");
    MLL_REQUIRE(softcap >= 0.0f, "bias_attention: the cap on the scores is positive, or 0 for none");
    if (n_tokens == 0) return 0;
    const int64_t blocks = static_cast<int64_t>(n_tokens) * heads;
    MLL_REQUIRE(blocks < (1ll << 31), "bias_attention: too many rows for one launch");
    const size_t lds = static_cast<size_t>(key_dim) * sizeof(float);
    MLL_REQUIRE(lds <= 64 * 1024, "bias_attention: key heads wider than 16384 are not supported");
#define MLL_BIAS_ATTENTION(T, O)                                                                                              \
    bias_attention_kernel<T, O><<<static_cast<unsigned>(blocks), kWave, lds, stream>>>(                                           \
        static_cast<const T*>(q), static_cast<const T*>(k_pages), static_cast<const T*>(v_pages), block_table, table_width,         \
        seq_of_token, positions, bias, longest, sink, static_cast<O*>(out), out_stride, heads, kv_heads, key_dim, value_dim,        \
        page_size, scale, out_scale, slopes, window, chunk, gate, gate_stride, softcap, gate_channels)
    if (dtype == kF32) {
        MLL_BIAS_ATTENTION(float, float);
    } else if (dtype == kBF16) {
        if (out_f32) MLL_BIAS_ATTENTION(bf16, float); else MLL_BIAS_ATTENTION(bf16, bf16);
    } else {
        return fail("bias_attention: unknown dtype");
    }
#undef MLL_BIAS_ATTENTION
    return check_launch("bias_attention");
}

}  // extern "C"
