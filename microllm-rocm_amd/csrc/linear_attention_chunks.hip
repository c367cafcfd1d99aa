// Linear attention with one fixed decay a head for long portions, in chunks of 64 tokens:
//
//   S_t = a S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t
//
// Within a chunk that begins with the state S (token t of the chunk, from 0)
//
//   o_t = a^(t+1) S^T q_t + sum_{j <= t} a^(t-j) (q_t . k_j) v_j,
//
// and a chunk of n tokens leaves a^n S + sum_j a^(n-1-j) k_j v_j^T. Three kernels: what every chunk adds to the state
// (all chunks at once), the states at the chunks' starts (a walk over a request's chunks, every element of the state on
// its own), and the results (all chunks at once). All products are float32 on the matrix units
// (v_mfma_f32_16x16x4_f32); state, powers of the decay and sums are float32. A chunk begins at every 64th token of a
// request's portion, so where a portion was cut changes a result by rounding alone.
#include "common.h"
#include "microllm_hip.h"

namespace mll {

typedef float floatx4 __attribute__((ext_vector_type(4)));

constexpr int kScanChunk = 64;          // tokens
constexpr int kScanThreads = 256;       // four waves: 16 rows (or 16 value channels) each
constexpr int kScanValues = 64;         // value channels a workgroup holds in LDS at a time

// Chunks are numbered so that every request's are consecutive and none are shared: request i's begin at
// cu[i] / 64 + i. Returns false for a number that no request uses.
__device__ inline bool find_chunk(const int32_t* cu_tokens, int n_seqs, int number, int* seq, int* first, int* count) {
    for (int i = 0; i < n_seqs; ++i) {
        const int begin = cu_tokens[i], end = cu_tokens[i + 1];
        const int base = begin / kScanChunk + i;
        const int chunks = (end - begin + kScanChunk - 1) / kScanChunk;
        if (number >= base && number < base + chunks) {
            *seq = i;
            *first = begin + (number - base) * kScanChunk;
            *count = min(kScanChunk, end - *first);
            return true;
        }
    }
    return false;
}

template <bool SILU>
__device__ inline float scan_input(float value) { return SILU ? activate(value, kActSilu) : value; }

// store(t, c, source[t][c]) for t < ROWS, c < COLUMNS; 0 beyond the first `count` rows and `channels` columns. Eight loads a
// thread are asked for before the first is used.
template <int ROWS, int COLUMNS, typename Store>
__device__ inline void load_tile(const float* source, int64_t row_stride, int count, int channels, Store store) {
    constexpr int kAtATime = 8;
    static_assert(ROWS * COLUMNS % (kScanThreads * kAtATime) == 0, "whole rounds of loads");
    for (int base = threadIdx.x; base < ROWS * COLUMNS; base += kScanThreads * kAtATime) {
        float value[kAtATime];
#pragma unroll
        for (int j = 0; j < kAtATime; ++j) {
            const int t = (base + j * kScanThreads) / COLUMNS, c = (base + j * kScanThreads) % COLUMNS;
            value[j] = t < count && c < channels ? source[t * row_stride + c] : 0.0f;
        }
#pragma unroll
        for (int j = 0; j < kAtATime; ++j) store((base + j * kScanThreads) / COLUMNS, (base + j * kScanThreads) % COLUMNS, value[j]);
    }
}

// powers[n] = decay^n for n <= 64.
__device__ inline void load_powers(float* powers, float decay) {
    if (threadIdx.x <= kScanChunk) powers[threadIdx.x] = threadIdx.x == 0 ? 1.0f : powf(decay, static_cast<float>(threadIdx.x));
}

// added[number][head][d][c] = sum_t decay^(n - 1 - t) k_t[d] v_t[c].
template <int KEYS, bool SILU>
__global__ void __launch_bounds__(kScanThreads)
gla_chunk_state_kernel(const float* __restrict__ proj, int64_t proj_stride, int k_offset, int v_offset, const float* __restrict__ decay,
                       const int32_t* __restrict__ cu_tokens, float* __restrict__ added, int n_seqs, int heads, int key_dim, int value_dim) {
    __shared__ float keys[kScanChunk][KEYS + 1];
    __shared__ float values[kScanChunk][kScanValues + 1];
    __shared__ float powers[kScanChunk + 1];
    const int number = blockIdx.x, head = blockIdx.y;
    int seq, first, count;
    if (!find_chunk(cu_tokens, n_seqs, number, &seq, &first, &count)) return;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int col = lane % 16, quad = lane / 16;
    const int key_tiles = (key_dim + 15) / 16;
    load_powers(powers, decay[head]);
    const float* row = proj + first * proj_stride;
    load_tile<kScanChunk, KEYS>(row + k_offset + head * key_dim, proj_stride, count, key_dim,
                                [&](int t, int c, float value) { keys[t][c] = scan_input<SILU>(value); });
    float* to = added + (static_cast<int64_t>(number) * heads + head) * key_dim * value_dim;
    for (int v0 = 0; v0 < value_dim; v0 += kScanValues) {
        __syncthreads();      // the tile before has been read (the first time: the powers are there)
        load_tile<kScanChunk, kScanValues>(row + v_offset + head * value_dim + v0, proj_stride, count, value_dim - v0, [&](int t, int c, float value) {
            values[t][c] = t < count ? powers[count - 1 - t] * scan_input<SILU>(value) : 0.0f;
        });
        __syncthreads();
        const int column = v0 + 16 * wave + col;
        for (int tile = 0; tile < key_tiles; ++tile) {
            floatx4 acc = floatx4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int t = 0; t < kScanChunk; t += 4)
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(keys[t + quad][16 * tile + col], values[t + quad][16 * wave + col], acc, 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = 16 * tile + 4 * quad + i;
                if (d < key_dim && column < value_dim) to[static_cast<int64_t>(d) * value_dim + column] = acc[i];
            }
        }
    }
}

// A request's chunks in order: what a chunk adds is replaced by the state it begins with; the state after the last one
// goes back to the request's slot.
__global__ void __launch_bounds__(256)
gla_chunk_carry_kernel(float* __restrict__ added, const float* __restrict__ decay, float* __restrict__ state,
                       const int32_t* __restrict__ cu_tokens, const int32_t* __restrict__ slots, int heads, int elements) {
    const int seq = blockIdx.x, head = blockIdx.y;
    const int element = blockIdx.z * blockDim.x + threadIdx.x;
    const int begin = cu_tokens[seq], tokens = cu_tokens[seq + 1] - begin;
    if (tokens <= 0 || element >= elements) return;
    const int chunks = (tokens + kScanChunk - 1) / kScanChunk;
    const int64_t step = static_cast<int64_t>(heads) * elements;
    float* place = added + (static_cast<int64_t>(begin / kScanChunk + seq) * heads + head) * elements + element;
    float* kept = state + (static_cast<int64_t>(slots[seq]) * heads + head) * elements + element;
    const float whole = powf(decay[head], static_cast<float>(kScanChunk));
    const int last = tokens - (chunks - 1) * kScanChunk;
    const float partly = powf(decay[head], static_cast<float>(last));
    float s = *kept;
    constexpr int kAtATime = 8;      // chunks asked for at a time, then walked in order
    for (int base = 0; base < chunks; base += kAtATime) {
        float more[kAtATime];
#pragma unroll
        for (int j = 0; j < kAtATime; ++j) more[j] = base + j < chunks ? place[(base + j) * step] : 0.0f;
#pragma unroll
        for (int j = 0; j < kAtATime; ++j)
            if (base + j < chunks) {
                place[(base + j) * step] = s;
                s = fmaf(base + j + 1 < chunks ? whole : partly, s, more[j]);
            }
    }
    *kept = s;
}

// The results of a chunk's tokens; wave w takes tokens 16 w .. 16 w + 15 of it.
template <int KEYS, bool SILU>
__global__ void __launch_bounds__(kScanThreads)
gla_chunk_out_kernel(const float* __restrict__ proj, int64_t proj_stride, int q_offset, int k_offset, int v_offset,
                     const float* __restrict__ decay, const int32_t* __restrict__ cu_tokens, const float* __restrict__ starts,
                     float* __restrict__ out, int n_seqs, int heads, int key_dim, int value_dim, float q_scale) {
    __shared__ float queries[kScanChunk][KEYS + 1];
    __shared__ float keys[kScanChunk][KEYS + 1];
    __shared__ float start[KEYS][kScanValues + 1];
    __shared__ float values[kScanChunk][kScanValues + 1];
    __shared__ float weights[kScanChunk][kScanChunk + 1];
    __shared__ float powers[kScanChunk + 1];
    const int number = blockIdx.x, head = blockIdx.y;
    int seq, first, count;
    if (!find_chunk(cu_tokens, n_seqs, number, &seq, &first, &count)) return;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int col = lane % 16, quad = lane / 16;
    const int padded = (key_dim + 15) / 16 * 16;
    load_powers(powers, decay[head]);
    const float* row = proj + first * proj_stride;
    load_tile<kScanChunk, KEYS>(row + q_offset + head * key_dim, proj_stride, count, key_dim,
                                [&](int t, int c, float value) { queries[t][c] = scan_input<SILU>(value); });
    load_tile<kScanChunk, KEYS>(row + k_offset + head * key_dim, proj_stride, count, key_dim,
                                [&](int t, int c, float value) { keys[t][c] = scan_input<SILU>(value); });
    __syncthreads();
    // weights[t][j] = decay^(t - j) q_t . k_j for j <= t
    for (int tile = 0; tile <= wave; ++tile) {
        floatx4 acc = floatx4{0.0f, 0.0f, 0.0f, 0.0f};
        for (int d = 0; d < padded; d += 4)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(queries[16 * wave + col][d + quad], keys[16 * tile + col][d + quad], acc, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int t = 16 * wave + 4 * quad + i, j = 16 * tile + col;
            weights[t][j] = j <= t ? acc[i] * powers[t - j] : 0.0f;
        }
    }
    const float* from = starts + (static_cast<int64_t>(number) * heads + head) * key_dim * value_dim;
    for (int v0 = 0; v0 < value_dim; v0 += kScanValues) {
        __syncthreads();      // the tile before has been read (the first time: the weights are there)
        load_tile<kScanChunk, kScanValues>(row + v_offset + head * value_dim + v0, proj_stride, count, value_dim - v0,
                                           [&](int t, int c, float value) { values[t][c] = scan_input<SILU>(value); });
        load_tile<KEYS, kScanValues>(from + v0, value_dim, key_dim, value_dim - v0, [&](int d, int c, float value) { start[d][c] = value; });
        __syncthreads();
        for (int tile = 0; tile < kScanValues / 16; ++tile) {
            const int column = v0 + 16 * tile + col;
            if (v0 + 16 * tile >= value_dim) break;
            floatx4 acc = floatx4{0.0f, 0.0f, 0.0f, 0.0f};
            for (int d = 0; d < padded; d += 4)
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(queries[16 * wave + col][d + quad], start[d + quad][16 * tile + col], acc, 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] *= powers[16 * wave + 4 * quad + i + 1];
            for (int j = 0; j < 16 * (wave + 1); j += 4)
                acc = __builtin_amdgcn_mfma_f32_16x16x4f32(weights[16 * wave + col][j + quad], values[j + quad][16 * tile + col], acc, 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int t = 16 * wave + 4 * quad + i;
                if (t < count && column < value_dim)
                    out[(static_cast<int64_t>(first + t) * heads + head) * value_dim + column] = acc[i] * q_scale;
            }
        }
    }
}

}  // namespace mll

using namespace mll;

extern "C" {

int64_t mll_gla_chunks_scratch(int n_tokens, int n_seqs, int heads, int key_dim, int value_dim) {
    return (static_cast<int64_t>(n_tokens) / kScanChunk + n_seqs) * heads * key_dim * value_dim;
}

int mll_gla_chunks(const float* proj, int64_t proj_stride, int q_offset, int k_offset, int v_offset, const float* decay, float* state,
                   const int32_t* cu_tokens, const int32_t* slots, float* out, float* scratch, int n_tokens, int n_seqs, int heads,
                   int key_dim, int value_dim, float q_scale, int silu_inputs, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && n_seqs >= 0 && heads > 0 && key_dim > 0 && value_dim > 0, "gla_chunks: sizes must be positive");
    MLL_REQUIRE(key_dim <= 128, "gla_chunks: key heads wider than 128 are not supported");
    MLL_REQUIRE(q_offset >= 0 && k_offset >= 0 && v_offset >= 0 && q_offset + heads * key_dim <= proj_stride &&
                    k_offset + heads * key_dim <= proj_stride && v_offset + heads * value_dim <= proj_stride,
                "gla_chunks: a projection lies outside its row");
    if (n_tokens == 0 || n_seqs == 0) return 0;
    const int64_t elements = static_cast<int64_t>(key_dim) * value_dim;
    MLL_REQUIRE(heads <= 65535 && elements <= 65535ll * 256, "gla_chunks: too many heads or a state too large for one launch");
    const dim3 chunks(n_tokens / kScanChunk + n_seqs, heads);
#define MLL_CHUNKS(KEYS, SILU)                                                                                                   \
    do {                                                                                                                         \
        gla_chunk_state_kernel<KEYS, SILU><<<chunks, kScanThreads, 0, stream>>>(proj, proj_stride, k_offset, v_offset, decay, cu_tokens, \
                                                                                scratch, n_seqs, heads, key_dim, value_dim);    \
        gla_chunk_carry_kernel<<<dim3(n_seqs, heads, static_cast<unsigned>((elements + 255) / 256)), 256, 0, stream>>>(         \
            scratch, decay, state, cu_tokens, slots, heads, static_cast<int>(elements));                                        \
        gla_chunk_out_kernel<KEYS, SILU><<<chunks, kScanThreads, 0, stream>>>(proj, proj_stride, q_offset, k_offset, v_offset, decay, \
                                                                              cu_tokens, scratch, out, n_seqs, heads, key_dim, value_dim, q_scale); \
    } while (0)
    if (key_dim <= 64 && silu_inputs) MLL_CHUNKS(64, true);
    else if (key_dim <= 64) MLL_CHUNKS(64, false);
    else if (silu_inputs) MLL_CHUNKS(128, true);
    else MLL_CHUNKS(128, false);
#undef MLL_CHUNKS
    return check_launch("gla_chunks");
}

}  // extern "C"
