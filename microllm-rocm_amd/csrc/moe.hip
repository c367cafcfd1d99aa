// A mixture of experts: the choice of every token's experts from router logits, and the experts' gated
// feed-forwards for (token, choice) pairs whose expert is only known on the device. An expert is gated,
// Wd (act(Wg x) * (Wu x)), or has one inner weight, Wd act(Wu x); act is chosen by number (common.h).
//
// Choice: scores are sigmoid(z) or softmax(z) over the experts, the `top` largest are taken (ties: the lower
// index), their weights are the scores, optionally divided by their sum and multiplied by a factor. A correction a
// expert may be added to the scores for the choice alone. Everything float32. Ids from the number of experts on name
// experts without weights, which return their input: they are chosen like the others and cost no product.
//
// Experts, plain kernels: a workgroup takes one expert and a stretch of its output rows, and goes through the (token, choice)
// pairs that chose it, four at a time, whose inputs lie in LDS; a wave forms eight outputs at a time with its lanes along
// the reduction (16-byte loads of the weight's rows, each used for every pair), so an expert's weights are read once for
// four pairs and a pair's sums never depend on the other pairs. These serve every dtype and number of tokens.
#include "common.h"
#include "microllm_hip.h"

namespace mll {

constexpr int kMaxTop = 16;

// One thread a token (taken beyond 256 experts; fewer go to the kernel below, a wave a token). z: float32 rows, z_stride apart, experts first; a further column `shared_at` (negative: none)
// holds the logit of the shared expert's gate, whose sigmoid goes to shared_gate[t].
__global__ void __launch_bounds__(64)
moe_route_kernel(const float* __restrict__ z, int64_t z_stride, int n_tokens, int experts, int top, int softmax_scores,
                 int renormalize, int shared_at, int32_t* __restrict__ ids, float* __restrict__ weights,
                 float* __restrict__ shared_gate, int groups, int keep, const float* __restrict__ correction, float weight_eps,
                 float weight_scale) {
    const int token = blockIdx.x * blockDim.x + threadIdx.x;
    if (token >= n_tokens) return;
    const float* row = z + static_cast<int64_t>(token) * z_stride;
    float peak = -INFINITY, total = 1.0f;
    if (softmax_scores) {
        for (int e = 0; e < experts; ++e) peak = fmaxf(peak, row[e]);
        total = 0.0f;
        for (int e = 0; e < experts; ++e) total += expf(row[e] - peak);
    }
    auto score = [&](int e) { return softmax_scores ? expf(row[e] - peak) / total : 1.0f / (1.0f + expf(-row[e])); };
    // What decides: without a correction the logit itself, since the scores rise with the logits
    auto deciding = [&](int e) { return correction ? score(e) + correction[e] : row[e]; };
    // Groups of neighbouring experts: a group counts as much as its best expert, and only the experts of the `keep`
    // best groups (ties: the lower group) can be chosen. A bit a group (at most 64).
    unsigned long long open_groups = ~0ull;
    const int group_size = groups > 0 ? experts / groups : experts;
    if (groups > 0 && keep < groups) {
        open_groups = 0ull;
        for (int n = 0; n < keep; ++n) {
            int best_group = -1;
            float best_logit = 0.0f;
            for (int g = 0; g < groups; ++g) {
                if ((open_groups >> g) & 1ull) continue;
                float top_logit = deciding(g * group_size);
                for (int e = 1; e < group_size; ++e) top_logit = fmaxf(top_logit, deciding(g * group_size + e));
                if (best_group < 0 || top_logit > best_logit) {
                    best_group = g;
                    best_logit = top_logit;
                }
            }
            open_groups |= 1ull << best_group;
        }
    }
    int chosen[kMaxTop];
    float taken[kMaxTop];
    float sum = 0.0f;
    for (int n = 0; n < top; ++n) {
        int best = -1;
        float best_logit = 0.0f;
        for (int e = 0; e < experts; ++e) {
            bool used = false;
            for (int m = 0; m < n; ++m) used = used || chosen[m] == e;
            if (used || (groups > 0 && !((open_groups >> (e / group_size)) & 1ull))) continue;
            const float value = deciding(e);     // one that is no number is never larger
            if (best < 0 || value > best_logit) {
                best = e;
                best_logit = value;
            }
        }
        chosen[n] = best;
        taken[n] = score(best);
        sum += taken[n];
    }
    for (int n = 0; n < top; ++n) {
        ids[static_cast<int64_t>(token) * top + n] = chosen[n];
        weights[static_cast<int64_t>(token) * top + n] = (renormalize ? taken[n] / (sum + weight_eps) : taken[n]) * weight_scale;
    }
    if (shared_at >= 0 && shared_gate != nullptr) shared_gate[token] = 1.0f / (1.0f + expf(-row[shared_at]));
}

// The same choice by one wave a token, for up to 64 * PER experts: lane l holds the experts l, l + 64, ...; maxima,
// sums and every "largest of what is left" are taken across the wave, ties to the lower index. The scores' sum is
// added in the wave's order, not in the experts'; everything else is the arithmetic of the kernel above, and a token's
// result depends on its own row alone.
struct Candidate {
    float value;
    int index;
};

__device__ inline Candidate wave_best(Candidate mine) {
#pragma unroll
    for (int offset = kWave / 2; offset > 0; offset >>= 1) {
        const float value = __shfl_xor(mine.value, offset, kWave);
        const int index = __shfl_xor(mine.index, offset, kWave);
        const bool better = index >= 0 && (mine.index < 0 || value > mine.value || (value == mine.value && index < mine.index));
        if (better) {
            mine.value = value;
            mine.index = index;
        }
    }
    return mine;
}

struct RouteForm {      // what mll_moe_route's arguments say, beside the logits and the results
    int experts, top, softmax_scores, renormalize, shared_at, groups, keep;
    const float* correction;
    float weight_eps, weight_scale;
};

template <int PER>
__device__ void route_token(const float* row, int token, int lane, const RouteForm& form, int32_t* __restrict__ ids,
                            float* __restrict__ weights, float* __restrict__ shared_gate) {
    const int experts = form.experts, top = form.top;
    float logit[PER];
    bool free_to_take[PER];
    float peak = -INFINITY;
#pragma unroll
    for (int n = 0; n < PER; ++n) {
        const int e = lane + n * kWave;
        const float value = e < experts ? row[e] : -INFINITY;
        logit[n] = value != value ? -INFINITY : value;       // a logit that is no number is never the largest
        free_to_take[n] = e < experts;
        peak = fmaxf(peak, logit[n]);
    }
    float total = 1.0f;
    if (form.softmax_scores) {
        peak = wave_max(peak);
        float part = 0.0f;
#pragma unroll
        for (int n = 0; n < PER; ++n)
            if (lane + n * kWave < experts) part += expf(logit[n] - peak);
        total = wave_sum(part);
    }
    auto score_of = [&](float value) { return form.softmax_scores ? expf(value - peak) / total : 1.0f / (1.0f + expf(-value)); };
    // What decides over experts and groups: the logits (the scores rise with them), or the scores with their correction;
    // the scores themselves are kept for the weights.
    float score[PER];
#pragma unroll
    for (int n = 0; n < PER; ++n) {
        score[n] = score_of(logit[n]);
        if (form.correction != nullptr) {
            const int e = lane + n * kWave;
            const float value = e < experts ? score[n] + form.correction[e] : -INFINITY;
            logit[n] = value != value ? -INFINITY : value;
        }
    }
    const bool grouped = form.groups > 0 && form.keep < form.groups;
    if (PER == 1) {
        // Up to a wave of places: every lane learns how many stand before it (a larger number, or as large and a lower
        // index), from values that are read lane by lane: no chain of exchanges for every choice.
        auto value_of = [&](int e) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, logit[0]), e)); };
        if (grouped) {
            const int group_size = experts / form.groups, mine = lane / group_size;
            float inside = -INFINITY;
            for (int g = 0, e = 0; g < form.groups; ++g)
                for (int i = 0; i < group_size; ++i, ++e) {
                    const float value = value_of(e);
                    if (g == mine) inside = fmaxf(inside, value);
                }
            int before = 0;
            for (int g = 0; g < form.groups; ++g) {
                const float theirs = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, inside), g * group_size));
                if (theirs > inside || (theirs == inside && g < mine)) ++before;
            }
            free_to_take[0] = free_to_take[0] && before < form.keep;
        }
        const unsigned long long open = __ballot(free_to_take[0]);
        int rank = 0;
        for (int e = 0; e < experts; ++e) {
            const float value = value_of(e);
            if (((open >> e) & 1ull) && (value > logit[0] || (value == logit[0] && e < lane))) ++rank;
        }
        const bool chosen = free_to_take[0] && rank < top;
        float sum = 0.0f;
        for (int choice = 0; choice < top; ++choice) {      // in the order of the choice
            const unsigned long long who = __ballot(chosen && rank == choice);
            if (who != 0ull) sum += __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, score[0]), __ffsll(who) - 1));
        }
        if (chosen) {
            ids[static_cast<int64_t>(token) * top + rank] = lane;
            weights[static_cast<int64_t>(token) * top + rank] = (form.renormalize ? score[0] / (sum + form.weight_eps) : score[0]) * form.weight_scale;
        }
    } else {
        if (grouped) {
            // lane g learns group g's largest number; then the best `keep` groups are opened, one after the other
            const int group_size = experts / form.groups;
            float group_top = -INFINITY;
            for (int g = 0; g < form.groups; ++g) {
                float inside = -INFINITY;
#pragma unroll
                for (int n = 0; n < PER; ++n) {
                    const int e = lane + n * kWave;
                    if (e < experts && e / group_size == g) inside = fmaxf(inside, logit[n]);
                }
                inside = wave_max(inside);
                if (lane == g) group_top = inside;
            }
            unsigned long long open_groups = 0ull;
            for (int n = 0; n < form.keep; ++n) {
                Candidate mine = {group_top, (lane < form.groups && !((open_groups >> lane) & 1ull)) ? lane : -1};
                open_groups |= 1ull << wave_best(mine).index;
            }
#pragma unroll
            for (int n = 0; n < PER; ++n) {
                const int e = lane + n * kWave;
                free_to_take[n] = free_to_take[n] && ((open_groups >> (e / group_size)) & 1ull);
            }
        }
        float sum = 0.0f, my_weight = 0.0f;
        int my_id = 0;
        for (int choice = 0; choice < top; ++choice) {
            Candidate mine = {-INFINITY, -1};
#pragma unroll
            for (int n = 0; n < PER; ++n)       // ascending index: of equal numbers the lower stays
                if (free_to_take[n] && (mine.index < 0 || logit[n] > mine.value)) mine = {logit[n], lane + n * kWave};
            const Candidate best = wave_best(mine);
            float taken = 0.0f;
#pragma unroll
            for (int n = 0; n < PER; ++n) {
                if (lane + n * kWave == best.index) free_to_take[n] = false;
                const float theirs = __shfl(score[n], best.index % kWave, kWave);
                if (best.index / kWave == n) taken = theirs;
            }
            sum += taken;
            if (lane == choice) {
                my_weight = taken;
                my_id = best.index;
            }
        }
        if (lane < top) {
            ids[static_cast<int64_t>(token) * top + lane] = my_id;
            weights[static_cast<int64_t>(token) * top + lane] = (form.renormalize ? my_weight / (sum + form.weight_eps) : my_weight) * form.weight_scale;
        }
    }
    if (lane == 0 && form.shared_at >= 0 && shared_gate != nullptr) shared_gate[token] = 1.0f / (1.0f + expf(-row[form.shared_at]));
}

template <int PER>
__global__ void __launch_bounds__(kWave)
moe_route_wave_kernel(const float* __restrict__ z, int64_t z_stride, RouteForm form, int32_t* __restrict__ ids, float* __restrict__ weights,
                      float* __restrict__ shared_gate) {
    route_token<PER>(z + static_cast<int64_t>(blockIdx.x) * z_stride, blockIdx.x, threadIdx.x, form, ids, weights, shared_gate);
}

// 16 bytes of a row as floats: four of them, or eight bfloat16.
template <typename T> __device__ inline void widen_piece(const uint32_t (&words)[4], float (&out)[16 / sizeof(T)]);
template <> __device__ inline void widen_piece<float>(const uint32_t (&words)[4], float (&out)[4]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) out[i] = __builtin_bit_cast(float, words[i]);
}
template <> __device__ inline void widen_piece<bf16>(const uint32_t (&words)[4], float (&out)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        out[2 * i] = __builtin_bit_cast(float, words[i] << 16);
        out[2 * i + 1] = __builtin_bit_cast(float, words[i] & 0xffff0000u);
    }
}

// A float32 row against TOKENS inputs in LDS, `stride` floats apart, by a wave: 16-byte loads where the row allows, eight asked for
// at a time. A sum takes its terms in the same order whatever TOKENS is.
template <int TOKENS>
__device__ inline void row_dot(const float* __restrict__ w, const float* x, int stride, int k, int lane, float (&sums)[TOKENS]) {
#pragma unroll
    for (int t = 0; t < TOKENS; ++t) sums[t] = 0.0f;
    if ((k & 3) == 0 && (reinterpret_cast<uintptr_t>(w) & 15) == 0) {
        constexpr int kAtATime = 8;
        for (int c0 = lane * 4; c0 < k; c0 += kWave * 4 * kAtATime) {
            float4 row[kAtATime];
#pragma unroll
            for (int n = 0; n < kAtATime; ++n) row[n] = *reinterpret_cast<const float4*>(w + min(c0 + n * kWave * 4, k - 4));
#pragma unroll
            for (int n = 0; n < kAtATime; ++n) {
                const int c = c0 + n * kWave * 4;
                if (c >= k) continue;
#pragma unroll
                for (int t = 0; t < TOKENS; ++t) {
                    const float* at = x + t * stride + c;
                    sums[t] = fmaf(row[n].x, at[0], sums[t]);
                    sums[t] = fmaf(row[n].y, at[1], sums[t]);
                    sums[t] = fmaf(row[n].z, at[2], sums[t]);
                    sums[t] = fmaf(row[n].w, at[3], sums[t]);
                }
            }
        }
    } else {
        for (int c = lane; c < k; c += kWave)
#pragma unroll
            for (int t = 0; t < TOKENS; ++t) sums[t] = fmaf(w[c], x[t * stride + c], sums[t]);
    }
#pragma unroll
    for (int t = 0; t < TOKENS; ++t) sums[t] = wave_sum(sums[t]);
}

// z[t][e] = w[e] . x[t], float32 sums: a workgroup takes a token and four rows of w, a wave a row.
template <typename T>
__global__ void __launch_bounds__(256)
router_logits_kernel(const T* __restrict__ x, const float* __restrict__ w, float* __restrict__ z, int n_out, int width) {
    extern __shared__ float xs[];
    const int token = blockIdx.x;
    for (int c = threadIdx.x; c < width; c += blockDim.x) xs[c] = to_float(x[static_cast<int64_t>(token) * width + c]);
    __syncthreads();
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int e = blockIdx.y * (blockDim.x / kWave) + wave;     // a wave a row of w
    if (e >= n_out) return;
    float value[1];
    row_dot<1>(w + static_cast<int64_t>(e) * width, xs, width, width, lane, value);
    if (lane == 0) z[static_cast<int64_t>(token) * n_out + e] = value[0];
}

// The router's logits and the choice of places by one workgroup for TOKENS tokens: the logits stay in LDS, and a wave a token
// chooses. For up to a wave of places (and what rides with them in w). The same sums as router_logits_kernel's.
constexpr int kRouterWaves = 16;

template <typename T, int TOKENS>
__global__ void __launch_bounds__(kRouterWaves * kWave)
moe_choose_kernel(const T* __restrict__ x, const float* __restrict__ w, int n_tokens, int n_out, int width, RouteForm form,
                  int32_t* __restrict__ ids, float* __restrict__ weights, float* __restrict__ shared_gate) {
    extern __shared__ float xs[];
    __shared__ float z[TOKENS][kWave + 1];
    const int first = blockIdx.x * TOKENS;
#pragma unroll
    for (int t = 0; t < TOKENS; ++t) {
        const T* from = x + static_cast<int64_t>(min(first + t, n_tokens - 1)) * width;
        for (int c = threadIdx.x; c < width; c += blockDim.x) xs[t * width + c] = to_float(from[c]);
    }
    __syncthreads();
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    for (int e = wave; e < n_out; e += kRouterWaves) {
        float value[TOKENS];
        row_dot<TOKENS>(w + static_cast<int64_t>(e) * width, xs, width, width, lane, value);
        if (lane == 0) {
#pragma unroll
            for (int t = 0; t < TOKENS; ++t) z[t][e] = value[t];
        }
    }
    __syncthreads();
    if (wave < TOKENS && first + wave < n_tokens) route_token<1>(z[wave], first + wave, lane, form, ids, weights, shared_gate);
}

constexpr int kExpertWaves = 4;
constexpr int kExpertRowsAWave = 8;     // rows of a weight a wave reads side by side
constexpr int kExpertPairs = 4;         // pairs whose inputs lie in LDS together; an expert with more reads its rows again

// Eight rows of a weight against the inputs of up to four pairs at once: eight loads of 16 bytes on their way a lane, each used
// for every pair. xs holds the pairs' inputs, `stride` elements apart. A sum over a row takes its terms as row_dot does, so a
// pair's result does not depend on which pairs or rows happen to go together.
template <typename T>
__device__ inline void rows_dot(const T* const (&w)[kExpertRowsAWave], const T* xs, int stride, int pairs, int k, int lane,
                                float (&sums)[kExpertPairs][kExpertRowsAWave]) {
    constexpr int kPiece = 16 / sizeof(T);
#pragma unroll
    for (int p = 0; p < kExpertPairs; ++p)
#pragma unroll
        for (int n = 0; n < kExpertRowsAWave; ++n) sums[p][n] = 0.0f;
    bool whole_pieces = k % kPiece == 0;
#pragma unroll
    for (int n = 0; n < kExpertRowsAWave; ++n) whole_pieces = whole_pieces && (reinterpret_cast<uintptr_t>(w[n]) & 15) == 0;
    if (whole_pieces) {
        typedef unsigned int uintx4_t __attribute__((ext_vector_type(4)));
        for (int c = lane * kPiece; c < k; c += kWave * kPiece) {
            uintx4_t raw[kExpertRowsAWave];
#pragma unroll
            for (int n = 0; n < kExpertRowsAWave; ++n) raw[n] = __builtin_nontemporal_load(reinterpret_cast<const uintx4_t*>(w[n] + c));
#pragma unroll
            for (int p = 0; p < kExpertPairs; ++p) {
                if (p >= pairs) break;
                float x[kPiece];
                const uint4 given = *reinterpret_cast<const uint4*>(xs + p * stride + c);
                const uint32_t words[4] = {given.x, given.y, given.z, given.w};
                widen_piece<T>(words, x);
#pragma unroll
                for (int n = 0; n < kExpertRowsAWave; ++n) {
                    const uint32_t row_words[4] = {raw[n][0], raw[n][1], raw[n][2], raw[n][3]};
                    float row[kPiece];
                    widen_piece<T>(row_words, row);
#pragma unroll
                    for (int i = 0; i < kPiece; ++i) sums[p][n] = fmaf(row[i], x[i], sums[p][n]);
                }
            }
        }
    } else {
        for (int c = lane; c < k; c += kWave)
            for (int p = 0; p < pairs; ++p) {
                const float x = to_float(xs[p * stride + c]);
#pragma unroll
                for (int q = 0; q < kExpertPairs; ++q)
                    if (q == p) {
#pragma unroll
                        for (int n = 0; n < kExpertRowsAWave; ++n) sums[q][n] = fmaf(to_float(w[n][c]), x, sums[q][n]);
                    }
            }
    }
#pragma unroll
    for (int p = 0; p < kExpertPairs; ++p) {
        if (p >= pairs) break;
#pragma unroll
        for (int n = 0; n < kExpertRowsAWave; ++n) sums[p][n] = wave_sum(sums[p][n]);
    }
}

// The (token, choice) pairs of one id, a few at a time: from a list in the order of the ids, or, for at most a wave of pairs,
// found by looking at all of them.
struct PairsOfId {
    const int32_t* order;
    unsigned long long mask;
    int count, taken;

    __device__ PairsOfId(const int32_t* ids, int n_pairs, const int32_t* offsets, const int32_t* order_, int first_id, int last_id) {
        taken = 0;
        mask = 0ull;
        order = nullptr;
        if (offsets != nullptr) {
            order = order_ + offsets[first_id];
            count = offsets[last_id + 1] - offsets[first_id];
        } else {
            const int lane = threadIdx.x % kWave;
            const int id = lane < n_pairs ? ids[lane] : -1;
            mask = __ballot(id >= first_id && id <= last_id);
            count = __popcll(mask);
        }
    }
    // As many pairs as there are columns, each lane the one of its own; how many there are.
    __device__ int next_columns(int col, int& mine) {
        const int found = min(count - taken, 16);
        if (order != nullptr) {
            mine = order[taken + min(col, max(found, 1) - 1)];
        } else {
            for (int p = 0; p < found; ++p) {
                const int pair = __ffsll(mask) - 1;
                if (p == col || p == 0) mine = pair;
                mask &= mask - 1ull;
            }
        }
        taken += found;
        return found;
    }
    // The next up to N pairs (the same for every thread of the workgroup); how many there are.
    template <int N>
    __device__ int next(int (&pairs)[N]) {
        int found = 0;
#pragma unroll
        for (int p = 0; p < N; ++p) {
            if (taken >= count) break;
            if (order != nullptr) {
                pairs[p] = order[taken];
            } else {
                pairs[p] = __ffsll(mask) - 1;
                mask &= mask - 1ull;
            }
            ++taken;
            ++found;
        }
        return found;
    }
};

// The places of a token's pairs that need no product: out = x * weight, this workgroup's `columns` columns of every pair of an id
// behind the experts'.
template <typename T>
__device__ inline void return_inputs(const T* x, const int32_t* ids, const float* weights, int top, int n_pairs, const int32_t* offsets,
                                     const int32_t* order, float* out, int part_tokens, int width, const MllExpertForm& form, int columns) {
    PairsOfId of_rest(ids, n_pairs, offsets, order, form.experts, form.experts + form.identity - 1);
    int pairs[kExpertPairs] = {};
    while (const int count = of_rest.next(pairs))
        for (int p = 0; p < count; ++p) {
            const int pair = pairs[p], token = pair / top;
            for (int n = threadIdx.x; n < columns; n += blockDim.x) {
                const int c = blockIdx.x * columns + n;
                if (c < width)
                    out[(static_cast<int64_t>(pair % top) * part_tokens + token) * width + c] = to_float(x[static_cast<int64_t>(token) * width + c]) * weights[pair];
            }
        }
}

// act[pair][f] = act(Wg_e[f] . xs) * (Wu_e[f] . xs), or another gated form (common.h), xs = x[token] * weight[pair] rounded to T
// (the weight multiplies the expert's input) or x[token] (weight_on_input 0). gate_up: [experts][2 * ff][width], gate rows
// first; not gated: [experts][ff][width] and act(Wu_e[f] . xs). A workgroup takes an expert and a stretch of its outputs.
template <typename T>
__global__ void __launch_bounds__(kExpertWaves * kWave)
moe_gate_up_kernel(const T* __restrict__ x, const int32_t* __restrict__ ids, const float* __restrict__ weights, int top, int n_pairs,
                   const int32_t* __restrict__ offsets, const int32_t* __restrict__ order, const T* __restrict__ gate_up,
                   T* __restrict__ act, int width, int ff, int stride, int weight_on_input, MllExpertForm form) {
    extern __shared__ __attribute__((aligned(16))) char lds[];
    T* xs = reinterpret_cast<T*>(lds);
    const int expert = blockIdx.y;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    PairsOfId of_expert(ids, n_pairs, offsets, order, expert, expert);
    const int outputs = form.gated ? kExpertRowsAWave / 2 : kExpertRowsAWave;      // of a wave: a gated one takes two rows
    const int f0 = (blockIdx.x * kExpertWaves + wave) * outputs;
    const T* base = gate_up + static_cast<int64_t>(expert) * (form.gated ? 2 : 1) * ff * width;
    const T* rows[kExpertRowsAWave];
#pragma unroll
    for (int n = 0; n < kExpertRowsAWave; ++n) {        // gated: the gate's and the up's row of one output side by side
        const int f = min(f0 + (form.gated ? n / 2 : n), ff - 1);
        rows[n] = base + static_cast<int64_t>(form.gated && n % 2 == 1 ? ff + f : f) * width;
    }
    int pairs[kExpertPairs] = {};
    while (const int count = of_expert.next(pairs)) {
        __syncthreads();        // the pairs before have been read
#pragma unroll
        for (int p = 0; p < kExpertPairs; ++p) {
            if (p >= count) break;
            const float factor = weight_on_input ? weights[pairs[p]] : 1.0f;
            const T* from = x + static_cast<int64_t>(pairs[p] / top) * width;
            for (int c = threadIdx.x; c < width; c += blockDim.x) xs[p * stride + c] = weight_on_input ? from_float<T>(to_float(from[c]) * factor) : from[c];
        }
        __syncthreads();
        if (f0 >= ff) continue;
        float sums[kExpertPairs][kExpertRowsAWave];
        rows_dot<T>(rows, xs, stride, count, width, lane, sums);
        if (lane == 0) {
#pragma unroll
            for (int p = 0; p < kExpertPairs; ++p) {
                if (p >= count) break;
                T* to = act + static_cast<int64_t>(pairs[p]) * ff + f0;
                if (form.gated) {
#pragma unroll
                    for (int n = 0; n < kExpertRowsAWave / 2; ++n)
                        if (f0 + n < ff) to[n] = from_float<T>(gated_value(sums[p][2 * n], sums[p][2 * n + 1], form.activation, form.limit, form.slope));
                } else {
#pragma unroll
                    for (int n = 0; n < kExpertRowsAWave; ++n)
                        if (f0 + n < ff) to[n] = from_float<T>(activate(sums[p][n], form.activation));
                }
            }
        }
    }
}

// out[choice][token][c] = (Wd_e[c] . act[pair]) (* weight[pair] with weight_on_input 0): float32, parts of part_tokens rows that
// the reader adds in order. down: [experts][width][ff]. The row of workgroups behind the experts' takes the ids that return
// their input.
template <typename T>
__global__ void __launch_bounds__(kExpertWaves * kWave)
moe_down_kernel(const T* __restrict__ x, const T* __restrict__ act, const int32_t* __restrict__ ids, const float* __restrict__ weights,
                int top, int n_pairs, const int32_t* __restrict__ offsets, const int32_t* __restrict__ order, const T* __restrict__ down,
                float* __restrict__ out, int part_tokens, int width, int ff, int stride, int weight_on_input, MllExpertForm form) {
    extern __shared__ __attribute__((aligned(16))) char lds[];
    T* as = reinterpret_cast<T*>(lds);
    const int expert = blockIdx.y;
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    constexpr int kBlockRows = kExpertWaves * kExpertRowsAWave;
    int pairs[kExpertPairs] = {};
    if (expert >= form.experts) {
        return_inputs(x, ids, weights, top, n_pairs, offsets, order, out, part_tokens, width, form, kBlockRows);
        return;
    }
    PairsOfId of_expert(ids, n_pairs, offsets, order, expert, expert);
    const int c0 = blockIdx.x * kBlockRows + wave * kExpertRowsAWave;
    const T* base = down + static_cast<int64_t>(expert) * width * ff;
    const T* rows[kExpertRowsAWave];
#pragma unroll
    for (int n = 0; n < kExpertRowsAWave; ++n) rows[n] = base + static_cast<int64_t>(min(c0 + n, width - 1)) * ff;
    while (const int count = of_expert.next(pairs)) {
        __syncthreads();        // the pairs before have been read
#pragma unroll
        for (int p = 0; p < kExpertPairs; ++p) {
            if (p >= count) break;
            const T* from = act + static_cast<int64_t>(pairs[p]) * ff;
            for (int c = threadIdx.x; c < ff; c += blockDim.x) as[p * stride + c] = from[c];
        }
        __syncthreads();
        if (c0 >= width) continue;
        float sums[kExpertPairs][kExpertRowsAWave];
        rows_dot<T>(rows, as, stride, count, ff, lane, sums);
        if (lane == 0) {
#pragma unroll
            for (int p = 0; p < kExpertPairs; ++p) {
                if (p >= count) break;
                const float factor = weight_on_input ? 1.0f : weights[pairs[p]];
                float* to = out + (static_cast<int64_t>(pairs[p] % top) * part_tokens + pairs[p] / top) * width + c0;
#pragma unroll
                for (int n = 0; n < kExpertRowsAWave; ++n)
                    if (c0 + n < width) to[n] = sums[p][n] * factor;
            }
        }
    }
}

// ---- few bfloat16 pairs on the matrix units ------------------------------------------------------------------------
// The same two steps for bfloat16 and reductions of a multiple of 32: a workgroup takes an expert and kStreamTiles tiles of 16 rows
// of its weight, one after the other; its waves share the reduction, eight steps of 32 each. A wave brings the inputs of up
// to 16 pairs of the expert for its part of the reduction into registers once, streams its part of every tile's rows from memory
// (the next tile's loads on their way while this one is multiplied) through v_mfma_f32_16x16x32_bf16 with the pairs as columns,
// and the waves' sums are added in wave order through LDS. A weight is thus read once for 16 pairs. A pair's sums do not
// depend on the other columns.
typedef __bf16 stream_bf16x8 __attribute__((ext_vector_type(8)));
typedef float stream_floatx4 __attribute__((ext_vector_type(4)));
typedef unsigned int stream_uintx4 __attribute__((ext_vector_type(4)));

constexpr int kStreamTiles = 2;
constexpr int kStreamSteps = 8;         // of 32 terms a wave
constexpr int kStreamWaves = 16;        // of a workgroup, at most: reductions from 256 to 4096 terms

// FORM as in moe_grouped_kernel: 1 gated (a tile holds 8 gate rows and their 8 up rows by turns), 2 one inner weight, 0 down (to the
// pair's token and choice, float32, times its weight). n_out: outputs of an expert; k: the reduction; `in` is x (rows of tokens)
// for forms 1 and 2, and the inner activations (rows of pairs) for form 0.
template <int FORM>
__global__ void __launch_bounds__(kStreamWaves * kWave)
moe_stream_kernel(const bf16* __restrict__ x, const bf16* __restrict__ in, const int32_t* __restrict__ ids, const float* __restrict__ weights,
                  int top, int n_pairs, const int32_t* __restrict__ offsets, const int32_t* __restrict__ order, const bf16* __restrict__ w,
                  void* __restrict__ out, int part_tokens, int n_out, int k, int weight_on_input, MllExpertForm form) {
    extern __shared__ __attribute__((aligned(16))) char lds[];
    stream_floatx4* slots = reinterpret_cast<stream_floatx4*>(lds);        // [2][waves - 1][64]
    constexpr int kOutputsATile = FORM == 1 ? 8 : 16;
    const int expert = blockIdx.y;
    if (FORM == 0 && expert >= form.experts) {
        return_inputs(x, ids, weights, top, n_pairs, offsets, order, static_cast<float*>(out), part_tokens, n_out, form, kStreamTiles * kOutputsATile);
        return;
    }
    const int lane = threadIdx.x % kWave, wave = threadIdx.x / kWave, waves = blockDim.x / kWave;
    const int col = lane % 16, quad = lane / 16;
    PairsOfId of_expert(ids, n_pairs, offsets, order, expert, expert);
    if (of_expert.count == 0) return;       // the same for every wave
    // The last wave begins early enough to have eight steps; the inputs of those that another wave has are zeros.
    const int own_step = wave * kStreamSteps, step0 = min(own_step, k / 32 - kStreamSteps);
    const int64_t row_stride = k;
    const bf16* w_expert = w + static_cast<int64_t>(expert) * (FORM == 1 ? 2 * n_out : n_out) * row_stride;
    const int first_tile = blockIdx.x * kStreamTiles;
    const int n_tiles = min(kStreamTiles, (n_out + kOutputsATile - 1) / kOutputsATile - first_tile);
    auto load_tile = [&](int tile, int zero, stream_uintx4 (&piece)[kStreamSteps]) {
        const int first = (first_tile + tile) * kOutputsATile;
        int row;
        if (FORM == 1) {
            const int output = min(first + col / 2, n_out - 1);
            row = col % 2 == 0 ? output : n_out + output;
        } else {
            row = min(first + col, n_out - 1);
        }
        const unsigned at = static_cast<unsigned>(row) * static_cast<unsigned>(k) + static_cast<unsigned>(step0 * 32 + quad * 8 + zero);      // of one expert's weight
#pragma unroll
        for (int s = 0; s < kStreamSteps; ++s) piece[s] = *reinterpret_cast<const stream_uintx4*>(w_expert + at + s * 32);
    };
    int mine = 0;       // the pair of this lane's column
    while (const int count = of_expert.next_columns(col, mine)) {
        stream_uintx4 even[kStreamSteps], odd[kStreamSteps];
        int zero = 0;
        asm volatile("v_mov_b32 %0, 0" : "=v"(zero));       // zero, but the compiler cannot tell: the first tile is not kept over the pairs
        load_tile(0, zero, even);
        const bool live = col < count;
        const float weight = weights[mine];
        stream_bf16x8 inputs[kStreamSteps];
        const bf16* from = in + static_cast<int64_t>(FORM == 0 ? mine : mine / top) * row_stride + step0 * 32 + quad * 8;
#pragma unroll
        for (int s = 0; s < kStreamSteps; ++s) inputs[s] = *reinterpret_cast<const stream_bf16x8*>(from + s * 32);
        if (FORM != 0 && weight_on_input) {
#pragma unroll
            for (int s = 0; s < kStreamSteps; ++s)
#pragma unroll
                for (int i = 0; i < 8; ++i) inputs[s][i] = static_cast<__bf16>(static_cast<float>(inputs[s][i]) * weight);
        }
#pragma unroll
        for (int s = 0; s < kStreamSteps; ++s) {
            const unsigned keep = live && step0 + s >= own_step ? ~0u : 0u;
            stream_uintx4 bits = __builtin_bit_cast(stream_uintx4, inputs[s]);
            bits &= stream_uintx4{keep, keep, keep, keep};
            inputs[s] = __builtin_bit_cast(stream_bf16x8, bits);
        }
        auto multiply = [&](int tile, const stream_uintx4 (&piece)[kStreamSteps]) {
            stream_floatx4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int s = 0; s < kStreamSteps; ++s)
                acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(stream_bf16x8, piece[s]), inputs[s], acc, 0, 0, 0);
            // acc[i]: row quad * 4 + i of the tile, pair `col`. The waves' sums meet in one of two places by turns, so that one
            // barrier a tile is enough.
            if (waves > 1) {
                stream_floatx4* here = slots + (tile % 2) * (waves - 1) * kWave;
                if (wave > 0) here[(wave - 1) * kWave + lane] = acc;
                __syncthreads();
                if (wave > 0) return;
                for (int base = 0; base < waves - 1; base += 7) {       // seven asked for at a time, added in wave order
                    stream_floatx4 part[7];
#pragma unroll
                    for (int n = 0; n < 7; ++n) part[n] = here[min(base + n, waves - 2) * kWave + lane];
#pragma unroll
                    for (int n = 0; n < 7; ++n)
                        if (base + n < waves - 1) acc += part[n];
                }
            }
            if (!live) return;
            const int first = (first_tile + tile) * kOutputsATile;
            if (FORM == 1) {
                bf16* to = static_cast<bf16*>(out) + static_cast<int64_t>(mine) * n_out;
#pragma unroll
                for (int i = 0; i < 4; i += 2) {
                    const int column = first + quad * 2 + i / 2;
                    if (column < n_out) to[column] = from_float<bf16>(gated_value(acc[i], acc[i + 1], form.activation, form.limit, form.slope));
                }
            } else if (FORM == 2) {
                bf16* to = static_cast<bf16*>(out) + static_cast<int64_t>(mine) * n_out;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int column = first + quad * 4 + i;
                    if (column < n_out) to[column] = from_float<bf16>(activate(acc[i], form.activation));
                }
            } else {
                const float factor = weight_on_input ? 1.0f : weight;
                float* to = static_cast<float*>(out) + (static_cast<int64_t>(mine % top) * part_tokens + mine / top) * n_out;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int column = first + quad * 4 + i;
                    if (column < n_out) to[column] = acc[i] * factor;
                }
            }
        };
        for (int tile = 0; tile < n_tiles; tile += 2) {
            load_tile(min(tile + 1, n_tiles - 1), zero, odd);
            __builtin_amdgcn_sched_barrier(0);      // the next tile's loads are on their way before this one is waited for
            multiply(tile, even);
            if (tile + 1 >= n_tiles) break;
            load_tile(min(tile + 2, n_tiles - 1), zero, even);
            __builtin_amdgcn_sched_barrier(0);
            multiply(tile + 1, odd);
        }
        if (waves > 1) __syncthreads();     // the first wave has read the places that the next pairs' first tile uses
    }
}

// out[t][c] = factor[t] * sum over parts of in[part][t][c], float32.
__global__ void __launch_bounds__(256)
scale_rows_kernel(const float* __restrict__ in, int n_parts, int64_t part_stride, const float* __restrict__ factor,
                  float* __restrict__ out, int width) {
    const int token = blockIdx.y;
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= width) return;
    const int64_t at = static_cast<int64_t>(token) * width + c;
    float value = in[at];
    for (int part = 1; part < n_parts; ++part) value += in[part * part_stride + at];
    out[at] = value * factor[token];
}

// ---- many pairs: rows sorted by expert and tiled MFMA products ---------------------------------------------------
// With many (token, choice) pairs the pairs are put in the order of their experts (stable: a pair keeps its place
// among its expert's; inputs that are multiplied by their weights are gathered into that order), and every expert
// multiplies its own stretch of rows: a workgroup takes a tile of up to 128 rows of one expert and 128 of its weight's
// rows, stages both through LDS in steps of 64 of the reduction and forms the products with
// v_mfma_f32_16x16x32_bf16 (four waves, 64 x 64 each). Which expert a tile belongs to is read from the device-side
// offsets; the grid has a tile for every case (pairs / 128 + experts), and tiles beyond the last expert's leave at once.
// A row's sums do not depend on the other rows of its tile.

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float floatx4_t __attribute__((ext_vector_type(4)));

// offsets[e] = pairs of the ids before e; order[offsets[e] + n] = the n-th pair (ascending) that named e. A workgroup an id: a
// thread looks at a run of neighbouring pairs, counts those of lower ids and its own, learns how many of its own stand before
// its run, and goes over the run again.
constexpr int kSortThreads = 1024;

__global__ void __launch_bounds__(kSortThreads)
moe_sort_kernel(const int32_t* __restrict__ ids, int n_pairs, int named, int32_t* __restrict__ offsets, int32_t* __restrict__ order) {
    __shared__ int lower_of_wave[kSortThreads / kWave], own_of_wave[kSortThreads / kWave];
    const int id = blockIdx.x, lane = threadIdx.x % kWave, wave = threadIdx.x / kWave;
    const int run = (n_pairs + kSortThreads - 1) / kSortThreads;
    const int first = min(static_cast<int>(threadIdx.x) * run, n_pairs), last = min(first + run, n_pairs);
    int lower = 0, own = 0;
    for (int p = first; p < last; ++p) {
        const int named_here = ids[p];
        lower += named_here < id ? 1 : 0;
        own += named_here == id ? 1 : 0;
    }
    int up_to_me = own;         // of the wave's threads up to this one
    for (int offset = 1; offset < kWave; offset <<= 1) {
        const int theirs = __shfl_up(up_to_me, offset, kWave);
        if (lane >= offset) up_to_me += theirs;
    }
    for (int offset = kWave / 2; offset > 0; offset >>= 1) lower += __shfl_xor(lower, offset, kWave);
    if (lane == kWave - 1) own_of_wave[wave] = up_to_me;
    if (lane == 0) lower_of_wave[wave] = lower;
    __syncthreads();
    int base = 0, before = 0, all = 0;
    for (int w = 0; w < kSortThreads / kWave; ++w) {
        base += lower_of_wave[w];
        before += w < wave ? own_of_wave[w] : 0;
        all += own_of_wave[w];
    }
    if (threadIdx.x == 0) {
        offsets[id] = base;
        if (id == named - 1) offsets[named] = base + all;
    }
    int at = base + before + up_to_me - own;
    for (int p = first; p < last; ++p)
        if (ids[p] == id) order[at++] = p;
}

// sorted[row] = x[token of order[row]] * weight of the pair, rounded to bfloat16: where the weight multiplies the expert's input.
// Otherwise the products read the tokens' rows where they lie.
__global__ void __launch_bounds__(256)
moe_gather_kernel(const bf16* __restrict__ x, const int32_t* __restrict__ order, const float* __restrict__ weights, int top,
                  bf16* __restrict__ sorted, int width) {
    const int row = blockIdx.x;
    const int pair = order[row];
    const bf16* from = x + static_cast<int64_t>(pair / top) * width;
    const float factor = weights[pair];
    bf16* to = sorted + static_cast<int64_t>(row) * width;
    for (int c = threadIdx.x; c < width; c += blockDim.x) to[c] = from_float<bf16>(to_float(from[c]) * factor);
}

constexpr int kGroupRows = 128, kGroupCols = 128, kGroupStep = 64, kGroupPad = 72;     // rows of a tile lie 144 bytes apart in LDS: 16-byte reads of 16 rows meet no bank twice

// FORM 2: w is [experts][n_out][k] and out (bfloat16 [pairs][n_out], sorted order) gets activation(product).
// FORM 1 (GATED): w is [experts][2 * n_half][k] (gate rows, then up rows); a tile holds 64 gate rows and the 64 up rows that
// belong to them, and out (bfloat16 [pairs][n_half], sorted order) gets act(gate) * up or another gated form. Otherwise w is
// [experts][n_out][k] and out (float32 [top][n_tokens][n_out]) gets the product at the pair's token and choice,
// times the pair's weight unless that multiplied the input.
template <int FORM>
__global__ void __launch_bounds__(256, 2)
moe_grouped_kernel(const bf16* __restrict__ a, const bf16* __restrict__ w, const int32_t* __restrict__ offsets,
                   const int32_t* __restrict__ order, const float* __restrict__ weights, int n_out, int k,
                   void* __restrict__ out, int top, int n_tokens, int weight_on_input, int from_tokens, const bf16* __restrict__ x,
                   MllExpertForm form) {
    const int experts = form.experts, activation = form.activation;
    constexpr bool GATED = FORM == 1;
    __shared__ __attribute__((aligned(16))) bf16 a_tile[kGroupRows * kGroupPad];
    __shared__ __attribute__((aligned(16))) bf16 w_tile[kGroupCols * kGroupPad];
    int expert = 0, first_row = 0, rows = 0, before = 0;
    for (; expert < experts; ++expert) {
        const int begin = offsets[expert], end = offsets[expert + 1];
        const int tiles = (end - begin + kGroupRows - 1) / kGroupRows;
        if (static_cast<int>(blockIdx.y) < before + tiles) {
            first_row = begin + (blockIdx.y - before) * kGroupRows;
            rows = min(kGroupRows, end - first_row);
            break;
        }
        before += tiles;
    }
    if (rows == 0) {        // a tile beyond the last expert's (the same for every thread of the workgroup)
        if (FORM != 0 || form.identity == 0) return;
        // the pairs of ids that return their input stand behind the experts': their inputs times their weights
        first_row = offsets[experts] + (static_cast<int>(blockIdx.y) - before) * kGroupRows;
        rows = min(kGroupRows, offsets[experts + form.identity] - first_row);
        const int column = blockIdx.x * kGroupCols + threadIdx.x % (kGroupCols / 8) * 8;      // n_out is a multiple of 8: eight columns or none
        if (column >= n_out) return;
#pragma unroll 4
        for (int row = threadIdx.x / (kGroupCols / 8); row < rows; row += 256 / (kGroupCols / 8)) {
            const int pair = order[first_row + row];
            const float weight = weights[pair];
            const uint4 given = *reinterpret_cast<const uint4*>(x + static_cast<int64_t>(pair / top) * n_out + column);
            const uint32_t words[4] = {given.x, given.y, given.z, given.w};
            float value[8];
            widen_piece<bf16>(words, value);
            float4* to = reinterpret_cast<float4*>(static_cast<float*>(out) + (static_cast<int64_t>(pair % top) * n_tokens + pair / top) * n_out + column);
            to[0] = make_float4(value[0] * weight, value[1] * weight, value[2] * weight, value[3] * weight);
            to[1] = make_float4(value[4] * weight, value[5] * weight, value[6] * weight, value[7] * weight);
        }
        return;
    }
    const int w_rows = GATED ? 2 * n_out : n_out;
    const bf16* w_expert = w + static_cast<int64_t>(expert) * w_rows * k;
    constexpr int kTiles = kGroupCols / 32;        // of 16 weight rows, of a wave
    const int col0 = blockIdx.x * (GATED ? kGroupCols / 2 : kGroupCols);
    const int t = threadIdx.x, lane = t % kWave, wave = t / kWave;
    const int wm = wave / 2, wn = wave % 2, r = lane % 16, quad = lane / 16;

    // what this thread brings into LDS each step: 16-byte pieces of the rows' tile and of the weight's
    constexpr int kRowPieces = kGroupRows * (kGroupStep / 8) / 256, kWeightPieces = kGroupCols * (kGroupStep / 8) / 256;
    const int segment = t % (kGroupStep / 8), piece_row = t / (kGroupStep / 8);
    constexpr int kRowsAPass = 256 / (kGroupStep / 8);
    const bf16* a_from[kRowPieces];
    const bf16* w_from[kWeightPieces];
#pragma unroll
    for (int i = 0; i < kRowPieces; ++i) {
        const int row = piece_row + i * kRowsAPass;
        // from_tokens: `a` holds the tokens' rows, not the pairs' in sorted order
        const int a_row = row >= rows ? 0 : (from_tokens ? order[first_row + row] / top : first_row + row);
        a_from[i] = row < rows ? a + static_cast<int64_t>(a_row) * k + segment * 8 : nullptr;
    }
#pragma unroll
    for (int i = 0; i < kWeightPieces; ++i) {
        const int row = piece_row + i * kRowsAPass;
        int w_row;
        bool live;
        if (GATED) {
            const int column = col0 + row % (kGroupCols / 2);
            live = column < n_out;
            w_row = row < kGroupCols / 2 ? column : n_out + column;
        } else {
            w_row = col0 + row;
            live = w_row < n_out;
        }
        w_from[i] = live ? w_expert + static_cast<int64_t>(w_row) * k + segment * 8 : nullptr;
    }
    floatx4_t acc[4][kTiles];
#pragma unroll
    for (int mt = 0; mt < 4; ++mt)
#pragma unroll
        for (int nt = 0; nt < kTiles; ++nt) acc[mt][nt] = floatx4_t{0.0f, 0.0f, 0.0f, 0.0f};
    int w_base[kTiles];
#pragma unroll
    for (int nt = 0; nt < kTiles; ++nt)
        w_base[nt] = GATED ? (nt < kTiles / 2 ? wn * (kGroupCols / 4) + nt * 16 : kGroupCols / 2 + wn * (kGroupCols / 4) + (nt - kTiles / 2) * 16) : wn * (kGroupCols / 2) + nt * 16;

    uint4 a_next[kRowPieces], w_next[kWeightPieces];
    auto fetch = [&](int k0) {
        const bool in_k = k0 + segment * 8 < k;        // k is a multiple of 8: a piece is whole or absent
#pragma unroll
        for (int i = 0; i < kRowPieces; ++i)
            a_next[i] = (a_from[i] != nullptr && in_k) ? *reinterpret_cast<const uint4*>(a_from[i] + k0) : make_uint4(0u, 0u, 0u, 0u);
#pragma unroll
        for (int i = 0; i < kWeightPieces; ++i)
            w_next[i] = (w_from[i] != nullptr && in_k) ? *reinterpret_cast<const uint4*>(w_from[i] + k0) : make_uint4(0u, 0u, 0u, 0u);
    };
    fetch(0);
    for (int k0 = 0; k0 < k; k0 += kGroupStep) {
        __syncthreads();        // the step before has read its tiles
        const int place = piece_row * kGroupPad + segment * 8;
#pragma unroll
        for (int i = 0; i < kRowPieces; ++i) *reinterpret_cast<uint4*>(a_tile + place + i * kRowsAPass * kGroupPad) = a_next[i];
#pragma unroll
        for (int i = 0; i < kWeightPieces; ++i) *reinterpret_cast<uint4*>(w_tile + place + i * kRowsAPass * kGroupPad) = w_next[i];
        __syncthreads();
        if (k0 + kGroupStep < k) fetch(k0 + kGroupStep);      // on its way while this step's products run
#pragma unroll
        for (int half = 0; half < kGroupStep / 32; ++half) {
            bf16x8_t a_piece[4], w_piece[kTiles];
#pragma unroll
            for (int mt = 0; mt < 4; ++mt)
                a_piece[mt] = *reinterpret_cast<const bf16x8_t*>(a_tile + (wm * 64 + mt * 16 + r) * kGroupPad + half * 32 + quad * 8);
#pragma unroll
            for (int nt = 0; nt < kTiles; ++nt)
                w_piece[nt] = *reinterpret_cast<const bf16x8_t*>(w_tile + (w_base[nt] + r) * kGroupPad + half * 32 + quad * 8);
#pragma unroll
            for (int mt = 0; mt < 4; ++mt)
#pragma unroll
                for (int nt = 0; nt < kTiles; ++nt)
                    acc[mt][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_piece[nt], a_piece[mt], acc[mt][nt], 0, 0, 0);
        }
    }
    // acc[mt][nt][i] of lane (r, quad): row wm * 64 + mt * 16 + r of the tile, weight row w_base[nt] + quad * 4 + i
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) {
        const int row = wm * 64 + mt * 16 + r;
        if (row >= rows) continue;
        if (GATED) {
            bf16* to = static_cast<bf16*>(out) + static_cast<int64_t>(first_row + row) * n_out;
#pragma unroll
            for (int nt = 0; nt < kTiles / 2; ++nt)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int column = col0 + wn * (kGroupCols / 4) + nt * 16 + quad * 4 + i;
                    const float g = acc[mt][nt][i], u = acc[mt][nt + kTiles / 2][i];
                    if (column < n_out) to[column] = from_float<bf16>(gated_value(g, u, activation, form.limit, form.slope));
                }
        } else if (FORM == 2) {
            bf16* to = static_cast<bf16*>(out) + static_cast<int64_t>(first_row + row) * n_out;
#pragma unroll
            for (int nt = 0; nt < kTiles; ++nt)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int column = col0 + w_base[nt] + quad * 4 + i;
                    if (column < n_out) to[column] = from_float<bf16>(activate(acc[mt][nt][i], activation));
                }
        } else {
            const int pair = order[first_row + row];
            const float factor = weight_on_input ? 1.0f : weights[pair];
            float* to = static_cast<float*>(out) + (static_cast<int64_t>(pair % top) * n_tokens + pair / top) * n_out;
#pragma unroll
            for (int nt = 0; nt < kTiles; ++nt)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int column = col0 + w_base[nt] + quad * 4 + i;
                    if (column < n_out) to[column] = acc[mt][nt][i] * factor;
                }
        }
    }
}

}  // namespace mll

using namespace mll;

extern "C" {

int mll_moe_route(const float* z, int64_t z_stride, int n_tokens, int experts, int top, int softmax_scores, int renormalize,
                  int shared_at, int32_t* ids, float* weights, float* shared_gate, int groups, int keep, const float* correction,
                  float weight_eps, float weight_scale, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && experts > 0 && top > 0 && top <= experts, "moe_route: 1 <= top <= experts");
    MLL_REQUIRE(top <= (experts <= 4 * kWave ? kWave : kMaxTop),
                "moe_route: at most 64 experts a token (16 where there are more than 256 experts)");
    MLL_REQUIRE(shared_at < 0 || shared_gate != nullptr, "moe_route: the shared expert's gate needs a place");
    MLL_REQUIRE(groups == 0 || (groups > 0 && groups <= 64 && experts % groups == 0 && keep >= 1 && keep <= groups &&
                                keep * (experts / groups) >= top),
                "moe_route: at most 64 equal groups, of which the kept ones hold at least `top` experts");
    if (n_tokens == 0) return 0;
    const RouteForm form = {experts, top, softmax_scores, renormalize, shared_at, groups, keep, correction, weight_eps, weight_scale};
#define MLL_ROUTE_WAVE(PER) moe_route_wave_kernel<PER><<<n_tokens, kWave, 0, stream>>>(z, z_stride, form, ids, weights, shared_gate)
    if (experts <= kWave) MLL_ROUTE_WAVE(1);
    else if (experts <= 2 * kWave) MLL_ROUTE_WAVE(2);
    else if (experts <= 4 * kWave) MLL_ROUTE_WAVE(4);
    else
        moe_route_kernel<<<(n_tokens + 63) / 64, 64, 0, stream>>>(z, z_stride, n_tokens, experts, top, softmax_scores, renormalize,
                                                                shared_at, ids, weights, shared_gate, groups, keep, correction,
                                                                weight_eps, weight_scale);
#undef MLL_ROUTE_WAVE
    return check_launch("moe_route");
}

static int check_form(const MllExpertForm* form, const char* who) {
    if (form == nullptr || form->experts <= 0 || form->identity < 0) return fail(std::string(who) + ": a form with at least one expert");
    if (form->activation < 0 || form->activation > (form->gated ? 3 : 2)) return fail(std::string(who) + ": 0 SiLU, 1 gelu (erf), 2 gelu (tanh), 3 clamped (gated)");
    if (form->activation == 3 && !(form->limit > 0.0f)) return fail(std::string(who) + ": the limit must be positive");
    return 0;
}

// Pairs in the order of their ids, where there are more than the kernels look through themselves.
static int check_order(const int32_t* offsets, const int32_t* order, int64_t pairs, const char* who) {
    if ((offsets == nullptr) != (order == nullptr)) return fail(std::string(who) + ": offsets and order come together");
    if (offsets == nullptr && pairs > kWave) return fail(std::string(who) + ": more than 64 pairs need their order");
    return 0;
}

// Whether the reduction goes over the matrix units' streaming kernel, and over how many waves of a workgroup.
static bool streams(int dtype, int k) {
    return dtype == kBF16 && k % 32 == 0 && k / 32 >= kStreamSteps && k / 32 <= kStreamWaves * kStreamSteps;
}
static int stream_waves(int k) { return (k / 32 + kStreamSteps - 1) / kStreamSteps; }

int mll_moe_sort(const int32_t* ids, int n_pairs, int named, int32_t* offsets, int32_t* order, hipStream_t stream) {
    MLL_REQUIRE(n_pairs >= 0 && named > 0, "moe_sort: sizes must be positive");
    moe_sort_kernel<<<named, kSortThreads, 0, stream>>>(ids, n_pairs, named, offsets, order);
    return check_launch("moe_sort");
}

int mll_moe_gate_up(const void* x, const int32_t* ids, const float* weights, int top, const int32_t* offsets, const int32_t* order,
                    const void* gate_up, void* act, int dtype, int n_tokens, int width, int ff, int weight_on_input,
                    const MllExpertForm* form, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && top > 0 && width > 0 && ff > 0, "moe_gate_up: sizes must be positive");
    if (check_form(form, "moe_gate_up") != 0) return 1;
    const int64_t pairs = static_cast<int64_t>(n_tokens) * top;
    MLL_REQUIRE(pairs < (1 << 30) && form->experts <= 65535, "moe_gate_up: too many pairs or experts for one launch");
    if (check_order(offsets, order, pairs, "moe_gate_up") != 0) return 1;
    const int stride = (width + 7) / 8 * 8;
    const size_t lds = static_cast<size_t>(stride) * kExpertPairs * (dtype == kF32 ? 4 : 2);
    MLL_REQUIRE(lds <= 160 * 1024, "moe_gate_up: rows wider than 10240 (float32) or 20480 are not supported");
    if (n_tokens == 0) return 0;
    if (streams(dtype, width)) {
        const int waves = stream_waves(width);
        const int tiles = form->gated ? (ff + 7) / 8 : (ff + 15) / 16;
        const dim3 stream_grid((tiles + kStreamTiles - 1) / kStreamTiles, form->experts);
        const size_t places = 2 * static_cast<size_t>(waves - 1) * kWave * sizeof(stream_floatx4);
#define MLL_MOE_STREAM(FORM)                                                                                                   \
    moe_stream_kernel<FORM><<<stream_grid, waves * kWave, places, stream>>>(                                                      \
        static_cast<const bf16*>(x), static_cast<const bf16*>(x), ids, weights, top, static_cast<int>(pairs), offsets, order,       \
        static_cast<const bf16*>(gate_up), act, n_tokens, ff, width, weight_on_input, *form)
        if (form->gated) MLL_MOE_STREAM(1); else MLL_MOE_STREAM(2);
#undef MLL_MOE_STREAM
        return check_launch("moe_gate_up");
    }
    const int outputs = kExpertWaves * (form->gated ? kExpertRowsAWave / 2 : kExpertRowsAWave);
    const dim3 grid((ff + outputs - 1) / outputs, form->experts);
    if (dtype == kF32) {
        moe_gate_up_kernel<float><<<grid, kExpertWaves * kWave, lds, stream>>>(
            static_cast<const float*>(x), ids, weights, top, static_cast<int>(pairs), offsets, order, static_cast<const float*>(gate_up),
            static_cast<float*>(act), width, ff, stride, weight_on_input, *form);
    } else if (dtype == kBF16) {
        moe_gate_up_kernel<bf16><<<grid, kExpertWaves * kWave, lds, stream>>>(
            static_cast<const bf16*>(x), ids, weights, top, static_cast<int>(pairs), offsets, order, static_cast<const bf16*>(gate_up),
            static_cast<bf16*>(act), width, ff, stride, weight_on_input, *form);
    } else {
        return fail("moe_gate_up: unknown dtype");
    }
    return check_launch("moe_gate_up");
}

int mll_moe_down(const void* x, const void* act, const int32_t* ids, const float* weights, int top, const int32_t* offsets,
                 const int32_t* order, const void* down, float* out, int dtype, int n_tokens, int width, int ff, int weight_on_input,
                 const MllExpertForm* form, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && top > 0 && width > 0 && ff > 0, "moe_down: sizes must be positive");
    if (check_form(form, "moe_down") != 0) return 1;
    const int64_t pairs = static_cast<int64_t>(n_tokens) * top;
    MLL_REQUIRE(pairs < (1 << 30) && form->experts < 65535, "moe_down: too many pairs or experts for one launch");
    if (check_order(offsets, order, pairs, "moe_down") != 0) return 1;
    const int stride = (ff + 7) / 8 * 8;
    const size_t lds = static_cast<size_t>(stride) * kExpertPairs * (dtype == kF32 ? 4 : 2);
    MLL_REQUIRE(lds <= 160 * 1024, "moe_down: experts wider than 10240 (float32) or 20480 are not supported");
    if (n_tokens == 0) return 0;
    if (streams(dtype, ff)) {
        const int waves = stream_waves(ff);
        const dim3 stream_grid(((width + 15) / 16 + kStreamTiles - 1) / kStreamTiles, form->experts + (form->identity > 0 ? 1 : 0));
        const size_t places = 2 * static_cast<size_t>(waves - 1) * kWave * sizeof(stream_floatx4);
        moe_stream_kernel<0><<<stream_grid, waves * kWave, places, stream>>>(
            static_cast<const bf16*>(x), static_cast<const bf16*>(act), ids, weights, top, static_cast<int>(pairs), offsets, order,
            static_cast<const bf16*>(down), out, n_tokens, width, ff, weight_on_input, *form);
        return check_launch("moe_down");
    }
    const int outputs = kExpertWaves * kExpertRowsAWave;
    const dim3 grid((width + outputs - 1) / outputs, form->experts + (form->identity > 0 ? 1 : 0));
    if (dtype == kF32) {
        moe_down_kernel<float><<<grid, kExpertWaves * kWave, lds, stream>>>(
            static_cast<const float*>(x), static_cast<const float*>(act), ids, weights, top, static_cast<int>(pairs), offsets, order,
            static_cast<const float*>(down), out, n_tokens, width, ff, stride, weight_on_input, *form);
    } else if (dtype == kBF16) {
        moe_down_kernel<bf16><<<grid, kExpertWaves * kWave, lds, stream>>>(
            static_cast<const bf16*>(x), static_cast<const bf16*>(act), ids, weights, top, static_cast<int>(pairs), offsets, order,
            static_cast<const bf16*>(down), out, n_tokens, width, ff, stride, weight_on_input, *form);
    } else {
        return fail("moe_down: unknown dtype");
    }
    return check_launch("moe_down");
}

int mll_scale_rows(const float* in, int n_parts, int64_t part_stride, const float* factor, float* out, int n_tokens, int width,
                   hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && width > 0 && n_parts >= 1, "scale_rows: sizes must be positive");
    MLL_REQUIRE(n_tokens < 65536, "scale_rows: too many rows for one launch");
    if (n_tokens == 0) return 0;
    scale_rows_kernel<<<dim3((width + 255) / 256, n_tokens), 256, 0, stream>>>(in, n_parts, part_stride, factor, out, width);
    return check_launch("scale_rows");
}

int mll_moe_grouped(const void* x, const int32_t* ids, const float* weights, int top, const void* gate_up, const void* down,
                    int32_t* offsets, int32_t* order, void* sorted, void* act, float* out, int n_tokens,
                    int width, int ff, int weight_on_input, const MllExpertForm* form, hipStream_t stream) {
    MLL_REQUIRE(n_tokens > 0 && top > 0 && width > 0 && ff > 0, "moe_grouped: sizes must be positive");
    if (check_form(form, "moe_grouped") != 0) return 1;
    const int experts = form->experts, named = form->experts + form->identity;
    MLL_REQUIRE(width % 8 == 0 && ff % 8 == 0, "moe_grouped: widths must be multiples of 8");
    const int64_t pairs = static_cast<int64_t>(n_tokens) * top;
    MLL_REQUIRE(pairs < (1 << 30), "moe_grouped: too many (token, expert) pairs");
    const int n_pairs = static_cast<int>(pairs);
    moe_sort_kernel<<<named, kSortThreads, 0, stream>>>(ids, n_pairs, named, offsets, order);
    MLL_REQUIRE(!weight_on_input || sorted != nullptr, "moe_grouped: weights on the inputs need a place for the inputs in order");
    const bf16* inputs = static_cast<const bf16*>(x);
    if (weight_on_input) {
        moe_gather_kernel<<<n_pairs, 256, 0, stream>>>(static_cast<const bf16*>(x), order, weights, top, static_cast<bf16*>(sorted), width);
        inputs = static_cast<const bf16*>(sorted);
    }
    const int tiles = (n_pairs + kGroupRows - 1) / kGroupRows + experts + 1;
    MLL_REQUIRE(tiles < 65536, "moe_grouped: too many tiles of rows for one launch");
#define MLL_MOE_GROUPED(FORM, columns, from, weight, to, n_out, k, from_tokens)                                                   \
    moe_grouped_kernel<FORM><<<dim3(((columns) + kGroupCols - 1) / kGroupCols, tiles), 256, 0, stream>>>(                         \
        from, static_cast<const bf16*>(weight), offsets, order, weights, n_out, k, to, top, n_tokens, weight_on_input, from_tokens, \
        static_cast<const bf16*>(x), *form)
    if (form->gated) MLL_MOE_GROUPED(1, 2 * ff, inputs, gate_up, act, ff, width, !weight_on_input);
    else MLL_MOE_GROUPED(2, ff, inputs, gate_up, act, ff, width, !weight_on_input);
    MLL_MOE_GROUPED(0, width, static_cast<const bf16*>(act), down, out, width, ff, 0);
#undef MLL_MOE_GROUPED
    return check_launch("moe_grouped");
}

int mll_moe_choose(const void* x, int dtype, const float* w, int n_tokens, int n_out, int width, int experts, int top, int softmax_scores,
                   int renormalize, int shared_at, int32_t* ids, float* weights, float* shared_gate, int groups, int keep,
                   const float* correction, float weight_eps, float weight_scale, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && width > 0 && experts > 0 && experts <= kWave && n_out >= experts && n_out <= kWave + 1,
                "moe_choose: at most 64 experts (and one row of w beside theirs)");
    MLL_REQUIRE(static_cast<size_t>(width) * sizeof(float) <= 64 * 1024, "moe_choose: rows wider than 16384 are not supported");
    MLL_REQUIRE(top > 0 && top <= experts, "moe_choose: 1 <= top <= experts");
    MLL_REQUIRE(shared_at < n_out && (shared_at < 0 || shared_gate != nullptr), "moe_choose: the shared expert's gate needs a row and a place");
    MLL_REQUIRE(groups == 0 || (groups > 0 && experts % groups == 0 && keep >= 1 && keep <= groups && keep * (experts / groups) >= top),
                "moe_choose: equal groups, of which the kept ones hold at least `top` experts");
    if (n_tokens == 0) return 0;
    const RouteForm form = {experts, top, softmax_scores, renormalize, shared_at, groups, keep, correction, weight_eps, weight_scale};
    // a prompt's tokens go in fours, so that a row of w is read once for four
    const bool fours = n_tokens >= 512 && static_cast<size_t>(width) * 4 * sizeof(float) <= 64 * 1024;
    const size_t lds = static_cast<size_t>(width) * (fours ? 4 : 1) * sizeof(float);
#define MLL_MOE_CHOOSE(T, TOKENS)                                                                                             \
    moe_choose_kernel<T, TOKENS><<<(n_tokens + TOKENS - 1) / TOKENS, kRouterWaves * kWave, lds, stream>>>(                        \
        static_cast<const T*>(x), w, n_tokens, n_out, width, form, ids, weights, shared_gate)
    if (dtype == kF32) {
        if (fours) MLL_MOE_CHOOSE(float, 4); else MLL_MOE_CHOOSE(float, 1);
    } else if (dtype == kBF16) {
        if (fours) MLL_MOE_CHOOSE(bf16, 4); else MLL_MOE_CHOOSE(bf16, 1);
    } else {
        return fail("moe_choose: unknown dtype");
    }
#undef MLL_MOE_CHOOSE
    return check_launch("moe_choose");
}

int mll_router_logits(const void* x, int dtype, const float* w, float* z, int n_tokens, int n_out, int width, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && n_out > 0 && width > 0, "router_logits: sizes must be positive");
    MLL_REQUIRE(static_cast<size_t>(width) * sizeof(float) <= 64 * 1024, "router_logits: rows wider than 16384 are not supported");
    MLL_REQUIRE(n_out <= 4 * 65535, "router_logits: too many rows of w for one launch");
    if (n_tokens == 0) return 0;
    const size_t lds = static_cast<size_t>(width) * sizeof(float);
    if (dtype == kF32) {
        router_logits_kernel<float><<<dim3(n_tokens, (n_out + 3) / 4), 256, lds, stream>>>(static_cast<const float*>(x), w, z, n_out, width);
    } else if (dtype == kBF16) {
        router_logits_kernel<bf16><<<dim3(n_tokens, (n_out + 3) / 4), 256, lds, stream>>>(static_cast<const bf16*>(x), w, z, n_out, width);
    } else {
        return fail("router_logits: unknown dtype");
    }
    return check_launch("router_logits");
}

}  // extern "C"
