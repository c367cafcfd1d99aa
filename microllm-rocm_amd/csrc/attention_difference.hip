// Differential attention: a head has two maps, each an attention of its own over the same values, and gives their
// difference, normed. What the attention kernels leave is combined here: with a_1 and a_2 the maps' results (rows 2 h and
// 2 h + 1 of a token's heads), o = a_1 - lambda * a_2 and out[head h] = o / sqrt(mean(o^2) + eps) * factor over the head's
// `value_dim` channels. The results come in float32, so that the difference is taken of numbers that were not rounded.
#include "common.h"
#include "microllm_hip.h"

namespace mll {

constexpr int kDifferenceWaves = 4;
constexpr int kDifferenceChannelsALane = 4;       // value heads up to 256 channels

template <typename T>
__global__ void __launch_bounds__(kDifferenceWaves * kWave)
attention_difference_kernel(const float* __restrict__ maps, int64_t map_stride, T* __restrict__ out, int64_t total, int heads,
                            int value_dim, float lambda, float eps, float factor) {
    const int64_t item = static_cast<int64_t>(blockIdx.x) * kDifferenceWaves + threadIdx.x / kWave;      // a wave a (token, head)
    if (item >= total) return;
    const int lane = threadIdx.x % kWave;
    const float* first = maps + 2 * item * map_stride;
    const float* second = first + map_stride;
    float o[kDifferenceChannelsALane];
    float squares = 0.0f;
#pragma unroll
    for (int m = 0; m < kDifferenceChannelsALane; ++m) {
        const int c = lane + m * kWave;
        o[m] = c < value_dim ? first[c] - lambda * second[c] : 0.0f;
        squares = fmaf(o[m], o[m], squares);
    }
    const float scale = factor / sqrtf(wave_sum(squares) / static_cast<float>(value_dim) + eps);
    T* to = out + item * value_dim;
#pragma unroll
    for (int m = 0; m < kDifferenceChannelsALane; ++m) {
        const int c = lane + m * kWave;
        if (c < value_dim) to[c] = from_float<T>(o[m] * scale);
    }
}

}  // namespace mll

using namespace mll;

extern "C" int mll_attention_difference(const float* maps, int64_t map_stride, void* out, int dtype, int n_tokens, int heads,
                                        int value_dim, float lambda, float eps, float factor, hipStream_t stream) {
    MLL_REQUIRE(n_tokens >= 0 && heads > 0 && value_dim > 0 && map_stride >= value_dim, "attention_difference: sizes must be positive");
    MLL_REQUIRE(value_dim <= kDifferenceChannelsALane * kWave, "attention_difference: value heads wider than 256 are not supported");
    MLL_REQUIRE(eps > 0.0f, "attention_difference: eps must be positive");
    if (n_tokens == 0) return 0;
    const int64_t total = static_cast<int64_t>(n_tokens) * heads;
    const int64_t blocks = (total + kDifferenceWaves - 1) / kDifferenceWaves;
    MLL_REQUIRE(blocks < (1ll << 31), "attention_difference: too many rows for one launch");
    if (dtype == kF32) {
        attention_difference_kernel<float><<<static_cast<unsigned>(blocks), kDifferenceWaves * kWave, 0, stream>>>(
            maps, map_stride, static_cast<float*>(out), total, heads, value_dim, lambda, eps, factor);
    } else if (dtype == kBF16) {
        attention_difference_kernel<bf16><<<static_cast<unsigned>(blocks), kDifferenceWaves * kWave, 0, stream>>>(
            maps, map_stride, static_cast<bf16*>(out), total, heads, value_dim, lambda, eps, factor);
    } else {
        return fail("attention_difference: unknown dtype");
    }
    return check_launch("attention_difference");
}
