// RMS norm over the float32 residual stream when several sublayers add to it at once: every sublayer hands on its result as
// partial sums in a tensor of its own, and one kernel adds them all (source by source, parts in order), writes the sum
// into the stream and norms it. The same as rms_norm (elementwise.hip) but for where the parts lie.
#include "common.h"
#include "microllm_hip.h"

namespace mll {

// The address of part j counted over all sources: the sources' parts lie part_stride elements apart.
__device__ inline const float* part_of(const MllDeltas& deltas, int j, int64_t part_stride) {
    const float* from = deltas.from[0];
    int first = 0, before = deltas.parts[0];
#pragma unroll
    for (int source = 1; source < kMllDeltaSources; ++source) {
        if (source < deltas.count && j >= before) {
            from = deltas.from[source];
            first = before;
        }
        before += source < deltas.count ? deltas.parts[source] : 0;
    }
    return from + static_cast<int64_t>(j - first) * part_stride;
}

template <typename T>
__global__ void rms_norm_sum_kernel(float* __restrict__ h, MllDeltas deltas, int n_parts, int64_t part_stride,
                                    const int32_t* __restrict__ rows, const float* __restrict__ weight, float eps,
                                    T* __restrict__ out, int width, int write_h) {
    __shared__ float scratch[16];
    const int64_t source = rows ? rows[blockIdx.x] : static_cast<int64_t>(blockIdx.x);
    float* h_row = h + source * width;
    T* out_row = out + static_cast<int64_t>(blockIdx.x) * width;
    auto sum_at = [&](int column) {
        float sum = part_of(deltas, 0, part_stride)[source * width + column];
        for (int j = 1; j < n_parts; ++j) sum += part_of(deltas, j, part_stride)[source * width + column];
        return h_row[column] + sum;
    };
    float squares = 0.0f;
    for (int column = threadIdx.x; column < width; column += blockDim.x) {
        const float value = sum_at(column);
        squares += value * value;
        if (write_h) h_row[column] = value;
    }
    const float inverse_rms = 1.0f / sqrtf(block_sum(squares, scratch) / static_cast<float>(width) + eps);
    for (int column = threadIdx.x; column < width; column += blockDim.x) {
        const float value = write_h ? h_row[column] : sum_at(column);       // a thread reads what it wrote itself
        out_row[column] = from_float<T>(value * inverse_rms * weight[column]);
    }
}

// Rows of float4, kept in registers between the sum of squares and the scaling; eight parts are asked for at a time.
template <typename T, int CHUNKS>
__global__ void rms_norm_sum_vec4_kernel(float* __restrict__ h, MllDeltas deltas, int n_parts, int64_t part_stride,
                                         const int32_t* __restrict__ rows, const float* __restrict__ weight, float eps,
                                         T* __restrict__ out, int width, int write_h) {
    __shared__ float scratch[16];
    const int64_t source = rows ? rows[blockIdx.x] : static_cast<int64_t>(blockIdx.x);
    float* h_row = h + source * width;
    T* out_row = out + static_cast<int64_t>(blockIdx.x) * width;
    const int quads = width / 4;
    float4 value[CHUNKS];
    float squares = 0.0f;
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int q = threadIdx.x + c * blockDim.x;
        value[c] = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
        if (q < quads) {
            const int64_t at = source * width + 4 * q;
            value[c] = reinterpret_cast<const float4*>(h_row)[q];
            float4 sum = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
            constexpr int kAtATime = 8;
            for (int base = 0; base < n_parts; base += kAtATime) {
                float4 more[kAtATime];
#pragma unroll
                for (int j = 0; j < kAtATime; ++j)
                    if (base + j < n_parts) more[j] = *reinterpret_cast<const float4*>(part_of(deltas, base + j, part_stride) + at);
#pragma unroll
                for (int j = 0; j < kAtATime; ++j)
                    if (base + j < n_parts) {
                        sum.x += more[j].x;
                        sum.y += more[j].y;
                        sum.z += more[j].z;
                        sum.w += more[j].w;
                    }
            }
            value[c].x += sum.x;
            value[c].y += sum.y;
            value[c].z += sum.z;
            value[c].w += sum.w;
            if (write_h) reinterpret_cast<float4*>(h_row)[q] = value[c];
            squares += value[c].x * value[c].x + value[c].y * value[c].y + value[c].z * value[c].z + value[c].w * value[c].w;
        }
    }
    const float inverse_rms = 1.0f / sqrtf(block_sum(squares, scratch) / static_cast<float>(width) + eps);
#pragma unroll
    for (int c = 0; c < CHUNKS; ++c) {
        const int q = threadIdx.x + c * blockDim.x;
        if (q < quads) {
            const float4 w = reinterpret_cast<const float4*>(weight)[q];
            T four[4] = {from_float<T>(value[c].x * inverse_rms * w.x), from_float<T>(value[c].y * inverse_rms * w.y),
                         from_float<T>(value[c].z * inverse_rms * w.z), from_float<T>(value[c].w * inverse_rms * w.w)};
#pragma unroll
            for (int i = 0; i < 4; ++i) out_row[4 * q + i] = four[i];
        }
    }
}

template <typename T>
static void launch_rms_norm_sum(float* h, const MllDeltas& deltas, int n_parts, int64_t part_stride, const int32_t* rows,
                                const float* weight, float eps, T* out, int n_rows, int width, int write_h, hipStream_t stream) {
    bool aligned = width % 4 == 0 && reinterpret_cast<uintptr_t>(h) % 16 == 0 && reinterpret_cast<uintptr_t>(weight) % 16 == 0 &&
                   part_stride % 4 == 0;
    for (int source = 0; source < deltas.count; ++source) aligned = aligned && reinterpret_cast<uintptr_t>(deltas.from[source]) % 16 == 0;
    const int quads = width / 4;
    if (aligned && quads <= 1024) {
        rms_norm_sum_vec4_kernel<T, 1><<<n_rows, max(64, (quads + 63) / 64 * 64), 0, stream>>>(h, deltas, n_parts, part_stride, rows, weight,
                                                                                             eps, out, width, write_h);
    } else if (aligned && quads <= 4096) {
        rms_norm_sum_vec4_kernel<T, 4><<<n_rows, 1024, 0, stream>>>(h, deltas, n_parts, part_stride, rows, weight, eps, out, width, write_h);
    } else {
        rms_norm_sum_kernel<T><<<n_rows, width >= 2048 ? 512 : 256, 0, stream>>>(h, deltas, n_parts, part_stride, rows, weight, eps, out,
                                                                                width, write_h);
    }
}

}  // namespace mll

using namespace mll;

extern "C" int mll_rms_norm_sum(float* h, const MllDeltas* deltas, int64_t part_stride, const int32_t* rows, const float* weight,
                                float eps, void* out, int dtype, int n_rows, int width, int write_h, hipStream_t stream) {
    MLL_REQUIRE(n_rows >= 0 && width > 0, "rms_norm_sum: sizes must be positive");
    MLL_REQUIRE(deltas != nullptr && deltas->count >= 1 && deltas->count <= kMllDeltaSources, "rms_norm_sum: one to four sources");
    MLL_REQUIRE(!(write_h && rows), "rms_norm_sum: cannot write the stream through a row selection");
    int n_parts = 0;
    for (int source = 0; source < deltas->count; ++source) {
        MLL_REQUIRE(deltas->from[source] != nullptr && deltas->parts[source] >= 1, "rms_norm_sum: every source has at least one part");
        n_parts += deltas->parts[source];
    }
    if (n_rows == 0) return 0;
    if (dtype == kF32) {
        launch_rms_norm_sum<float>(h, *deltas, n_parts, part_stride, rows, weight, eps, static_cast<float*>(out), n_rows, width, write_h, stream);
    } else if (dtype == kBF16) {
        launch_rms_norm_sum<bf16>(h, *deltas, n_parts, part_stride, rows, weight, eps, static_cast<bf16*>(out), n_rows, width, write_h, stream);
    } else {
        return fail("rms_norm_sum: unknown dtype");
    }
    return check_launch("rms_norm_sum");
}
