// Row-wise device helpers of the kernels over an fp32 residual stream.
#pragma once

#include <math.h>

#include "raven_common.h"

namespace raven {

__device__ __forceinline__ f32x4 load4(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
__device__ __forceinline__ f32x4 load4(const bf16* p) {
    bf16 v[4];
    *reinterpret_cast<uint2*>(v) = *reinterpret_cast<const uint2*>(p);
    return f32x4{to_f32(v[0]), to_f32(v[1]), to_f32(v[2]), to_f32(v[3])};
}
__device__ __forceinline__ void store4(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
__device__ __forceinline__ void store4(bf16* p, f32x4 v) {
    bf16 o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = from_f32<bf16>(v[i]);
    *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(o);
}
template <typename T>
__device__ __forceinline__ float soft_exp(float x) {  // natural exponential of a score difference
    if constexpr (sizeof(T) == 4) return expf(x);
    else return __builtin_amdgcn_exp2f(x * 1.4426950408889634f);
}

// one wave: T(in / rms(in) * w) over n elements (mean over dim), n a multiple of 8
template <typename T, typename Z>
__device__ __forceinline__ void wave_norm(const Z* in, const float* w, T* out, int n, int dim, float eps) {
    const int lane = threadIdx.x & 63;
    float ss = 0.f;
    for (int i = 4 * lane; i < n; i += 256) {
        const f32x4 v = load4(in + i);
        ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)dim + eps);
    for (int i = 4 * lane; i < n; i += 256) store4(out + i, load4(in + i) * inv * load4(w + i));
}

// A product with a small matrix over RB token rows at once, 16 lanes to a weight row (256 threads):
// rows r0 .. r0 + 16 * per_wg - 1 (below n) of w [n, K] against xs [RB][K] in LDS; emit(r, b, sum) in one lane per row
template <typename T, int RB, typename F>
__device__ __forceinline__ void head_product(const T* w, const T* xs, int K, int n, int r0, int per_wg, F&& emit) {
    constexpr int E = Chunk<T>::N;
    const int c16 = threadIdx.x & 15, nc = K / E;
    for (int p = 0; p < per_wg; ++p) {
        const int r = r0 + p * 16 + (threadIdx.x >> 4);
        float acc[RB];
#pragma unroll
        for (int b = 0; b < RB; ++b) acc[b] = 0.f;
        const T* row = w + (int64_t)min(r, n - 1) * K;
        for (int c0 = c16; c0 < nc; c0 += 64) {
            Chunk<T> v[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) v[j] = c0 + 16 * j < nc ? load_chunk(row + (c0 + 16 * j) * E) : zero_chunk<T>();
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int c = min(c0 + 16 * j, nc - 1);
#pragma unroll
                for (int b = 0; b < RB; ++b) acc[b] = dot_chunk(v[j], load_chunk(xs + (int64_t)b * K + c * E), acc[b]);
            }
        }
#pragma unroll
        for (int b = 0; b < RB; ++b) {
            const float s = row16_sum(acc[b]);
            if (c16 == 0 && r < n) emit(r, b, s);
        }
    }
}

}  // namespace raven
