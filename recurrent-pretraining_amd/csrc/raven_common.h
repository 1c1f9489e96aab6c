// Device helpers shared by the gfx950 kernels: dtype traits, 16-byte vector access,
// wave64 reductions built on DPP row operations.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

#include "raven_hip.h"

namespace raven {

typedef __bf16 bf16;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2;
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(16))) float f32x16;

constexpr int kWave = 64;

// One 16-byte chunk of T: 8 bf16 or 4 floats.
template <typename T> struct Chunk;
template <> struct Chunk<float> {
    static constexpr int N = 4;
    float v[4];
};
template <> struct Chunk<bf16> {
    static constexpr int N = 8;
    bf16 v[8];
};

template <typename T>
__device__ __forceinline__ Chunk<T> load_chunk(const T* p) {
    Chunk<T> c;
    *reinterpret_cast<uint4*>(&c) = *reinterpret_cast<const uint4*>(p);
    return c;
}
// for data that is read once per launch: a load hinted to stream past the caches
template <typename T>
__device__ __forceinline__ Chunk<T> load_chunk_stream(const T* p) {
    typedef unsigned int u32x4_t __attribute__((ext_vector_type(4)));
    Chunk<T> c;
    *reinterpret_cast<u32x4_t*>(&c) = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(p));
    return c;
}
template <typename T>
__device__ __forceinline__ void store_chunk(T* p, const Chunk<T>& c) {
    *reinterpret_cast<uint4*>(p) = *reinterpret_cast<const uint4*>(&c);
}
template <typename T>
__device__ __forceinline__ Chunk<T> zero_chunk() {
    Chunk<T> c;
    *reinterpret_cast<uint4*>(&c) = make_uint4(0, 0, 0, 0);
    return c;
}

__device__ __forceinline__ float to_f32(float x) { return x; }
__device__ __forceinline__ float to_f32(bf16 x) { return static_cast<float>(x); }
template <typename T> __device__ __forceinline__ T from_f32(float x);
template <> __device__ __forceinline__ float from_f32<float>(float x) { return x; }
template <> __device__ __forceinline__ bf16 from_f32<bf16>(float x) { return static_cast<bf16>(x); }  // RNE

// round-trip through T: what storing an fp32 value in a T tensor and reading it back gives
template <typename T> __device__ __forceinline__ float round_to(float x) { return to_f32(from_f32<T>(x)); }

// dot of two 16-byte chunks, accumulated in fp32
__device__ __forceinline__ float dot_chunk(const Chunk<float>& a, const Chunk<float>& b, float acc) {
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = __builtin_fmaf(a.v[i], b.v[i], acc);
    return acc;
}
__device__ __forceinline__ float dot_chunk(const Chunk<bf16>& a, const Chunk<bf16>& b, float acc) {
    const bf16x2* pa = reinterpret_cast<const bf16x2*>(&a);
    const bf16x2* pb = reinterpret_cast<const bf16x2*>(&b);
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_fdot2_f32_bf16(pa[i], pb[i], acc, false);
    return acc;
}

// ---- DPP based reductions -------------------------------------------------------------------
template <int CTRL>
__device__ __forceinline__ float dpp_f(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// sum over each row of 16 lanes, result in all 16 lanes
__device__ __forceinline__ float row16_sum(float v) {
    v += dpp_f<0xB1>(v);   // quad_perm [1,0,3,2]
    v += dpp_f<0x4E>(v);   // quad_perm [2,3,0,1]
    v += dpp_f<0x141>(v);  // row_half_mirror
    v += dpp_f<0x140>(v);  // row_mirror
    return v;
}
__device__ __forceinline__ float row16_max(float v) {
    v = fmaxf(v, dpp_f<0xB1>(v));
    v = fmaxf(v, dpp_f<0x4E>(v));
    v = fmaxf(v, dpp_f<0x141>(v));
    v = fmaxf(v, dpp_f<0x140>(v));
    return v;
}
// sum over the 64 lanes of a wave, result in all lanes
__device__ __forceinline__ float wave_sum(float v) {
    v = row16_sum(v);
    v += __shfl_xor(v, 16, 64);
    v += __shfl_xor(v, 32, 64);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
    v = row16_max(v);
    v = fmaxf(v, __shfl_xor(v, 16, 64));
    v = fmaxf(v, __shfl_xor(v, 32, 64));
    return v;
}

// Maximum over the four lanes l, l^16, l^32, l^48 (the lanes that share a query), in every lane, with the two row-swap
// instructions of gfx950 instead of two round trips through the LDS crossbar: after v_permlane16_swap of a register
// with a copy of itself the pair holds rows (0,0,2,2) and (1,1,3,3) of 16 lanes, after v_permlane32_swap the two halves.
__device__ __forceinline__ float max_over_quarters(float x) {
    typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
    // the pair's elements go through plain variables: __builtin_bit_cast of a vector's element reads element 0 whatever the index
    const unsigned u = __builtin_bit_cast(unsigned, x);
    const u32x2 r = __builtin_amdgcn_permlane16_swap(u, u, false, false);
    const unsigned r0 = r[0], r1 = r[1];
    const unsigned v = __builtin_bit_cast(unsigned, fmaxf(__builtin_bit_cast(float, r0), __builtin_bit_cast(float, r1)));
    const u32x2 q = __builtin_amdgcn_permlane32_swap(v, v, false, false);
    const unsigned q0 = q[0], q1 = q[1];
    return fmaxf(__builtin_bit_cast(float, q0), __builtin_bit_cast(float, q1));
}

// x * sigmoid(x).  The reciprocal is the hardware's (1 ulp): its error vanishes in the bf16 rounding that follows and stays
// inside the fp32 bar, and a true division costs five times the instructions in the SwiGLU epilogue of a 256 x 256 tile.
__device__ __forceinline__ float silu_f32(float x) { return x * __builtin_amdgcn_rcpf(1.0f + __expf(-x)); }

__device__ __forceinline__ float sigmoid_f32(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---- the free epilogue of the linear kernels (raven_linear_epilogue) --------------------------------------------
// Which epilogue a linear kernel is compiled with: the nn.Linear one (rounded to T, then a residual in T), SwiGLU, or the
// free one, whose sums stay unrounded until they are stored -- one value per activation, so that a tile's hundreds of
// unrolled elements carry no code for the other activations (with all of them behind run-time branches the 256 x 256 kernel
// outgrew the instruction cache and lost a third of its speed even without an activation).
enum { EPI_PLAIN = 0, EPI_SWIGLU = 1, EPI_FREE = 2, EPI_FREE_GELU = EPI_FREE + RAVEN_ACT_GELU, EPI_FREE_TANH = EPI_FREE + RAVEN_ACT_TANH };
constexpr bool is_free(int epi) { return epi >= EPI_FREE; }

// z (1 + erf(z / sqrt 2)) / 2.  float: the library's erf.  bf16 results: erf by the rational approximation 7.1.26 of Abramowitz and
// Stegun, Handbook of Mathematical Functions (absolute error 1.5e-7), in the form 1 - erf(x) = poly(t) exp(-x^2), t = 1 / (1 + p x).
template <typename T>
__device__ __forceinline__ float gelu_f32(float z) {
    if constexpr (sizeof(T) == 4) {
        return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f));
    } else {
        const float x = fabsf(z) * 0.70710678118654752f;
        const float t = __builtin_amdgcn_rcpf(__builtin_fmaf(0.3275911f, x, 1.0f));
        float p = __builtin_fmaf(1.061405429f, t, -1.453152027f);
        p = __builtin_fmaf(p, t, 1.421413741f);
        p = __builtin_fmaf(p, t, -0.284496736f);
        p = __builtin_fmaf(p, t, 0.254829592f);
        const float tail = p * t * __builtin_amdgcn_exp2f(x * x * -1.4426950408889634f);  // erfc(x)
        return 0.5f * z * (z < 0.f ? tail : 2.0f - tail);
    }
}

// act(scale * z + bias[n]) + residual[at], z an fp32 sum and `at` its element offset in the output
template <typename T, int EPI>
__device__ __forceinline__ float free_epilogue(const raven_epilogue& e, int64_t at, int n, float z) {
    float v = z * e.scale;
    if (e.bias) v += e.bias[n];
    if (EPI == EPI_FREE_GELU) v = gelu_f32<T>(v);
    if (EPI == EPI_FREE_TANH) v = tanhf(v);
    if (e.residual) v += e.residual[at];
    return v;
}
template <typename T, int EPI>
__device__ __forceinline__ void store_free(const raven_epilogue& e, void* y, int64_t at, int n, float z) {
    const float v = free_epilogue<T, EPI>(e, at, n, z);
    if (e.out_f32) static_cast<float*>(y)[at] = v;
    else static_cast<T*>(y)[at] = from_f32<T>(v);
}

// One RoPE pair, adjacent elements (recpre/raven_modeling_minimal.py:118-131): products and sums rounded one by one in
// fp32, as the reference's separate elementwise kernels do; every kernel that rotates uses this one function, so that
// the fused and the two-launch paths write the same bits.
template <typename T>
__device__ __forceinline__ void rope_pair(T& a, T& b, float cs, float sn) {
#pragma clang fp contract(off)
    const float x0 = to_f32(a), x1 = to_f32(b);
    const float r0 = x0 * cs - x1 * sn;
    const float r1 = x1 * cs + x0 * sn;
    a = from_f32<T>(r0);
    b = from_f32<T>(r1);
}

}  // namespace raven

// ---- host side ------------------------------------------------------------------------------
namespace raven_host {
void set_error(const char* fmt, ...);
int  check_launch(const char* what);
inline size_t elt_size(int dtype) { return dtype == RAVEN_BF16 ? 2 : 4; }
inline size_t align_up(size_t x, size_t a = 256) { return (x + a - 1) / a * a; }
}  // namespace raven_host

#define RAVEN_REQUIRE(cond, ...)                 \
    do {                                         \
        if (!(cond)) {                           \
            raven_host::set_error(__VA_ARGS__);  \
            return -1;                           \
        }                                        \
    } while (0)
