// RMSNorm over an fp32 residual stream, optionally followed by a causal depthwise convolution over time of the normed rows:
//     h_t = x_t / sqrt(mean(x_t^2) + eps) * w
//     y_t = T(h_t + sum_j c_j * h_(t - taps + 1 + j))          (without a convolution: y_t = T(h_t))
// and the two row helpers of such a stream: the scaled embedding gather and the rounding of rows to the product dtype.
//
// The rows h of the last taps - 1 tokens are a sequence's state between calls.  They live in a ring of `taps` fp32 rows per
// sequence, position p in row p mod taps: the row a decode step writes is never one that it reads, so one launch does both,
// and positions before the sequence's start are recognised by their index, so a ring never needs clearing.  A chunk of
// several tokens forms the rows before it from the ring and the rows inside it from x itself (a workgroup walks a tile of
// rows and starts taps - 1 rows early); its last rows go to the ring in a second small launch, when every reader of the
// old ones is done.
//
// Each thread owns the same 4-channel pieces in every row, so the convolution's window is private to a thread: it sits in LDS
// without any barrier, only the row's sum of squares is exchanged.

#include "raven_common.h"

namespace raven {

struct NormConvArgs {
    const float* x;     // [B*S, ld]
    const float* w;     // [ld], zero past dim
    const float* conv;  // [taps, ld] or null
    float* ring;        // [B, taps, ld]
    void* y;            // [B*S, ld]
    int S, dim, ld, taps, pos0, rows_per_wg;
    const int* pos_dev;
    float eps;
};

__device__ __forceinline__ float wg_sum4(float v, float* red) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return red[0] + red[1] + red[2] + red[3];
}

// P: 4-channel pieces per thread.  RING_ONLY: store the normed rows of the chunk's last min(S, taps - 1) tokens to the ring.
template <typename T, int P, bool RING_ONLY>
__global__ __launch_bounds__(256) void norm_conv_kernel(NormConvArgs a) {
    extern __shared__ __align__(16) float window[];  // [taps][ld], with a convolution
    __shared__ float red[4];
    const int b = blockIdx.y, tid = threadIdx.x;
    const int pos0 = a.pos_dev ? *a.pos_dev : a.pos0;
    const int pieces = a.ld / 4;
    f32x4 w[P];
#pragma unroll
    for (int j = 0; j < P; ++j) {
        const int c = tid + 256 * j;
        w[j] = c < pieces ? *reinterpret_cast<const f32x4*>(a.w + 4 * c) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    auto normed = [&](int s, f32x4* h) {  // row s of the chunk
        const float* row = a.x + ((int64_t)b * a.S + s) * a.ld;
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < P; ++j) {
            const int c = tid + 256 * j;
            h[j] = c < pieces ? *reinterpret_cast<const f32x4*>(row + 4 * c) : f32x4{0.f, 0.f, 0.f, 0.f};
            ss += h[j][0] * h[j][0] + h[j][1] * h[j][1] + h[j][2] * h[j][2] + h[j][3] * h[j][3];
        }
        const float inv = 1.0f / sqrtf(wg_sum4(ss, red) / (float)a.dim + a.eps);
#pragma unroll
        for (int j = 0; j < P; ++j) h[j] = h[j] * inv * w[j];
    };
    auto store = [&](int s, const f32x4* h) {
        T* row = static_cast<T*>(a.y) + ((int64_t)b * a.S + s) * a.ld;
#pragma unroll
        for (int j = 0; j < P; ++j) {
            const int c = tid + 256 * j;
            if (c >= pieces) continue;
            if constexpr (sizeof(T) == 4) {
                *reinterpret_cast<f32x4*>(row + 4 * c) = h[j];
            } else {
                bf16 o[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] = from_f32<bf16>(h[j][i]);
                *reinterpret_cast<uint2*>(row + 4 * c) = *reinterpret_cast<const uint2*>(o);
            }
        }
    };
    float* ring = a.ring ? a.ring + (int64_t)b * a.taps * a.ld : nullptr;
    auto to_ring = [&](int s, const f32x4* h) {
        float* row = ring + (int64_t)((pos0 + s) % a.taps) * a.ld;
#pragma unroll
        for (int j = 0; j < P; ++j) {
            const int c = tid + 256 * j;
            if (c < pieces) *reinterpret_cast<f32x4*>(row + 4 * c) = h[j];
        }
    };

    if (RING_ONLY) {
        const int s = a.S - 1 - (int)blockIdx.x;  // the grid covers min(S, taps - 1) rows
        f32x4 h[P];
        normed(s, h);
        to_ring(s, h);
        return;
    }
    const int first = blockIdx.x * a.rows_per_wg, last = min(first + a.rows_per_wg, a.S);
    if (!a.conv) {
        for (int s = first; s < last; ++s) {
            f32x4 h[P];
            normed(s, h);
            store(s, h);
        }
        return;
    }
    for (int s = first - (a.taps - 1); s < last; ++s) {
        f32x4 h[P];
        const int pos = pos0 + s;
        if (s >= 0) {
            normed(s, h);  // the branch is uniform over the workgroup
        } else {
#pragma unroll
            for (int j = 0; j < P; ++j) {
                const int c = tid + 256 * j;
                h[j] = (pos >= 0 && c < pieces) ? *reinterpret_cast<const f32x4*>(ring + (int64_t)(pos % a.taps) * a.ld + 4 * c)
                                                : f32x4{0.f, 0.f, 0.f, 0.f};
            }
        }
        // window row of token s: (s - first + taps - 1) mod taps, counted from the first token of this walk
        const int step = s - first + a.taps - 1;
        const int slot = step % a.taps;
#pragma unroll
        for (int j = 0; j < P; ++j) {
            const int c = tid + 256 * j;
            if (c < pieces) *reinterpret_cast<f32x4*>(window + (int64_t)slot * a.ld + 4 * c) = h[j];
        }
        if (s < first) continue;
        f32x4 o[P];
#pragma unroll
        for (int j = 0; j < P; ++j) o[j] = h[j];
        for (int t = 0; t < a.taps; ++t) {  // tap t sees token s - taps + 1 + t
            const float* hist = window + (int64_t)((step + 1 + t) % a.taps) * a.ld;
            const float* cw = a.conv + (int64_t)t * a.ld;
#pragma unroll
            for (int j = 0; j < P; ++j) {
                const int c = tid + 256 * j;
                if (c < pieces) o[j] += *reinterpret_cast<const f32x4*>(cw + 4 * c) * *reinterpret_cast<const f32x4*>(hist + 4 * c);
            }
        }
        store(s, o);
        if (a.S == 1) to_ring(s, h);
    }
}

// One token per sequence: the row, the weights and every row of the window are requested at once, one memory latency instead of one
// per window row.  TAPS: window rows held (taps <= TAPS; the others are skipped).
template <typename T, int P, int TAPS>
__global__ __launch_bounds__(256) void norm_conv_step_kernel(NormConvArgs a) {
    __shared__ float red[4];
    const int b = blockIdx.x, tid = threadIdx.x;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos0;
    const int pieces = a.ld / 4;
    const float* row = a.x + (int64_t)b * a.ld;
    float* ring = a.ring + (int64_t)b * a.taps * a.ld;
    f32x4 h[P], w[P], c[TAPS][P], past[TAPS][P];
#pragma unroll
    for (int j = 0; j < P; ++j) {
        const int at = 4 * min(tid + 256 * j, pieces - 1);
        h[j] = *reinterpret_cast<const f32x4*>(row + at);
        w[j] = *reinterpret_cast<const f32x4*>(a.w + at);
#pragma unroll
        for (int t = 0; t < TAPS; ++t) {  // t = tokens back; beyond the window or the sequence's start any row will do
            const int back = min(t, a.taps - 1), p = max(pos - back, 0);
            c[t][j] = *reinterpret_cast<const f32x4*>(a.conv + (int64_t)(a.taps - 1 - back) * a.ld + at);
            past[t][j] = *reinterpret_cast<const f32x4*>(ring + (int64_t)(p % a.taps) * a.ld + at);
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < P; ++j)
        if (tid + 256 * j < pieces) ss += h[j][0] * h[j][0] + h[j][1] * h[j][1] + h[j][2] * h[j][2] + h[j][3] * h[j][3];
    const float inv = 1.0f / sqrtf(wg_sum4(ss, red) / (float)a.dim + a.eps);
    T* y = static_cast<T*>(a.y) + (int64_t)b * a.ld;
    float* keep = ring + (int64_t)(pos % a.taps) * a.ld;  // not one of the rows read above, except as the ignored t = 0
#pragma unroll
    for (int j = 0; j < P; ++j) {
        const int at = 4 * (tid + 256 * j);
        if (tid + 256 * j >= pieces) continue;
        const f32x4 n = h[j] * inv * w[j];
        f32x4 o = n;
        for (int t = TAPS - 1; t > 0; --t)  // oldest first, as over chunks
            if (t < a.taps && t <= pos) o += c[t][j] * past[t][j];
        o += c[0][j] * n;
        *reinterpret_cast<f32x4*>(keep + at) = n;
        if constexpr (sizeof(T) == 4) {
            *reinterpret_cast<f32x4*>(y + at) = o;
        } else {
            bf16 q[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) q[i] = from_f32<bf16>(o[i]);
            *reinterpret_cast<uint2*>(y + at) = *reinterpret_cast<const uint2*>(q);
        }
    }
}

// x[m] = float(table[ids[m]]) * scale, and the same row rounded to T
template <typename T>
__global__ __launch_bounds__(256) void embed_stream_kernel(const T* __restrict__ table, const int64_t* __restrict__ ids, float* __restrict__ x,
                                                           T* __restrict__ xt, int ld, int64_t vocab, float scale) {
    constexpr int E = Chunk<T>::N;
    const int64_t m = blockIdx.x;
    int64_t id = ids[m];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);  // never read outside the table
    for (int c = threadIdx.x; c < ld / E; c += 256) {
        Chunk<T> v = load_chunk(table + id * ld + c * E);
        float f[E];
#pragma unroll
        for (int e = 0; e < E; ++e) {
            f[e] = to_f32(v.v[e]) * scale;
            v.v[e] = from_f32<T>(f[e]);
        }
#pragma unroll
        for (int e = 0; e < E; e += 4) *reinterpret_cast<f32x4*>(x + m * ld + c * E + e) = f32x4{f[e], f[e + 1], f[e + 2], f[e + 3]};
        if (xt) store_chunk(xt + m * ld + c * E, v);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void round_rows_kernel(const float* __restrict__ x, T* __restrict__ y, int64_t pieces) {
    const int64_t c = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (c >= pieces) return;
    const f32x4 v = *reinterpret_cast<const f32x4*>(x + 4 * c);
    if constexpr (sizeof(T) == 4) {
        *reinterpret_cast<f32x4*>(y + 4 * c) = v;
    } else {
        bf16 o[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = from_f32<bf16>(v[i]);
        *reinterpret_cast<uint2*>(y + 4 * c) = *reinterpret_cast<const uint2*>(o);
    }
}

template <typename T, int P>
static int launch_norm_conv(const NormConvArgs& a, int B, hipStream_t s) {
    if constexpr (P <= 4) {
        if (a.conv && a.S == 1 && a.taps <= 4) {
            norm_conv_step_kernel<T, P, 4><<<dim3(B), dim3(256), 0, s>>>(a);
            return raven_host::check_launch("norm_conv (step)");
        }
    }
    const size_t lds = a.conv ? (size_t)a.taps * a.ld * sizeof(float) : 0;
    if (lds > 48 * 1024) {
        static bool attr_set = false;
        if (!attr_set) {
            hipError_t e = hipFuncSetAttribute((const void*)norm_conv_kernel<T, P, false>, hipFuncAttributeMaxDynamicSharedMemorySize, 156 * 1024);
            if (e != hipSuccess) {
                raven_host::set_error("norm_conv: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
                return (int)e;
            }
            attr_set = true;
        }
    }
    const dim3 grid((a.S + a.rows_per_wg - 1) / a.rows_per_wg, B);
    norm_conv_kernel<T, P, false><<<grid, dim3(256), lds, s>>>(a);
    if (a.conv && a.S > 1 && a.taps > 1) {
        const int tail = a.S < a.taps - 1 ? a.S : a.taps - 1;
        norm_conv_kernel<T, P, true><<<dim3(tail, B), dim3(256), 0, s>>>(a);
    }
    return raven_host::check_launch("norm_conv");
}

}  // namespace raven

extern "C" int raven_norm_conv(const float* x, const float* weight, const float* conv, float* ring, void* y, int32_t B, int32_t S, int32_t dim,
                               int32_t ld, int32_t taps, float eps, int32_t pos0, const int32_t* pos_dev, int32_t dtype, void* stream) {
    using namespace raven;
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "norm_conv: unknown dtype %d", dtype);
    RAVEN_REQUIRE(B >= 0 && B <= 65535 && S >= 0 && dim > 0 && ld >= dim && ld % 8 == 0 && ld <= 16384 && pos0 >= 0,
                  "norm_conv: bad shape B=%d S=%d dim=%d ld=%d pos0=%d", B, S, dim, ld, pos0);
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(x && weight && y, "norm_conv: null pointer");
    if (conv) {
        RAVEN_REQUIRE(ring && taps >= 1 && (size_t)taps * ld * sizeof(float) <= 156 * 1024, "norm_conv: %d taps of %d channels do not fit the LDS window",
                      taps, ld);
    }
    NormConvArgs a{};
    a.x = x; a.w = weight; a.conv = conv; a.ring = ring; a.y = y;
    a.S = S; a.dim = dim; a.ld = ld; a.taps = conv ? taps : 1; a.pos0 = pos0; a.pos_dev = pos_dev; a.eps = eps;
    // with a convolution every tile repeats taps - 1 rows of the one before: longer tiles once there are rows to fill the chip
    a.rows_per_wg = !conv ? 1 : (int64_t)B * S >= 16384 ? 16 : (int64_t)B * S >= 2048 ? 8 : 4;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const int p = (ld / 4 + 255) / 256;
#define RAVEN_NORM_CONV(P) return dtype == RAVEN_BF16 ? launch_norm_conv<bf16, P>(a, B, s) : launch_norm_conv<float, P>(a, B, s)
    if (p <= 1) RAVEN_NORM_CONV(1);
    if (p <= 2) RAVEN_NORM_CONV(2);
    if (p <= 4) RAVEN_NORM_CONV(4);
    if (p <= 8) RAVEN_NORM_CONV(8);
    RAVEN_NORM_CONV(16);
#undef RAVEN_NORM_CONV
}

extern "C" int raven_embed_stream(const void* table, const int64_t* ids, float* x, void* x_rounded, int32_t M, int32_t ld, int64_t vocab,
                                  float scale, int32_t dtype, void* stream) {
    using namespace raven;
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "embed_stream: unknown dtype %d", dtype);
    RAVEN_REQUIRE(M >= 0 && ld > 0 && ld % 8 == 0 && vocab > 0, "embed_stream: bad shape M=%d ld=%d", M, ld);
    if (M == 0) return 0;
    RAVEN_REQUIRE(table && ids && x, "embed_stream: null pointer");
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == RAVEN_BF16) embed_stream_kernel<bf16><<<dim3(M), dim3(256), 0, s>>>((const bf16*)table, ids, x, (bf16*)x_rounded, ld, vocab, scale);
    else embed_stream_kernel<float><<<dim3(M), dim3(256), 0, s>>>((const float*)table, ids, x, (float*)x_rounded, ld, vocab, scale);
    return raven_host::check_launch("embed_stream");
}

extern "C" int raven_round_rows(const float* x, void* y, int64_t n, int32_t dtype, void* stream) {
    using namespace raven;
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "round_rows: unknown dtype %d", dtype);
    RAVEN_REQUIRE(n >= 0 && n % 4 == 0 && n / 1024 < 0x7fffffff, "round_rows: bad element count %lld", (long long)n);
    if (n == 0) return 0;
    RAVEN_REQUIRE(x && y, "round_rows: null pointer");
    const dim3 grid((unsigned)((n / 4 + 255) / 256));
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == RAVEN_BF16) round_rows_kernel<bf16><<<grid, dim3(256), 0, s>>>(x, (bf16*)y, n / 4);
    else round_rows_kernel<float><<<grid, dim3(256), 0, s>>>(x, (float*)y, n / 4);
    return raven_host::check_launch("round_rows");
}
