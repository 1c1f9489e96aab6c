// Real-gated linear recurrent unit behind a causal convolution per channel (raven_rglru_forward):
//     u_t = T(bias + sum_j conv[j] x_(t - taps + 1 + j)),   r = sigmoid(W_r u + b_r),   i = sigmoid(W_i u + b_i)
//     log a = -8 r softplus(lam),   S_t = a S_(t-1) + sqrt(1 - a^2) i u,   y = T(S gelu(v))
//
// One token per sequence: rglru_step_kernel does everything in one launch.  A chunk: the convolution, then the gates (both matrices of a
// block against the same rows; on the matrix cores for bf16 chunks) which leave log a and the input term in fp32, then the
// recurrence in pieces of kPiece tokens -- each piece alone gives its decay and what it adds, a short walk over the pieces gives
// the state each starts from, and a second pass over the tokens forms the outputs.
//
// The rows x of the last taps - 1 tokens live in a ring of `taps` fp32 rows, position p in row p mod taps, written by the last launch of a
// call, when every reader of the old rows is done.

#include "row_helpers.h"

namespace raven {

constexpr int kPiece = 32;

struct RglruArgs {
    const float *conv, *conv_bias, *gate_bias, *softplus;
    const void* gates;      // [blocks, 2, bl, bl] of T
    const void* z;          // [M, 2 W] of T: v | x
    float *ring, *state;    // [B, taps, W], [B, W]
    void *u, *y;            // [M, W] of T
    float *la, *in;         // [M, W]: log a, sqrt(1 - a^2) i u
    float *sum, *end, *carry;  // [B, pieces, W]: log of a piece's decay, what it adds, the state it starts from
    int M, S, W, bl, blocks, taps, pos0, pieces, parts;
    const int* pos_dev;
};

__device__ __forceinline__ float gelu_tanh_f32(float z) {
    // 1 + tanh(x) = 2 / (1 + exp(-2 x))
    const float x = 0.79788456080286536f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * x));
}

// log a and the input term of one channel from the gates' sums.  float: the library's functions.  bf16 operands: hardware exp2 and
// reciprocal (1 ulp), and 1 - exp(-t) by its series where the subtraction would lose digits (the first term left out is 1.5e-7 of the sum).
template <typename T>
__device__ __forceinline__ void gate_terms(float zr, float zi, float softplus, float u, float* la, float* in) {
    if constexpr (sizeof(T) == 4) {
        *la = -8.0f * sigmoid_f32(zr) * softplus;
        *in = sqrtf(-expm1f(2.0f * *la)) * sigmoid_f32(zi) * u;
    } else {
        const float log2e = 1.4426950408889634f;
        const float r = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-log2e * zr)), i = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-log2e * zi));
        const float t = 16.0f * r * softplus;
        const float series = t * (1.0f + t * (-0.5f + t * (1.f / 6.f + t * (-1.f / 24.f + t * (1.f / 120.f - t * (1.f / 720.f))))));
        const float gain2 = t < 0.3f ? series : 1.0f - __builtin_amdgcn_exp2f(-log2e * t);
        *la = -0.5f * t;
        *in = __builtin_amdgcn_sqrtf(gain2) * i * u;
    }
}

// x of channel group c (4 channels) at position pos0 + s, s < 0: from the ring
template <typename T>
__device__ __forceinline__ f32x4 past_x(const RglruArgs& a, int b, int pos0, int s, int c) {
    if (s >= 0) return load4(static_cast<const T*>(a.z) + ((int64_t)b * a.S + s) * 2 * a.W + a.W + 4 * c);
    const int p = pos0 + s;
    if (p < 0) return f32x4{0.f, 0.f, 0.f, 0.f};
    return load4(a.ring + ((int64_t)b * a.taps + p % a.taps) * a.W + 4 * c);
}
template <typename T>
__device__ __forceinline__ f32x4 conv_at(const RglruArgs& a, int b, int pos0, int s, int c) {
    f32x4 o = load4(a.conv_bias + 4 * c);
    for (int t = 0; t < a.taps; ++t) o += load4(a.conv + (int64_t)t * a.W + 4 * c) * past_x<T>(a, b, pos0, s - a.taps + 1 + t, c);
    return o;
}

// kConvRows rows and 4 channels per thread
constexpr int kConvRows = 8;
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void rglru_conv_kernel(RglruArgs a) {
    const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, s0 = blockIdx.y * kConvRows;
    if (c >= a.W / 4) return;
    const int pos0 = a.pos_dev ? *a.pos_dev : a.pos0;
    T* u = static_cast<T*>(a.u) + (int64_t)b * a.S * a.W + 4 * c;
    if constexpr (TAPS == 0) {  // any number of taps
        for (int s = s0; s < min(s0 + kConvRows, a.S); ++s) store4(u + (int64_t)s * a.W, conv_at<T>(a, b, pos0, s, c));
    } else {
        f32x4 x[kConvRows + TAPS - 1], w[TAPS];
        const f32x4 bias = load4(a.conv_bias + 4 * c);
#pragma unroll
        for (int t = 0; t < TAPS; ++t) w[t] = load4(a.conv + (int64_t)t * a.W + 4 * c);
#pragma unroll
        for (int i = 0; i < kConvRows + TAPS - 1; ++i) x[i] = past_x<T>(a, b, pos0, min(s0 - TAPS + 1 + i, a.S - 1), c);
#pragma unroll
        for (int i = 0; i < kConvRows; ++i) {
            f32x4 o = bias;
#pragma unroll
            for (int t = 0; t < TAPS; ++t) o += w[t] * x[i + t];
            if (s0 + i < a.S) store4(u + (int64_t)(s0 + i) * a.W, o);
        }
    }
}

// Gates of RB rows and 16 channels of a block on the vector units: 16 lanes to a channel
template <typename T, int RB>
__global__ __launch_bounds__(256) void rglru_gates_kernel(RglruArgs a) {
    constexpr int E = Chunk<T>::N;
    extern __shared__ __align__(16) unsigned char smem_raw[];
    T* xs = reinterpret_cast<T*>(smem_raw);  // [RB][bl]
    const int blk = blockIdx.x / a.parts, part = blockIdx.x % a.parts, m0 = blockIdx.y * RB, nc = a.bl / E;
    for (int i = threadIdx.x; i < RB * nc; i += 256) {
        const int b = i / nc, c = i % nc;
        store_chunk(xs + b * a.bl + c * E, m0 + b < a.M ? load_chunk(static_cast<const T*>(a.u) + (int64_t)(m0 + b) * a.W + blk * a.bl + c * E) : zero_chunk<T>());
    }
    __syncthreads();
    const int r = part * 16 + (threadIdx.x >> 4), c16 = threadIdx.x & 15, rr = min(r, a.bl - 1), ch = blk * a.bl + rr;
    const T* wr = static_cast<const T*>(a.gates) + ((int64_t)blk * 2 * a.bl + rr) * a.bl;
    const T* wi = wr + (int64_t)a.bl * a.bl;
    float zr[RB], zi[RB];
#pragma unroll
    for (int b = 0; b < RB; ++b) zr[b] = zi[b] = 0.f;
    for (int c = c16; c < nc; c += 16) {
        const Chunk<T> vr = load_chunk(wr + c * E), vi = load_chunk(wi + c * E);
#pragma unroll
        for (int b = 0; b < RB; ++b) {
            const Chunk<T> x = load_chunk(xs + b * a.bl + c * E);
            zr[b] = dot_chunk(vr, x, zr[b]);
            zi[b] = dot_chunk(vi, x, zi[b]);
        }
    }
#pragma unroll
    for (int b = 0; b < RB; ++b) {
        const float sr = row16_sum(zr[b]), si = row16_sum(zi[b]);
        if (c16 != 0 || r >= a.bl || m0 + b >= a.M) continue;
        const int64_t at = (int64_t)(m0 + b) * a.W + ch;
        gate_terms<T>(sr + a.gate_bias[ch], si + a.gate_bias[a.W + ch], a.softplus[ch], to_f32(xs[b * a.bl + rr]), a.la + at, a.in + at);
    }
}

// bf16 chunks: 128 token rows x 32 channels of a block per workgroup (32 rows of W_r and the 32 of W_i: a lane that ends up with
// a channel's r has its i too).  A wave owns 32 token rows; the matrices' rows are staged through LDS once per workgroup, 128 columns
// at a time, the token rows come straight from global memory, requested one step ahead.
__global__ __launch_bounds__(256) void rglru_gates_mfma_kernel(RglruArgs a) {
    typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
    constexpr int KC = 128, PITCH = KC + 8;
    __shared__ __align__(16) bf16 ws[64][PITCH];  // W_r rows c0 .. +31, W_i rows c0 .. +31
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, q4 = lane >> 4;
    const int blk = blockIdx.x / a.parts, c0 = (blockIdx.x % a.parts) * 32, m0 = blockIdx.y * 128 + wave * 32;
    const bf16* W = static_cast<const bf16*>(a.gates) + (int64_t)blk * 2 * a.bl * a.bl;
    const u32x4 zero = {0, 0, 0, 0};
    const bf16* u[2];
#pragma unroll
    for (int r = 0; r < 2; ++r) u[r] = static_cast<const bf16*>(a.u) + (int64_t)min(m0 + 16 * r + l16, a.M - 1) * a.W + blk * a.bl;
    f32x4 acc[2][4];
#pragma unroll
    for (int r = 0; r < 2; ++r)
#pragma unroll
        for (int t = 0; t < 4; ++t) acc[r][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.bl; k0 += KC) {
        u32x4 x[2][KC / 32];
#pragma unroll
        for (int r = 0; r < 2; ++r)
#pragma unroll
            for (int j = 0; j < KC / 32; ++j) {
                const int d = k0 + 32 * j + 8 * q4;
                x[r][j] = *reinterpret_cast<const u32x4*>(u[r] + (d < a.bl ? d : 0));
                if (d >= a.bl) x[r][j] = zero;
            }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 64 * (KC / 8) / 256; ++i) {
            const int p = threadIdx.x + 256 * i, row = p / (KC / 8), d = k0 + (p % (KC / 8)) * 8;
            const bf16* src = W + ((int64_t)(row >> 5) * a.bl + min(c0 + (row & 31), a.bl - 1)) * a.bl;
            const u32x4 v = *reinterpret_cast<const u32x4*>(src + (d < a.bl ? d : 0));
            *reinterpret_cast<u32x4*>(&ws[row][(p % (KC / 8)) * 8]) = d < a.bl ? v : zero;
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < KC / 32; ++j)
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const bf16x8 wf = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(&ws[16 * t + l16][32 * j + 8 * q4]));
#pragma unroll
                for (int r = 0; r < 2; ++r) {
                    const u32x4 xv = x[r][j];
                    acc[r][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf, __builtin_bit_cast(bf16x8, xv), acc[r][t], 0, 0, 0);
                }
            }
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        const int c = c0 + 16 * t + 4 * q4;  // four channels; bl is a multiple of 8
        if (c >= a.bl) continue;
        const int ch = blk * a.bl + c;
        const f32x4 br = load4(a.gate_bias + ch), bi = load4(a.gate_bias + a.W + ch), sp = load4(a.softplus + ch);
#pragma unroll
        for (int r = 0; r < 2; ++r) {
            const int m = m0 + 16 * r + l16;
            if (m >= a.M) continue;
            const f32x4 uu = load4(static_cast<const bf16*>(a.u) + (int64_t)m * a.W + ch);
            f32x4 la, in;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                float x, y;
                gate_terms<bf16>(acc[r][t][i] + br[i], acc[r][2 + t][i] + bi[i], sp[i], uu[i], &x, &y);
                la[i] = x;
                in[i] = y;
            }
            store4(a.la + (int64_t)m * a.W + ch, la);
            store4(a.in + (int64_t)m * a.W + ch, in);
        }
    }
}

// a piece alone: its decay and what it adds to a state
__global__ __launch_bounds__(256) void rglru_piece_kernel(RglruArgs a) {
    const int ch = blockIdx.x * 256 + threadIdx.x, piece = blockIdx.y, b = blockIdx.z;
    if (ch >= a.W) return;
    const int64_t row = (int64_t)b * a.S + piece * kPiece;
    float sum = 0.f, end = 0.f;
#pragma unroll 8
    for (int t = 0; t < kPiece; ++t) {  // only whole pieces come here: the last one's sums are not used
        const int64_t at = (row + t) * a.W + ch;
        const float la = a.la[at];
        sum += la;
        end = expf(la) * end + a.in[at];
    }
    const int64_t o = ((int64_t)b * a.pieces + piece) * a.W + ch;
    a.sum[o] = sum;
    a.end[o] = end;
}
__global__ __launch_bounds__(64) void rglru_carry_kernel(RglruArgs a) {
    const int ch = blockIdx.x * 64 + threadIdx.x, b = blockIdx.y;
    if (ch >= a.W) return;
    const int pos0 = a.pos_dev ? *a.pos_dev : a.pos0;
    float S = pos0 > 0 ? a.state[(int64_t)b * a.W + ch] : 0.f;
    const int64_t base = (int64_t)b * a.pieces * a.W + ch;
    constexpr int U = 32;
    for (int p0 = 0; p0 < a.pieces; p0 += U) {
        float sum[U], end[U];
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int64_t at = base + (int64_t)min(p0 + i, max(a.pieces - 2, 0)) * a.W;
            sum[i] = a.sum[at];
            end[i] = a.end[at];
        }
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (p0 + i >= a.pieces) break;
            a.carry[base + (int64_t)(p0 + i) * a.W] = S;
            S = expf(sum[i]) * S + end[i];
        }
    }
}
template <typename T>
__global__ __launch_bounds__(256) void rglru_finish_kernel(RglruArgs a) {
    const int ch = blockIdx.x * 256 + threadIdx.x, piece = blockIdx.y, b = blockIdx.z;
    if (ch >= a.W) return;
    const int pos0 = a.pos_dev ? *a.pos_dev : a.pos0;
    float S = a.pieces > 1 ? a.carry[((int64_t)b * a.pieces + piece) * a.W + ch] : pos0 > 0 ? a.state[(int64_t)b * a.W + ch] : 0.f;
    const int s0 = piece * kPiece, s1 = min(s0 + kPiece, a.S);
    const T* z = static_cast<const T*>(a.z);
#pragma unroll 4
    for (int s = s0; s < s1; ++s) {
        const int64_t m = (int64_t)b * a.S + s, at = m * a.W + ch;
        S = expf(a.la[at]) * S + a.in[at];
        static_cast<T*>(a.y)[at] = from_f32<T>(S * gelu_tanh_f32(to_f32(z[m * 2 * a.W + ch])));
        if (s >= a.S - (a.taps - 1)) a.ring[((int64_t)b * a.taps + (pos0 + s) % a.taps) * a.W + ch] = to_f32(z[m * 2 * a.W + a.W + ch]);
    }
    if (s1 == a.S) a.state[(int64_t)b * a.W + ch] = S;
}

// One token per sequence: 16 channels of a block per workgroup.  The block's convolution is formed by every workgroup of the block
// (a few KB), then 16 lanes per channel multiply both matrices' rows.
template <typename T>
__global__ __launch_bounds__(256) void rglru_step_kernel(RglruArgs a) {
    constexpr int E = Chunk<T>::N;
    extern __shared__ __align__(16) unsigned char smem_raw[];
    T* xs = reinterpret_cast<T*>(smem_raw);  // [bl]
    const int blk = blockIdx.x / a.parts, part = blockIdx.x % a.parts, b = blockIdx.y, nc = a.bl / E;
    const int pos = a.pos_dev ? *a.pos_dev : a.pos0;
    const int r = part * 16 + (threadIdx.x >> 4), c16 = threadIdx.x & 15, rr = min(r, a.bl - 1), ch = blk * a.bl + rr;
    const T* wr = static_cast<const T*>(a.gates) + ((int64_t)blk * 2 * a.bl + rr) * a.bl;
    const T* wi = wr + (int64_t)a.bl * a.bl;
    // the first pieces of the matrices are requested before the convolution's inputs are waited for
    Chunk<T> vr[2], vi[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int c = min(c16 + 16 * j, nc - 1);
        vr[j] = load_chunk(wr + c * E);
        vi[j] = load_chunk(wi + c * E);
    }
    for (int c = threadIdx.x; c < a.bl / 4; c += 256) store4(xs + 4 * c, conv_at<T>(a, b, pos, 0, blk * (a.bl / 4) + c));
    const float old = pos > 0 ? a.state[(int64_t)b * a.W + ch] : 0.f;
    const T* z = static_cast<const T*>(a.z) + (int64_t)b * 2 * a.W;
    const float v = to_f32(z[ch]), x = to_f32(z[a.W + ch]);
    __syncthreads();
    float zr = 0.f, zi = 0.f;
    for (int c0 = 0; c0 < nc; c0 += 32) {
        if (c0 > 0) {
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const int c = min(c0 + c16 + 16 * j, nc - 1);
                vr[j] = load_chunk(wr + c * E);
                vi[j] = load_chunk(wi + c * E);
            }
        }
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int c = c0 + c16 + 16 * j;
            if (c < nc) {
                const Chunk<T> xc = load_chunk(xs + c * E);
                zr = dot_chunk(vr[j], xc, zr);
                zi = dot_chunk(vi[j], xc, zi);
            }
        }
    }
    zr = row16_sum(zr);
    zi = row16_sum(zi);
    if (c16 != 0 || r >= a.bl) return;
    float la, in;
    gate_terms<T>(zr + a.gate_bias[ch], zi + a.gate_bias[a.W + ch], a.softplus[ch], to_f32(xs[rr]), &la, &in);
    const float S = expf(la) * old + in;
    a.state[(int64_t)b * a.W + ch] = S;
    a.ring[((int64_t)b * a.taps + pos % a.taps) * a.W + ch] = x;  // not one of the rows the convolution reads
    static_cast<T*>(a.y)[(int64_t)b * a.W + ch] = from_f32<T>(S * gelu_tanh_f32(v));
}

static size_t carve_rglru(const raven_rglru* l, int B, int S, int dtype, char* base, RglruArgs* a) {
    if (S == 1) return 0;
    const size_t M = (size_t)B * S, W = l->width, pieces = (S + kPiece - 1) / kPiece;
    size_t off = 0;
    auto take = [&](size_t bytes) {
        char* p = base ? base + off : nullptr;
        off += raven_host::align_up(bytes);
        return p;
    };
    char* u = take(M * W * raven_host::elt_size(dtype));
    float* f[5];
    for (int i = 0; i < 5; ++i) f[i] = reinterpret_cast<float*>(take((i < 2 ? M : B * pieces) * W * sizeof(float)));
    if (a) {
        a->u = u;
        a->la = f[0]; a->in = f[1]; a->sum = f[2]; a->end = f[3]; a->carry = f[4];
        a->pieces = (int)pieces;
    }
    return off;
}

template <typename T>
static int run_rglru(RglruArgs a, int B, hipStream_t s) {
    const size_t lds = (size_t)a.bl * sizeof(T);
    if (a.S == 1) {
        a.parts = (a.bl + 15) / 16;
        rglru_step_kernel<T><<<dim3(a.blocks * a.parts, B), dim3(256), lds, s>>>(a);
        return raven_host::check_launch("rglru (step)");
    }
    const dim3 conv_grid((a.W / 4 + 255) / 256, (a.S + kConvRows - 1) / kConvRows, B);
    if (a.taps == 4) rglru_conv_kernel<T, 4><<<conv_grid, dim3(256), 0, s>>>(a);
    else rglru_conv_kernel<T, 0><<<conv_grid, dim3(256), 0, s>>>(a);
    bool done = false;
    if constexpr (sizeof(T) == 2) {
        if (a.M >= 16) {
            a.parts = (a.bl + 31) / 32;
            rglru_gates_mfma_kernel<<<dim3(a.blocks * a.parts, (a.M + 127) / 128), dim3(256), 0, s>>>(a);
            done = true;
        }
    }
    if (!done) {
        a.parts = (a.bl + 15) / 16;
        rglru_gates_kernel<T, 4><<<dim3(a.blocks * a.parts, (a.M + 3) / 4), dim3(256), 4 * lds, s>>>(a);
    }
    const dim3 grid((a.W + 255) / 256, a.pieces, B);
    if (a.pieces > 1) {
        rglru_piece_kernel<<<dim3(grid.x, a.pieces - 1, B), dim3(256), 0, s>>>(a);
        rglru_carry_kernel<<<dim3((a.W + 63) / 64, B), dim3(64), 0, s>>>(a);
    }
    rglru_finish_kernel<T><<<grid, dim3(256), 0, s>>>(a);
    return raven_host::check_launch("rglru");
}

static int check_rglru(const char* who, const raven_rglru* l, int B, int S, int dtype) {
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "%s: unknown dtype %d", who, dtype);
    RAVEN_REQUIRE(l && l->blocks > 0 && l->block_ld > 0 && l->block_ld % 8 == 0 && l->block_ld <= 8192 && l->width == l->blocks * l->block_ld && l->taps >= 1,
                  "%s: bad sizes", who);
    RAVEN_REQUIRE(B >= 0 && B <= 65535 && S >= 0 && (int64_t)B * S <= 65535 * 4, "%s: bad B=%d S=%d", who, B, S);
    return 0;
}

}  // namespace raven

extern "C" size_t raven_rglru_workspace_bytes(const raven_rglru* l, int32_t B, int32_t S, int32_t dtype) {
    if (raven::check_rglru("rglru_workspace_bytes", l, B, S, dtype) || B == 0 || S == 0) return 0;
    return raven::carve_rglru(l, B, S, dtype, nullptr, nullptr);
}

extern "C" int raven_rglru_forward(const raven_rglru* l, const void* z, float* ring, float* state, void* y, int32_t B, int32_t S, int32_t pos0,
                                   const int32_t* pos_dev, int32_t dtype, void* workspace, size_t workspace_bytes, void* stream) {
    using namespace raven;
    if (const int rc = check_rglru("rglru", l, B, S, dtype)) return rc;
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(l->conv && l->conv_bias && l->gates && l->gate_bias && l->softplus && z && ring && state && y && pos0 >= 0, "rglru: null pointer");
    const size_t need = carve_rglru(l, B, S, dtype, nullptr, nullptr);
    RAVEN_REQUIRE(need == 0 || (workspace && ((uintptr_t)workspace & 255) == 0 && need <= workspace_bytes), "rglru: workspace of %zu bytes is too small or unaligned",
                  workspace_bytes);
    RglruArgs a{};
    carve_rglru(l, B, S, dtype, static_cast<char*>(workspace), &a);
    a.conv = l->conv; a.conv_bias = l->conv_bias; a.gate_bias = l->gate_bias; a.softplus = l->softplus; a.gates = l->gates;
    a.z = z; a.ring = ring; a.state = state; a.y = y;
    a.M = B * S; a.S = S; a.W = l->width; a.bl = l->block_ld; a.blocks = l->blocks; a.taps = l->taps; a.pos0 = pos0; a.pos_dev = pos_dev;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == RAVEN_BF16 ? run_rglru<bf16>(a, B, s) : run_rglru<float>(a, B, s);
}
