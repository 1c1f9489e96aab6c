// Attention over a cache of low-rank rows: a position leaves one normed latent c [kp] and one rotated key part [rp] for all heads.
//     s_ij = scale (q_n . W_uk c_j + q_r . k_r,j),  0 <= i - j < window;   y = T( (softmax . W_uv c) * sigmoid(gate) )
//
// Two ways to the same numbers:
//   expanded  a chunk multiplies the visible latents by [W_uk; W_uv] once (a plain product over the cache's own rows) and attends to
//             keys of nope + rp and values of vp channels: latent_prefill_kernel, on the matrix cores;
//   absorbed  few rows take W_uk over to the query, q' = W_uk^T q_n [kp], attend to the latents themselves -- one row of kp + rp
//             elements per position whatever the number of heads -- and apply W_uv to the weighted sum of latents:
//             absorb_kernel, latent_rows_attention_kernel (vector units) or latent_step_kernel (matrix cores), latent_out_kernel.
//
// The two halves of a rotation are stored side by side, so a rotation is private to a lane (rope_pair).

#include <math.h>

#include "row_helpers.h"

namespace raven {

struct LatentArgs {
    const void* q;        // [M, H * (np + rp)] of T, not rotated
    const void* z;        // [M, ldz] of Z
    void* latent;         // [batch, t_max, kp] of T
    void* rotated;        // [batch, t_max, rp] of T
    const float* angles;  // [t_max, rp]: (cos, sin) pairs
    const void* w_uk_t;   // [H, kp, np]
    const void* w_uv;     // [H * vp, kp]
    const float *q_norm, *kv_norm;
    void *cq, *qa, *y;    // [M, qp], [M, H, kp + rp], [M, H * vp]
    float* part;          // [M, H, splits, kp + 4]: weighted latents, then reference and sum
    const void* kv;       // expanded: [B, n_rows, H * np + H * vp], row 0 = position k0
    int H, qd, qp, kd, kp, np, rp, vp, window, ldz, z_kv, z_gate;  // z_kv / z_gate: column of the key latent / the gate
    int M, S, pos0, t_max, splits, append, rows_out, k0, n_rows, per_wg;
    const int* pos_dev;
    float scale, eps;
};

// one wave: the cache entry of row m
template <typename T, typename Z>
__device__ __forceinline__ void append_row(const LatentArgs& a, int m) {
    const int b = m / a.S, pos = (a.pos_dev ? *a.pos_dev : a.pos0) + m % a.S;
    if (pos >= a.t_max) return;
    const Z* z = static_cast<const Z*>(a.z) + (int64_t)m * a.ldz + a.z_kv;
    const int64_t at = (int64_t)b * a.t_max + pos;
    wave_norm<T, Z>(z, a.kv_norm, static_cast<T*>(a.latent) + at * a.kp, a.kp, a.kd, a.eps);
    for (int i = 4 * (threadIdx.x & 63); i < a.rp; i += 256) {
        const f32x4 v = load4(z + a.kp + i), cs = load4(a.angles + (int64_t)pos * a.rp + i);
        T x[4] = {from_f32<T>(v[0]), from_f32<T>(v[1]), from_f32<T>(v[2]), from_f32<T>(v[3])};
        if constexpr (sizeof(Z) == 4 && sizeof(T) == 2) {  // float rows: rotate before the one rounding
            x[0] = from_f32<T>(v[0] * cs[0] - v[1] * cs[1]);
            x[1] = from_f32<T>(v[1] * cs[0] + v[0] * cs[1]);
            x[2] = from_f32<T>(v[2] * cs[2] - v[3] * cs[3]);
            x[3] = from_f32<T>(v[3] * cs[2] + v[2] * cs[3]);
        } else {
            rope_pair<T>(x[0], x[1], cs[0], cs[1]);
            rope_pair<T>(x[2], x[3], cs[2], cs[3]);
        }
        T* out = static_cast<T*>(a.rotated) + at * a.rp + i;
#pragma unroll
        for (int e = 0; e < 4; ++e) out[e] = x[e];
    }
}

// a wave per row: the normed query latent and the cache entry
template <typename T, typename Z>
__global__ __launch_bounds__(256) void latent_rows_kernel(LatentArgs a) {
    const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (m >= a.M) return;
    if (a.cq) wave_norm<T, Z>(static_cast<const Z*>(a.z) + (int64_t)m * a.ldz, a.q_norm, static_cast<T*>(a.cq) + (int64_t)m * a.qp, a.qp, a.qd, a.eps);
    if (a.append) append_row<T, Z>(a, m);
}

// ------------------------------------------------------------------------------------------------
// Absorbed route
// ------------------------------------------------------------------------------------------------
// q' = [W_uk^T q_n | rotated q_r]; with `append` the last column of workgroups writes the rows' cache entries
template <typename T, typename Z, int RB>
__global__ __launch_bounds__(256) void absorb_kernel(LatentArgs a) {
    constexpr int E = Chunk<T>::N;
    extern __shared__ __align__(16) unsigned char smem_raw[];
    T* xs = reinterpret_cast<T*>(smem_raw);  // [RB][np]
    const int m0 = blockIdx.y * RB;
    if ((int)blockIdx.x == a.H * a.rows_out) {
        for (int b = threadIdx.x >> 6; b < RB && m0 + b < a.M; b += 4) append_row<T, Z>(a, m0 + b);
        return;
    }
    const int h = blockIdx.x / a.rows_out, part = blockIdx.x % a.rows_out;
    const int hd = a.np + a.rp, ld = a.kp + a.rp;
    const T* q = static_cast<const T*>(a.q) + (int64_t)h * hd;
    T* out = static_cast<T*>(a.qa);
    for (int i = threadIdx.x; i < RB * (a.np / E); i += 256) {
        const int b = i / (a.np / E), c = i % (a.np / E);
        store_chunk(xs + b * a.np + c * E, m0 + b < a.M ? load_chunk(q + (int64_t)(m0 + b) * a.H * hd + c * E) : zero_chunk<T>());
    }
    if (part == 0) {
        for (int i = threadIdx.x; i < RB * (a.rp / 2); i += 256) {
            const int b = i / (a.rp / 2), c = 2 * (i % (a.rp / 2)), m = m0 + b;
            if (m >= a.M) continue;
            const int pos = min((a.pos_dev ? *a.pos_dev : a.pos0) + m % a.S, a.t_max - 1);
            const float* cs = a.angles + (int64_t)pos * a.rp + c;
            T x0 = q[(int64_t)m * a.H * hd + a.np + c], x1 = q[(int64_t)m * a.H * hd + a.np + c + 1];
            rope_pair<T>(x0, x1, cs[0], cs[1]);
            T* o = out + ((int64_t)m * a.H + h) * ld + a.kp + c;
            o[0] = x0;
            o[1] = x1;
        }
    }
    __syncthreads();
    head_product<T, RB>(static_cast<const T*>(a.w_uk_t) + (int64_t)h * a.kp * a.np, xs, a.np, a.kp, part * 16 * a.per_wg, a.per_wg,
                        [&](int r, int b, float s) {
                            if (m0 + b < a.M) out[((int64_t)(m0 + b) * a.H + h) * ld + r] = from_f32<T>(s);
                        });
}

// Ranges merged, W_uv, gate: y = T( (W_uv o) * sigmoid(gate) )
template <typename T, typename Z, int RB>
__global__ __launch_bounds__(256) void latent_out_kernel(LatentArgs a) {
    extern __shared__ __align__(16) unsigned char smem_raw[];
    T* xs = reinterpret_cast<T*>(smem_raw);  // [RB][kp]
    const int h = blockIdx.x / a.rows_out, part = blockIdx.x % a.rows_out, m0 = blockIdx.y * RB;
    const int ld = a.kp + 4;
    {
        // RB 4: a wave per row; RB 1: the four waves share the row's columns
        static_assert(RB == 1 || RB == 4, "rows per workgroup");
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, b = RB == 4 ? wave : 0;
        const int m = min(m0 + b, a.M - 1);
        const float* p = a.part + ((int64_t)m * a.H + h) * a.splits * ld;
        // lane n holds range n (at most 64); some range always holds a position
        const int mine = min(lane, a.splits - 1);
        const float ref = p[(int64_t)mine * ld + a.kp], sum = p[(int64_t)mine * ld + a.kp + 1];
        const float top = wave_max(ref);
        const float w = lane < a.splits ? soft_exp<T>(ref - top) : 0.f;
        const float f = w / wave_sum(w * sum);
        constexpr int STEP = RB == 4 ? 256 : 1024;
        for (int i0 = 0; i0 < a.kp; i0 += STEP) {  // uniform trip count: every lane takes part in the exchanges
            const int i = i0 + 4 * (RB == 4 ? lane : (int)threadIdx.x);
            const int at = min(i, a.kp - 4);
            f32x4 o = {0.f, 0.f, 0.f, 0.f};
            for (int s0 = 0; s0 < a.splits; s0 += 8) {
                f32x4 x[8];
#pragma unroll
                for (int s = 0; s < 8; ++s) x[s] = load4(p + (int64_t)min(s0 + s, a.splits - 1) * ld + at);
#pragma unroll
                for (int s = 0; s < 8; ++s) o += x[s] * __shfl(f, (s0 + s) & 63, 64);  // ranges past the last: factor 0
            }
            if (i < a.kp) store4(xs + b * a.kp + i, o);
        }
    }
    __syncthreads();
    const Z* z = static_cast<const Z*>(a.z);
    head_product<T, RB>(static_cast<const T*>(a.w_uv) + (int64_t)h * a.vp * a.kp, xs, a.kp, a.vp, part * 16 * a.per_wg, a.per_wg,
                        [&](int r, int b, float s) {
                            const int m = m0 + b;
                            if (m >= a.M) return;
                            const float g = to_f32(z[(int64_t)m * a.ldz + a.z_gate + h * a.vp + r]);
                            static_cast<T*>(a.y)[((int64_t)m * a.H + h) * a.vp + r] = from_f32<T>(s * sigmoid_f32(g));
                        });
}

// The positions [lo, hi) that range `split` of a row at position pos covers
__device__ __forceinline__ void row_range(const LatentArgs& a, int pos, int split, int* lo, int* hi) {
    const int first = a.window > 0 ? max(0, pos - a.window + 1) : 0;
    const int span = (pos + 1 - first + a.splits - 1) / a.splits;
    *lo = first + split * span;
    *hi = min(pos + 1, *lo + span);
}

// One token row, NH heads, one range of positions; each wave walks 16 positions at a time on its own and the four are merged
// at the end.  16 lanes share a position for the scores (a row group of the wave takes 4 of the 16); for the weighted sum a lane owns
// 16-byte pieces of the latent, CJ of them.
template <typename T, int NH, int CJ>
__global__ __launch_bounds__(256) void latent_rows_attention_kernel(LatentArgs a) {
    constexpr int E = Chunk<T>::N;
    extern __shared__ __align__(16) unsigned char smem_raw[];
    const int ld = a.kp + a.rp, nk = a.kp / E, nc = ld / E;
    T* qs = reinterpret_cast<T*>(smem_raw);                                             // [NH][ld]
    float* merge = reinterpret_cast<float*>(smem_raw + (((size_t)NH * ld * sizeof(T) + 15) & ~(size_t)15));  // [4][NH][kp]
    __shared__ float sm[4][NH], sl[4][NH];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c16 = lane & 15, grp = lane >> 4;
    const int h0 = blockIdx.y * NH, m = blockIdx.z, b = m / a.S;
    const int pos = (a.pos_dev ? *a.pos_dev : a.pos0) + m % a.S;
    int lo, hi;
    row_range(a, min(pos, a.t_max - 1), blockIdx.x, &lo, &hi);
    const T* qa = static_cast<const T*>(a.qa) + (int64_t)m * a.H * ld;
    for (int i = threadIdx.x; i < NH * nc; i += 256) {
        const int n = i / nc, c = i % nc;
        store_chunk(qs + n * ld + c * E, load_chunk(qa + (int64_t)min(h0 + n, a.H - 1) * ld + c * E));
    }
    __syncthreads();
    const T* lat = static_cast<const T*>(a.latent) + (int64_t)b * a.t_max * a.kp;
    const T* rot = static_cast<const T*>(a.rotated) + (int64_t)b * a.t_max * a.rp;
    float mx[NH], l[NH], acc[NH][CJ][E];
#pragma unroll
    for (int n = 0; n < NH; ++n) {
        mx[n] = -INFINITY;
        l[n] = 0.f;
#pragma unroll
        for (int j = 0; j < CJ; ++j)
#pragma unroll
            for (int e = 0; e < E; ++e) acc[n][j][e] = 0.f;
    }
    for (int p0 = lo + 16 * wave; p0 < hi; p0 += 64) {
        float sc[4][NH];  // position p0 + 4 u + grp
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int n = 0; n < NH; ++n) sc[u][n] = 0.f;
        for (int c = c16; c < nc; c += 16) {
            Chunk<T> k[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int64_t p = min(p0 + 4 * u + grp, hi - 1);
                k[u] = load_chunk(c < nk ? lat + p * a.kp + c * E : rot + p * a.rp + (c - nk) * E);
            }
#pragma unroll
            for (int n = 0; n < NH; ++n) {
                const Chunk<T> q = load_chunk(qs + n * ld + c * E);
#pragma unroll
                for (int u = 0; u < 4; ++u) sc[u][n] = dot_chunk(k[u], q, sc[u][n]);
            }
        }
#pragma unroll
        for (int n = 0; n < NH; ++n) {
            float top = mx[n];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const float s = row16_sum(sc[u][n]) * a.scale;
                sc[u][n] = p0 + 4 * u + grp < hi ? s : -INFINITY;
                top = fmaxf(top, sc[u][n]);
            }
            top = fmaxf(top, __shfl_xor(top, 16, 64));
            top = fmaxf(top, __shfl_xor(top, 32, 64));  // finite: position p0 exists
            const float corr = soft_exp<T>(mx[n] - top);
            mx[n] = top;
            float sum = 0.f;
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                sc[u][n] = soft_exp<T>(sc[u][n] - top);
                sum += sc[u][n];
            }
            sum += __shfl_xor(sum, 16, 64);
            sum += __shfl_xor(sum, 32, 64);
            l[n] = l[n] * corr + sum;
#pragma unroll
            for (int j = 0; j < CJ; ++j)
#pragma unroll
                for (int e = 0; e < E; ++e) acc[n][j][e] *= corr;
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const int64_t p = min(p0 + 4 * u + g, hi - 1);
                float w[NH];
#pragma unroll
                for (int n = 0; n < NH; ++n) w[n] = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, sc[u][n]), 16 * g));
#pragma unroll
                for (int j = 0; j < CJ; ++j) {
                    const Chunk<T> v = load_chunk(lat + p * a.kp + min(lane + 64 * j, nk - 1) * E);
#pragma unroll
                    for (int n = 0; n < NH; ++n)
#pragma unroll
                        for (int e = 0; e < E; ++e) acc[n][j][e] = __builtin_fmaf(w[n], to_f32(v.v[e]), acc[n][j][e]);
                }
            }
    }
#pragma unroll
    for (int n = 0; n < NH; ++n) {
        if (lane == 0) {
            sm[wave][n] = mx[n];
            sl[wave][n] = l[n];
        }
#pragma unroll
        for (int j = 0; j < CJ; ++j) {
            if (lane + 64 * j >= nk) continue;
#pragma unroll
            for (int e = 0; e < E; e += 4)
                store4(merge + ((int64_t)wave * NH + n) * a.kp + (lane + 64 * j) * E + e, f32x4{acc[n][j][e], acc[n][j][e + 1], acc[n][j][e + 2], acc[n][j][e + 3]});
        }
    }
    __syncthreads();
    for (int n = 0; n < NH && h0 + n < a.H; ++n) {
        const float top = fmaxf(fmaxf(sm[0][n], sm[1][n]), fmaxf(sm[2][n], sm[3][n]));
        const float ref = top == -INFINITY ? 0.f : top;
        float f[4];
#pragma unroll
        for (int w = 0; w < 4; ++w) f[w] = soft_exp<T>(sm[w][n] - ref);
        float* out = a.part + (((int64_t)m * a.H + h0 + n) * a.splits + blockIdx.x) * (a.kp + 4);
        for (int i = 4 * threadIdx.x; i < a.kp; i += 1024) {
            f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int w = 0; w < 4; ++w) o += load4(merge + ((int64_t)w * NH + n) * a.kp + i) * f[w];
            store4(out + i, o);
        }
        if (threadIdx.x == 0) {
            out[a.kp] = top;
            out[a.kp + 1] = sl[0][n] * f[0] + sl[1][n] * f[1] + sl[2][n] * f[2] + sl[3][n] * f[3];
        }
    }
}

// ------------------------------------------------------------------------------------------------
// The same on the matrix cores (bf16): the query rows are the heads.  A workgroup takes RG groups of 16 of a sequence's S * H rows and
// walks its range in tiles of 64 positions; one staged tile [64][kp + rp] serves both products.  Scores: wave w multiplies positions
// 16 w .. + 15 with every row.  The four exchange their maxima and weights through LDS.  Weighted sum: wave w owns every fourth tile of 16
// latent channels, read through the transposing loads; the weights are picked up in the key order those deliver.
// ------------------------------------------------------------------------------------------------
constexpr int kLsKeys = 64;

template <int KS, int NTW, int RG>
__global__ __launch_bounds__(256) void latent_step_kernel(LatentArgs a) {
    constexpr int PITCH = KS * 32 + 16, CPR = KS * 4, NKC = kLsKeys * CPR / 256, PP = kLsKeys + 8;
    static_assert(kLsKeys * CPR % 256 == 0, "staging shape");
    typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
    typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
    typedef short s16x4 __attribute__((ext_vector_type(4)));
    extern __shared__ __align__(16) unsigned char smem_raw[];
    bf16(*sk)[PITCH] = reinterpret_cast<bf16(*)[PITCH]>(smem_raw);
    __shared__ __align__(16) bf16 sp[16 * RG][PP];
    __shared__ float smx[4][16 * RG];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, q4 = lane >> 4;
    const int b = blockIdx.z, r0 = blockIdx.y * 16 * RG, n_rows = a.S * a.H, ld = a.kp + a.rp;
    const int pos0 = min(a.pos_dev ? *a.pos_dev : a.pos0, a.t_max - a.S);
    const int window = a.window > 0 ? a.window : 0x40000000;
    // the positions that these rows see
    const int first = max(0, pos0 + r0 / a.H - window + 1), end = pos0 + min(r0 + 16 * RG - 1, n_rows - 1) / a.H + 1;
    const int span = (end - first + a.splits - 1) / a.splits;
    const int lo = first + (int)blockIdx.x * span, hi = min(end, lo + span);
    const bf16* lat = static_cast<const bf16*>(a.latent) + (int64_t)b * a.t_max * a.kp;
    const bf16* rot = static_cast<const bf16*>(a.rotated) + (int64_t)b * a.t_max * a.rp;

    u32x4 reg[NKC];
    auto fetch = [&](int kt) {
#pragma unroll
        for (int i = 0; i < NKC; ++i) {
            const int c = threadIdx.x + 256 * i, d = (c % CPR) * 8;
            const int64_t p = min(kt + c / CPR, hi - 1);
            const u32x4 v = *reinterpret_cast<const u32x4*>(d < a.kp ? lat + p * a.kp + d : d < ld ? rot + p * a.rp + (d - a.kp) : lat + p * a.kp);
            reg[i] = d < ld ? v : u32x4{0, 0, 0, 0};
        }
    };
    if (lo < hi) fetch(lo);
    bf16x8 qf[RG][KS];
    int my_pos[RG];
#pragma unroll
    for (int g = 0; g < RG; ++g) {
        const int row = min(r0 + 16 * g + l16, n_rows - 1);
        my_pos[g] = pos0 + row / a.H;
        const bf16* qp = static_cast<const bf16*>(a.qa) + ((int64_t)b * n_rows + row) * ld;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int d = 32 * ks + 8 * q4;
            const u32x4 v = *reinterpret_cast<const u32x4*>(qp + (d < ld ? d : 0));
            qf[g][ks] = __builtin_bit_cast(bf16x8, d < ld ? v : u32x4{0, 0, 0, 0});
        }
    }
    f32x4 o[RG][NTW], osum[RG];
    float ref[RG];
#pragma unroll
    for (int g = 0; g < RG; ++g) {
        ref[g] = -INFINITY;
        osum[g] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int n = 0; n < NTW; ++n) o[g][n] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    bf16x8 ones;
#pragma unroll
    for (int e = 0; e < 8; ++e) ones[e] = static_cast<bf16>(1.0f);
    const float in_scale = a.scale * 1.4426950408889634f;
    const int n_tiles = (a.kp + 15) / 16;

    for (int kt = lo; kt < hi; kt += kLsKeys) {
#pragma unroll
        for (int i = 0; i < NKC; ++i) {
            const int c = threadIdx.x + 256 * i;
            *reinterpret_cast<u32x4*>(&sk[c / CPR][(c % CPR) * 8]) = reg[i];
        }
        __syncthreads();
        if (kt + kLsKeys < hi) fetch(kt + kLsKeys);
        f32x4 sc[RG];
#pragma unroll
        for (int g = 0; g < RG; ++g) sc[g] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const bf16x8 kf = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(&sk[16 * wave + l16][32 * ks + 8 * q4]));
#pragma unroll
            for (int g = 0; g < RG; ++g) sc[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[g][ks], sc[g], 0, 0, 0);
        }
        // lane: positions kt + 16 wave + 4 q4 + (0 .. 3) of row l16
        const int p0 = kt + 16 * wave + 4 * q4;
#pragma unroll
        for (int g = 0; g < RG; ++g) {
            float mx = -INFINITY;
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const bool seen = p0 + v < hi && (unsigned)(my_pos[g] - p0 - v) < (unsigned)window;
                sc[g][v] = seen ? sc[g][v] * in_scale : -INFINITY;
                mx = fmaxf(mx, sc[g][v]);
            }
            mx = max_over_quarters(mx);
            if (q4 == 0) smx[wave][16 * g + l16] = mx;
        }
        __syncthreads();
#pragma unroll
        for (int g = 0; g < RG; ++g) {
            const int r = 16 * g + l16;
            const float top = fmaxf(ref[g], fmaxf(fmaxf(smx[0][r], smx[1][r]), fmaxf(smx[2][r], smx[3][r])));
            const float m = top == -INFINITY ? 0.f : top;
            bf16 w[4];
#pragma unroll
            for (int v = 0; v < 4; ++v) w[v] = from_f32<bf16>(__builtin_amdgcn_exp2f(sc[g][v] - m));
            *reinterpret_cast<u32x2*>(&sp[r][16 * wave + 4 * q4]) = *reinterpret_cast<const u32x2*>(w);
            const float corr = __builtin_amdgcn_exp2f(ref[g] - m);  // 0 while nothing has been seen
            ref[g] = top;
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const float cv = __shfl(corr, 4 * q4 + v, 64);
                osum[g][v] *= cv;
#pragma unroll
                for (int n = 0; n < NTW; ++n) o[g][n][v] *= cv;
            }
        }
        __syncthreads();
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            bf16x8 pf[RG];
#pragma unroll
            for (int g = 0; g < RG; ++g) {  // keys 32 c + 4 q4 + (0 .. 3) and 16 further
                const u32x2 p_lo = *reinterpret_cast<const u32x2*>(&sp[16 * g + l16][32 * c + 4 * q4]);
                const u32x2 p_hi = *reinterpret_cast<const u32x2*>(&sp[16 * g + l16][32 * c + 16 + 4 * q4]);
                const u32x4 both = {p_lo[0], p_lo[1], p_hi[0], p_hi[1]};
                pf[g] = __builtin_bit_cast(bf16x8, both);
                osum[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[g], ones, osum[g], 0, 0, 0);
            }
#pragma unroll
            for (int n = 0; n < NTW; ++n) {
                const int col = 16 * min(wave + 4 * n, n_tiles - 1);
                const bf16* src = &sk[32 * c + 4 * q4 + (l16 >> 2)][col + 4 * (l16 & 3)];
                const s16x4 v_lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3)))*)(src));
                const s16x4 v_hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3)))*)(src + 16 * PITCH));
                const bf16x8 vf = __builtin_bit_cast(bf16x8, __builtin_shufflevector(v_lo, v_hi, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
                for (int g = 0; g < RG; ++g) o[g][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[g], vf, o[g][n], 0, 0, 0);
            }
        }
        __syncthreads();
    }
    // lane: rows 4 q4 + v, channel l16 of each of the wave's tiles
#pragma unroll
    for (int g = 0; g < RG; ++g)
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const int row = r0 + 16 * g + 4 * q4 + v;
            const float m = __shfl(ref[g], 4 * q4 + v, 64);
            if (row >= n_rows) continue;
            float* out = a.part + (((int64_t)b * n_rows + row) * a.splits + blockIdx.x) * (a.kp + 4);
#pragma unroll
            for (int n = 0; n < NTW; ++n) {
                const int col = 16 * (wave + 4 * n) + l16;
                if (col < a.kp) out[col] = o[g][n][v];
            }
            if (wave == 0 && l16 == 0) {
                out[a.kp] = m == -INFINITY ? m : m * 0.69314718055994531f;  // natural units
                out[a.kp + 1] = osum[g][v];
            }
        }
}

template <int KS, int NTW, int RG>
static int launch_step(const LatentArgs& a, hipStream_t s) {
    const size_t lds = (size_t)kLsKeys * (KS * 32 + 16) * sizeof(bf16);
    if (lds > 32 * 1024) {
        static bool attr_set = false;
        if (!attr_set) {
            const hipError_t e = hipFuncSetAttribute((const void*)latent_step_kernel<KS, NTW, RG>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
            if (e != hipSuccess) {
                raven_host::set_error("latent_attention: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
                return (int)e;
            }
            attr_set = true;
        }
    }
    const int groups = (a.S * a.H + 16 * RG - 1) / (16 * RG);
    latent_step_kernel<KS, NTW, RG><<<dim3(a.splits, groups, a.M / a.S), dim3(256), lds, s>>>(a);
    return raven_host::check_launch("latent_attention (step)");
}
// rows of 16 heads per workgroup: 2 once a sequence has more than 16 (head, row) pairs
static bool step_fits(int kp, int rp) { return kp <= 512 && kp + rp <= 576; }
static int run_step(const LatentArgs& a, hipStream_t s) {
    const bool two = a.S * a.H > 16;
    if (a.kp <= 256 && a.kp + a.rp <= 320) return two ? launch_step<10, 4, 2>(a, s) : launch_step<10, 4, 1>(a, s);
    return two ? launch_step<18, 8, 2>(a, s) : launch_step<18, 8, 1>(a, s);
}

// ------------------------------------------------------------------------------------------------
// Expanded route: the scheme of attention_capped.hip's chunk kernel -- a wave owns RG groups of 16 query rows and walks tiles of 64 keys;
// S^T = K Q^T leaves a lane with the scores of 16 keys of one query per group, in the layout the A operand of P V wants; row sums
// come from one more product against ones; the reference maximum moves only when a tile exceeds it by 2^8.  A key is nope channels
// of its own head and the rotated part that all heads share; queries are rotated on their way into the fragments.  Tiles in front
// of the first row's window and behind the last row are never touched.  One LDS stage, the next tile in registers.
// ------------------------------------------------------------------------------------------------
constexpr int kLpKeys = 64;

template <int HDQ, int HDV, int RG>
__global__ __launch_bounds__(256, 2) void latent_prefill_kernel(LatentArgs a) {
    constexpr int KS = HDQ / 32, NT = HDV / 16;
    constexpr int KP = HDQ + 8;   // 16 neighbouring rows, 16 bytes each: 64 banks once
    constexpr int VP = HDV + 16;  // an odd multiple of 8 banks for the transposing reads
    constexpr int WR = 16 * RG, ROWS = 4 * WR;
    constexpr int CQ = HDQ / 8, CV = HDV / 8, NKC = kLpKeys * CQ / 256, NVC = kLpKeys * CV / 256;
    static_assert(kLpKeys * CQ % 256 == 0 && kLpKeys * CV % 256 == 0, "staging shape");
    __shared__ __align__(16) bf16 sk[kLpKeys][KP];
    __shared__ __align__(16) bf16 sv[kLpKeys][VP];
    typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
    typedef short s16x4 __attribute__((ext_vector_type(4)));

    const int qb = gridDim.x - 1 - blockIdx.x;
    const int head = blockIdx.y, b = blockIdx.z;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int qc = lane & 15, s4 = lane >> 4;
    const int pos0 = a.pos0, row0 = qb * ROWS + wave * WR;
    const int hd = a.np + a.rp, ldkv = a.H * (a.np + a.vp);
    const bf16* kv = static_cast<const bf16*>(a.kv) + (int64_t)b * a.n_rows * ldkv;
    const bf16* kn = kv + head * a.np;
    const bf16* vn = kv + a.H * a.np + head * a.vp;
    const bf16* kr = static_cast<const bf16*>(a.rotated) + (int64_t)b * a.t_max * a.rp;
    const int window = a.window > 0 ? a.window : 0x40000000;

    bf16x8 qf[RG][KS];
    int my_pos[RG];
#pragma unroll
    for (int r = 0; r < RG; ++r) {
        const int row = min(row0 + 16 * r + qc, a.S - 1);
        my_pos[r] = pos0 + row0 + 16 * r + qc;
        const bf16* qp = static_cast<const bf16*>(a.q) + ((int64_t)b * a.S + row) * a.H * hd + head * hd;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int d = 32 * ks + 8 * s4;
            Chunk<bf16> v = load_chunk(qp + (d < hd ? d : 0));
            if (d >= a.np && d < hd) {
                const float* cs = a.angles + (int64_t)(pos0 + row) * a.rp + d - a.np;
                const f32x4 c0 = load4(cs), c1 = load4(cs + 4);
                rope_pair<bf16>(v.v[0], v.v[1], c0[0], c0[1]);
                rope_pair<bf16>(v.v[2], v.v[3], c0[2], c0[3]);
                rope_pair<bf16>(v.v[4], v.v[5], c1[0], c1[1]);
                rope_pair<bf16>(v.v[6], v.v[7], c1[2], c1[3]);
            }
            if (d >= hd) v = zero_chunk<bf16>();
            qf[r][ks] = __builtin_bit_cast(bf16x8, v);
        }
    }
    f32x4 o[RG][NT + 1];
    float ref[RG];
#pragma unroll
    for (int r = 0; r < RG; ++r) {
        ref[r] = -INFINITY;
#pragma unroll
        for (int nt = 0; nt <= NT; ++nt) o[r][nt] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    bf16x8 ones;
#pragma unroll
    for (int e = 0; e < 8; ++e) ones[e] = static_cast<bf16>(1.0f);
    const float in_scale = a.scale * 1.4426950408889634f;

    const int n_keys = pos0 + min(qb * ROWS + ROWS, a.S);                // keys 0 .. n_keys - 1 exist for this workgroup
    const int first = max(0, pos0 + qb * ROWS - window + 1);              // the first one its first row sees (>= k0)
    const int t0 = a.k0 + (first - a.k0) / kLpKeys * kLpKeys;
    const int wave_first = pos0 + row0 - window + 1, wave_last = pos0 + row0 + WR - 1;
    u32x4 rk[NKC], rv[NVC];
    auto fetch = [&](int kt) {
#pragma unroll
        for (int i = 0; i < NKC; ++i) {
            const int c = threadIdx.x + 256 * i, d = (c % CQ) * 8;
            const int64_t key = min(kt + c / CQ, n_keys - 1);
            const bf16* p = d < a.np ? kn + (key - a.k0) * ldkv + d : kr + key * a.rp + (d < hd ? d - a.np : 0);
            const u32x4 v = *reinterpret_cast<const u32x4*>(p);
            rk[i] = d < hd ? v : u32x4{0, 0, 0, 0};
        }
#pragma unroll
        for (int i = 0; i < NVC; ++i) {
            const int c = threadIdx.x + 256 * i, d = (c % CV) * 8;
            const int64_t key = min(kt + c / CV, n_keys - 1);
            const u32x4 v = *reinterpret_cast<const u32x4*>(vn + (key - a.k0) * ldkv + (d < a.vp ? d : 0));
            rv[i] = d < a.vp ? v : u32x4{0, 0, 0, 0};
        }
    };
    auto park = [&]() {
#pragma unroll
        for (int i = 0; i < NKC; ++i) {
            const int c = threadIdx.x + 256 * i;
            *reinterpret_cast<u32x4*>(&sk[c / CQ][(c % CQ) * 8]) = rk[i];
        }
#pragma unroll
        for (int i = 0; i < NVC; ++i) {
            const int c = threadIdx.x + 256 * i;
            *reinterpret_cast<u32x4*>(&sv[c / CV][(c % CV) * 8]) = rv[i];
        }
    };
    auto tile = [&](int kt, bool masked) {
        f32x4 sc[RG][4];
#pragma unroll
        for (int r = 0; r < RG; ++r)
#pragma unroll
            for (int t = 0; t < 4; ++t) sc[r][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const bf16x8 kf = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(&sk[16 * t + qc][32 * ks + 8 * s4]));
#pragma unroll
                for (int r = 0; r < RG; ++r) sc[r][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[r][ks], sc[r][t], 0, 0, 0);
            }
        bool moved = false;
        float next[RG];
#pragma unroll
        for (int r = 0; r < RG; ++r) {
            const int d0 = my_pos[r] - kt - 4 * s4;  // distance of this lane's first key
            float mx = -INFINITY;
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    float s = sc[r][t][v] * in_scale;
                    if (masked && (unsigned)(d0 - 16 * t - v) >= (unsigned)window) s = -INFINITY;
                    sc[r][t][v] = s;
                    mx = fmaxf(mx, s);
                }
            mx = max_over_quarters(mx);
            const bool up = mx > ref[r] + 8.f;
            next[r] = up ? mx : ref[r];
            moved |= up;
        }
        if (__builtin_amdgcn_ballot_w64(moved) != 0) {
#pragma unroll
            for (int r = 0; r < RG; ++r) {
                const float corr = next[r] == -INFINITY ? 1.f : __builtin_amdgcn_exp2f(ref[r] - next[r]);
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    const float cv = __shfl(corr, 4 * s4 + v, 64);
#pragma unroll
                    for (int nt = 0; nt <= NT; ++nt) o[r][nt][v] *= cv;
                }
                ref[r] = next[r];
            }
        }
        const bf16* vtr = &sv[4 * s4 + (qc >> 2)][4 * (qc & 3)];
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            bf16x8 pf[RG];
#pragma unroll
            for (int r = 0; r < RG; ++r) {
                const float m = ref[r] == -INFINITY ? 0.f : ref[r];
#pragma unroll
                for (int e = 0; e < 8; ++e) pf[r][e] = static_cast<bf16>(__builtin_amdgcn_exp2f(sc[r][2 * c + e / 4][e % 4] - m));
            }
#pragma unroll
            for (int nt = 0; nt < NT; ++nt) {
                const bf16* p0 = vtr + (32 * c) * VP + 16 * nt;
                const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3)))*)(p0));
                const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3)))*)(p0 + 16 * VP));
                const bf16x8 vf = __builtin_bit_cast(bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
                for (int r = 0; r < RG; ++r) o[r][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[r], vf, o[r][nt], 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < RG; ++r) o[r][NT] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[r], ones, o[r][NT], 0, 0, 0);
        }
    };

    fetch(t0);
    for (int kt = t0; kt < n_keys; kt += kLpKeys) {
        park();
        __syncthreads();
        if (kt + kLpKeys < n_keys) fetch(kt + kLpKeys);
        if (kt <= wave_last && kt + kLpKeys - 1 >= wave_first)
            tile(kt, kt + kLpKeys - 1 > pos0 + row0 || kt < wave_last - window + 1);
        __syncthreads();
    }

    // rows leave through LDS (free behind the last barrier) as 16-byte pieces, gated on the way; each wave has its own 16 rows
    bf16* ot = &sv[0][0] + wave * (16 * VP);
    const bf16* z = static_cast<const bf16*>(a.z) + (int64_t)b * a.S * a.ldz + a.z_gate + head * a.vp;
    bf16* y = static_cast<bf16*>(a.y) + (int64_t)b * a.S * a.H * a.vp + head * a.vp;
#pragma unroll
    for (int r = 0; r < RG; ++r) {
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const float inv = 1.0f / o[r][NT][v];
#pragma unroll
            for (int nt = 0; nt < NT; ++nt) ot[(4 * s4 + v) * VP + 16 * nt + qc] = from_f32<bf16>(o[r][nt][v] * inv);
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        for (int c = lane; c < 16 * CV; c += 64) {
            const int rr = c / CV, d = (c % CV) * 8, row = row0 + 16 * r + rr;
            if (row < a.S && d < a.vp) {
                Chunk<bf16> v;
                *reinterpret_cast<u32x4*>(&v) = *reinterpret_cast<const u32x4*>(ot + rr * VP + d);
                const Chunk<bf16> g = load_chunk(z + (int64_t)row * a.ldz + d);
#pragma unroll
                for (int e = 0; e < 8; ++e) v.v[e] = from_f32<bf16>(to_f32(v.v[e]) * __builtin_amdgcn_rcpf(1.0f + __expf(-to_f32(g.v[e]))));
                store_chunk(y + (int64_t)row * a.H * a.vp + d, v);
            }
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    }
}

template <int HDQ, int HDV>
static int launch_latent_prefill(const LatentArgs& a, int B, hipStream_t s) {
    if ((int64_t)((a.S + 127) / 128) * a.H * B >= 512)
        latent_prefill_kernel<HDQ, HDV, 2><<<dim3((a.S + 127) / 128, a.H, B), dim3(256), 0, s>>>(a);
    else
        latent_prefill_kernel<HDQ, HDV, 1><<<dim3((a.S + 63) / 64, a.H, B), dim3(256), 0, s>>>(a);
    return raven_host::check_launch("latent_attention (chunk)");
}

constexpr int kLpMinRows = 16;  // fewer new rows per sequence take the absorbed route

static bool expands(const raven_latent* l, int S, int pos0, const int* pos_dev, int dtype, int* k0, int* n_rows) {
    if (dtype != RAVEN_BF16 || S < kLpMinRows || pos_dev || l->nope + l->rot > 256 || l->vdim > 128) return false;
    *k0 = l->window > 0 && pos0 - l->window + 1 > 0 ? pos0 - l->window + 1 : 0;
    *n_rows = pos0 + S - *k0;
    return *n_rows <= 64 * S;  // a short chunk behind a very long visible past reads the latents as they are
}

constexpr int kRowHeads = 4;  // heads a workgroup of the vector kernel takes

// position ranges per row: enough workgroups for the chip, at least 64 positions each
static int latent_splits(const raven_latent* l, int B, int S, int dtype, int visible) {
    const bool step = dtype == RAVEN_BF16 && step_fits(l->kv_rank, l->rot);
    const int rg = S * l->heads > 16 ? 32 : 16;
    const int64_t wgs = step ? (int64_t)B * ((S * l->heads + rg - 1) / rg) : (int64_t)B * S * ((l->heads + kRowHeads - 1) / kRowHeads);
    int64_t n = ((step ? 256 : 512) + wgs - 1) / wgs;
    if (n > (visible + 63) / 64) n = (visible + 63) / 64;
    if (n > 32) n = 32;
    return n < 1 ? 1 : (int)n;
}
static int visible_positions(const raven_latent* l, int pos0, int S) {  // by a sequence's S rows together
    const int all = pos0 + S;
    return l->window > 0 && l->window + S - 1 < all ? l->window + S - 1 : all;
}

template <typename T, int CJ>
static int launch_rows_attention(const LatentArgs& a, hipStream_t s) {
    const size_t lds = (((size_t)kRowHeads * (a.kp + a.rp) * sizeof(T) + 15) & ~(size_t)15) + (size_t)4 * kRowHeads * a.kp * sizeof(float);
    if (lds > 48 * 1024) {
        static bool attr_set = false;
        if (!attr_set) {
            const hipError_t e = hipFuncSetAttribute((const void*)latent_rows_attention_kernel<T, kRowHeads, CJ>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
            if (e != hipSuccess) {
                raven_host::set_error("latent_attention: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
                return (int)e;
            }
            attr_set = true;
        }
    }
    latent_rows_attention_kernel<T, kRowHeads, CJ><<<dim3(a.splits, (a.H + kRowHeads - 1) / kRowHeads, a.M), dim3(256), lds, s>>>(a);
    return raven_host::check_launch("latent_attention (rows)");
}

template <typename T, typename Z, int RB>
static int run_absorbed(LatentArgs a, hipStream_t s) {
    // weight rows per workgroup: 16 for one or two token rows (latency), more for more
    a.per_wg = a.M <= 2 ? 1 : a.M <= 64 ? 2 : 4;
    const int rows = 16 * a.per_wg, blocks = (a.M + RB - 1) / RB;
    a.rows_out = (a.kp + rows - 1) / rows;
    absorb_kernel<T, Z, RB><<<dim3(a.H * a.rows_out + (a.append ? 1 : 0), blocks), dim3(256), (size_t)RB * a.np * sizeof(T), s>>>(a);
    if (const int rc = raven_host::check_launch("latent_attention (absorb)")) return rc;
    const int pieces = (a.kp / Chunk<T>::N + 63) / 64;
    int rc;
    if (sizeof(T) == 2 && step_fits(a.kp, a.rp)) rc = run_step(a, s);
    else if (pieces <= 1) rc = launch_rows_attention<T, 1>(a, s);
    else if (pieces <= 2) rc = launch_rows_attention<T, 2>(a, s);
    else rc = launch_rows_attention<T, 4>(a, s);
    if (rc) return rc;
    a.rows_out = (a.vp + rows - 1) / rows;
    latent_out_kernel<T, Z, RB><<<dim3(a.H * a.rows_out, blocks), dim3(256), (size_t)RB * a.kp * sizeof(T), s>>>(a);
    return raven_host::check_launch("latent_attention (out)");
}

static int check_latent(const char* who, const raven_latent* l, const raven_latent_cache* c, int B, int S, int pos0, int dtype) {
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "%s: unknown dtype %d", who, dtype);
    RAVEN_REQUIRE(l && l->heads > 0 && l->q_rank > 0 && l->kv_rank > 0 && l->nope >= 0 && l->rot >= 0 && l->vdim > 0, "%s: bad sizes", who);
    RAVEN_REQUIRE(l->q_rank % 8 == 0 && l->kv_rank % 8 == 0 && l->nope % 8 == 0 && l->rot % 8 == 0 && l->vdim % 8 == 0 && l->nope + l->rot > 0,
                  "%s: sizes must be multiples of 8", who);
    RAVEN_REQUIRE(l->kv_rank <= 1024 && l->rot <= 256 && l->nope <= 1024 && l->vdim <= 1024, "%s: kv_rank %d, rot %d, nope %d or vdim %d is too large", who,
                  l->kv_rank, l->rot, l->nope, l->vdim);
    RAVEN_REQUIRE(l->q_dim > 0 && l->q_dim <= l->q_rank && l->kv_dim > 0 && l->kv_dim <= l->kv_rank, "%s: true sizes exceed the padded ones", who);
    RAVEN_REQUIRE(B >= 0 && S >= 0 && pos0 >= 0 && (int64_t)B * S <= (1 << 24), "%s: bad B=%d S=%d pos0=%d", who, B, S, pos0);
    if (c) {
        RAVEN_REQUIRE(c->latent && (c->rotated || l->rot == 0) && (c->angles || l->rot == 0), "%s: null cache pointer", who);
        RAVEN_REQUIRE(B <= c->batch && pos0 + S <= c->t_max, "%s: %d sequences up to position %d do not fit the cache (%d, %d)", who, B, pos0 + S - 1,
                      c->batch, c->t_max);
    }
    return 0;
}

static LatentArgs latent_args(const raven_latent* l, const raven_latent_cache* c, const void* z, int ldz, int B, int S, int pos0, const int* pos_dev,
                              int dtype) {
    LatentArgs a{};
    const size_t es = raven_host::elt_size(dtype);
    a.z = z; a.ldz = ldz;
    a.latent = c->latent; a.rotated = c->rotated; a.angles = c->angles; a.t_max = c->t_max;
    a.w_uk_t = l->w_uk_t;
    a.w_uv = static_cast<const char*>(l->w_ukv) + (size_t)l->heads * l->nope * l->kv_rank * es;
    a.q_norm = l->q_norm; a.kv_norm = l->kv_norm;
    a.H = l->heads; a.qd = l->q_dim; a.qp = l->q_rank; a.kd = l->kv_dim; a.kp = l->kv_rank; a.np = l->nope; a.rp = l->rot; a.vp = l->vdim;
    a.window = l->window; a.scale = l->scale; a.eps = l->eps;
    a.z_kv = l->q_rank;
    a.z_gate = l->q_rank + (l->own_kv ? l->kv_rank + l->rot : 0);
    a.M = B * S; a.S = S; a.pos0 = pos0; a.pos_dev = pos_dev;
    return a;
}

}  // namespace raven

extern "C" int raven_latent_rows(const raven_latent* l, const void* z, int32_t ldz, int32_t z_f32, const raven_latent_cache* cache, void* cq, int32_t B,
                                 int32_t S, int32_t pos0, const int32_t* pos_dev, int32_t dtype, void* stream) {
    using namespace raven;
    if (const int rc = check_latent("latent_rows", l, cache, B, S, pos0, dtype)) return rc;
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(cache && z && (!cq || l->q_norm) && (!l->own_kv || l->kv_norm) && ldz % 8 == 0, "latent_rows: null pointer or bad pitch %d", ldz);
    LatentArgs a = latent_args(l, cache, z, ldz, B, S, pos0, pos_dev, dtype);
    a.cq = cq;
    a.append = l->own_kv;
    if (!a.cq && !a.append) return 0;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const dim3 grid((a.M + 3) / 4);
    if (dtype == RAVEN_F32) latent_rows_kernel<float, float><<<grid, dim3(256), 0, s>>>(a);
    else if (z_f32) latent_rows_kernel<bf16, float><<<grid, dim3(256), 0, s>>>(a);
    else latent_rows_kernel<bf16, bf16><<<grid, dim3(256), 0, s>>>(a);
    return raven_host::check_launch("latent_rows");
}

extern "C" size_t raven_latent_attention_workspace_bytes(const raven_latent* l, int32_t B, int32_t S, int32_t pos0, int32_t dtype) {
    using namespace raven;
    if (check_latent("latent_attention_workspace_bytes", l, nullptr, B, S, pos0, dtype) || B == 0 || S == 0) return 0;
    const size_t es = raven_host::elt_size(dtype), M = (size_t)B * S;
    const size_t part = M * l->heads * latent_splits(l, B, S, dtype, 1 << 30) * (l->kv_rank + 4) * sizeof(float);
    const size_t absorbed = raven_host::align_up(M * l->heads * (l->kv_rank + l->rot) * es) + raven_host::align_up(part);
    int k0, n_rows;
    if (!expands(l, S, pos0, nullptr, dtype, &k0, &n_rows)) return absorbed;
    const int width = l->heads * (l->nope + l->vdim);
    return raven_host::align_up((size_t)B * n_rows * width * es) + raven_linear_workspace_bytes(n_rows, width);
}

// append: the call writes the rows' cache entries itself (absorbed route only; what raven_latent_rows does otherwise)
namespace raven {
int latent_attention(const raven_latent* l, const void* q, const void* z, int ldz, int z_f32, const raven_latent_cache* cache, void* y, int B, int S,
                     int pos0, const int* pos_dev, int append, int dtype, void* workspace, size_t workspace_bytes, hipStream_t s) {
    if (const int rc = check_latent("latent_attention", l, cache, B, S, pos0, dtype)) return rc;
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(cache && q && z && y && l->w_uk_t && l->w_ukv && ldz % 8 == 0, "latent_attention: null pointer or bad pitch %d", ldz);
    const size_t es = raven_host::elt_size(dtype);
    char* ws = static_cast<char*>(workspace);
    RAVEN_REQUIRE(ws && ((uintptr_t)ws & 255) == 0, "latent_attention: null or unaligned workspace");
    LatentArgs a = latent_args(l, cache, z, ldz, B, S, pos0, pos_dev, dtype);
    a.q = q;
    a.y = y;
    int k0, n_rows;
    if (!z_f32 && !append && expands(l, S, pos0, pos_dev, dtype, &k0, &n_rows)) {
        const int width = l->heads * (l->nope + l->vdim);
        const size_t kv_bytes = raven_host::align_up((size_t)B * n_rows * width * es), lin = raven_linear_workspace_bytes(n_rows, width);
        RAVEN_REQUIRE(kv_bytes + lin <= workspace_bytes, "latent_attention: workspace of %zu bytes is too small", workspace_bytes);
        RAVEN_REQUIRE(B <= 65535 && l->heads <= 65535, "latent_attention: grid too large");
        raven_epilogue e{};
        e.scale = 1.f;
        for (int b = 0; b < B; ++b) {
            const char* c = static_cast<const char*>(cache->latent) + ((size_t)b * cache->t_max + k0) * l->kv_rank * es;
            if (const int rc = raven_linear_epilogue(c, nullptr, l->w_ukv, ws + (size_t)b * n_rows * width * es, n_rows, width, l->kv_rank, 0, &e, dtype,
                                                     ws + kv_bytes, lin, s)) return rc;
        }
        a.kv = ws; a.k0 = k0; a.n_rows = n_rows;
        const int hd = l->nope + l->rot;
        if (l->vdim <= 64) {
            if (hd <= 96) return launch_latent_prefill<96, 64>(a, B, s);
            if (hd <= 192) return launch_latent_prefill<192, 64>(a, B, s);
            return launch_latent_prefill<256, 64>(a, B, s);
        }
        if (hd <= 96) return launch_latent_prefill<96, 128>(a, B, s);
        if (hd <= 192) return launch_latent_prefill<192, 128>(a, B, s);
        return launch_latent_prefill<256, 128>(a, B, s);
    }
    RAVEN_REQUIRE(a.M <= 65535, "latent_attention: %d x %d rows in one call of the absorbed route", B, S);
    a.append = append && l->own_kv;
    a.splits = latent_splits(l, B, S, dtype, visible_positions(l, pos0, S));
    const size_t qa = raven_host::align_up((size_t)a.M * a.H * (a.kp + a.rp) * es);
    RAVEN_REQUIRE(qa + (size_t)a.M * a.H * a.splits * (a.kp + 4) * sizeof(float) <= workspace_bytes, "latent_attention: workspace of %zu bytes is too small",
                  workspace_bytes);
    a.qa = ws;
    a.part = reinterpret_cast<float*>(ws + qa);
    if (dtype == RAVEN_F32) return a.M == 1 ? run_absorbed<float, float, 1>(a, s) : run_absorbed<float, float, 4>(a, s);
    if (z_f32) return a.M == 1 ? run_absorbed<bf16, float, 1>(a, s) : run_absorbed<bf16, float, 4>(a, s);
    return a.M == 1 ? run_absorbed<bf16, bf16, 1>(a, s) : run_absorbed<bf16, bf16, 4>(a, s);
}
}  // namespace raven

extern "C" int raven_latent_attention(const raven_latent* l, const void* q, const void* z, int32_t ldz, int32_t z_f32, const raven_latent_cache* cache,
                                      void* y, int32_t B, int32_t S, int32_t pos0, const int32_t* pos_dev, int32_t dtype, void* workspace,
                                      size_t workspace_bytes, void* stream) {
    return raven::latent_attention(l, q, z, ldz, z_f32, cache, y, B, S, pos0, pos_dev, 0, dtype, workspace, workspace_bytes, static_cast<hipStream_t>(stream));
}
