// Generalised delta rule: a recurrent mixer whose state is one fp32 matrix per sequence and head (row = key channel, column =
// value channel),
//     S_t = diag(w_t) S_(t-1) - (a_t * u_t) (u_t^T S_(t-1)) + k_t v_t^T,     o_t = S_t^T r_t,     u_t = k_t / sqrt(|k_t|^2 + 1e-6)
// with per-channel decays w = exp(-exp(-1/2) sigmoid(.)) and removal rates a = sigmoid(.), followed by the output stage
//     y_t = T( o_t / rms(o_t) * norm * sigmoid(g_t) )       (root mean square per head)
// Everything here is fp32, whatever the model's dtype: the projections arrive as unrounded fp32 rows
//     z = r | k | v | g | a-logits   (five sections of n_heads * head_dim, heads of head_dim channels, zero past the true size)
// and the decay logits in a matrix of their own (they come out of a low-rank product).
//
// The columns of the state never interact, so lanes own columns: 16 lanes share a column (RPL rows each, in registers) and a
// dot product with the column is four DPP adds.
//
//   delta_steps_kernel   one workgroup per (head, sequence) walks the tokens one by one, eight at a time: each of its eight
//       waves prepares one token's vectors into LDS, then all columns advance through the eight tokens without a barrier, then
//       each wave finishes one token's output row.  Decode steps and short chunks.

#include <math.h>

#include "raven_common.h"

namespace raven {

struct DeltaArgs {
    const float* z;       // [M, ldz]: r | k | v | g | a
    const float* decay;   // [M, inner] logits
    const float* a_bias;  // [inner]
    const float* norm;    // [inner]
    float* state;         // [batch, H, hd columns, hd rows]
    void* y;              // [M, inner]
    int H, dim, hd, ldz, S, pos0;
    const int* pos_dev;
    float eps;
};

constexpr int kDeltaTile = 8;  // tokens prepared together = waves of the workgroup

__device__ __forceinline__ float delta_decay(float logit) { return expf(-0.60653065971263342f * sigmoid_f32(logit)); }

// RPL rows per lane (16 * RPL >= hd), CP columns per lane group (32 * CP >= hd)
template <typename T, int RPL, int CP>
__global__ __launch_bounds__(512) void delta_steps_kernel(DeltaArgs a) {
    constexpr int R = 16 * RPL;       // rows held, the last ones zero
    constexpr int KEEP = (R + 63) / 64;
    __shared__ __align__(16) float sw[kDeltaTile][R], su[kDeltaTile][R], sb[kDeltaTile][R], sk[kDeltaTile][R], sr[kDeltaTile][R];
    __shared__ __align__(16) float sv[kDeltaTile][32 * CP], so[kDeltaTile][32 * CP];
    const int h = blockIdx.x, b = blockIdx.y;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int l16 = lane & 15, col0 = wave * 4 + (lane >> 4);
    const int hd = a.hd, inner = a.H * hd;
    const int pos0 = a.pos_dev ? *a.pos_dev : a.pos0;
    float* state = a.state + ((int64_t)b * a.H + h) * hd * hd;

    float S[CP][RPL];
#pragma unroll
    for (int c = 0; c < CP; ++c)
#pragma unroll
        for (int i = 0; i < RPL; ++i) {
            const int col = col0 + 32 * c, r = l16 * RPL + i;
            S[c][i] = (pos0 > 0 && col < hd && r < hd) ? state[(int64_t)col * hd + r] : 0.f;  // a sequence starts from zero
        }

    for (int t0 = 0; t0 < a.S; t0 += kDeltaTile) {
        const int mine = t0 + wave;
        const int64_t m = (int64_t)b * a.S + mine;
        float g[KEEP];
        if (mine < a.S) {
            const float* z = a.z + m * a.ldz + h * hd;
            float k[KEEP], kk = 0.f;
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {
                const int r = lane + 64 * i;
                const bool in = r < hd;
                k[i] = in ? z[inner + r] : 0.f;
                kk = __builtin_fmaf(k[i], k[i], kk);
                g[i] = in ? z[3 * inner + r] : 0.f;
            }
            const float inv = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {
                const int r = lane + 64 * i;
                if (r >= R) continue;
                const bool in = r < hd;
                const float u = k[i] * inv;
                sk[wave][r] = k[i];
                su[wave][r] = u;
                sb[wave][r] = in ? sigmoid_f32(z[4 * inner + r] + a.a_bias[h * hd + r]) * u : 0.f;
                sw[wave][r] = in ? delta_decay(a.decay[m * inner + h * hd + r]) : 0.f;
                sr[wave][r] = in ? z[r] : 0.f;
                if (in) sv[wave][r] = z[2 * inner + r];
            }
        }
        __syncthreads();
        const int n = min(kDeltaTile, a.S - t0);
        for (int t = 0; t < n; ++t) {
            float w[RPL], u[RPL], bb[RPL], k[RPL], r[RPL];
#pragma unroll
            for (int i = 0; i < RPL; ++i) {
                w[i] = sw[t][l16 * RPL + i];
                u[i] = su[t][l16 * RPL + i];
                bb[i] = sb[t][l16 * RPL + i];
                k[i] = sk[t][l16 * RPL + i];
                r[i] = sr[t][l16 * RPL + i];
            }
            float p[CP], o[CP], v[CP];
#pragma unroll
            for (int c = 0; c < CP; ++c) {
                v[c] = sv[t][col0 + 32 * c];
                p[c] = 0.f;
#pragma unroll
                for (int i = 0; i < RPL; ++i) p[c] = __builtin_fmaf(u[i], S[c][i], p[c]);
            }
#pragma unroll
            for (int c = 0; c < CP; ++c) p[c] = row16_sum(p[c]);
#pragma unroll
            for (int c = 0; c < CP; ++c) {
                o[c] = 0.f;
#pragma unroll
                for (int i = 0; i < RPL; ++i) {
                    S[c][i] = __builtin_fmaf(w[i], S[c][i], __builtin_fmaf(k[i], v[c], -bb[i] * p[c]));
                    o[c] = __builtin_fmaf(r[i], S[c][i], o[c]);
                }
            }
#pragma unroll
            for (int c = 0; c < CP; ++c) {
                o[c] = row16_sum(o[c]);
                if (l16 == 0) so[t][col0 + 32 * c] = o[c];
            }
        }
        __syncthreads();
        if (mine < a.S) {
            float o[KEEP], ss = 0.f;
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {
                const int r = lane + 64 * i;
                o[i] = r < hd ? so[wave][r] : 0.f;
                ss = __builtin_fmaf(o[i], o[i], ss);
            }
            const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
            T* y = static_cast<T*>(a.y) + m * inner + h * hd;
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {
                const int r = lane + 64 * i;
                if (r < hd) y[r] = from_f32<T>(o[i] * inv * a.norm[h * hd + r] * sigmoid_f32(g[i]));
            }
        }
    }
#pragma unroll
    for (int c = 0; c < CP; ++c)
#pragma unroll
        for (int i = 0; i < RPL; ++i) {
            const int col = col0 + 32 * c, r = l16 * RPL + i;
            if (col < hd && r < hd) state[(int64_t)col * hd + r] = S[c][i];
        }
}

template <typename T>
static int launch_delta_steps(const DeltaArgs& a, int B, hipStream_t s) {
    const dim3 grid(a.H, B), block(512);
    if (a.hd <= 32) delta_steps_kernel<T, 2, 1><<<grid, block, 0, s>>>(a);
    else if (a.hd <= 48) delta_steps_kernel<T, 3, 2><<<grid, block, 0, s>>>(a);
    else if (a.hd <= 64) delta_steps_kernel<T, 4, 2><<<grid, block, 0, s>>>(a);
    else if (a.hd <= 96) delta_steps_kernel<T, 6, 3><<<grid, block, 0, s>>>(a);
    else if (a.hd <= 128) delta_steps_kernel<T, 8, 4><<<grid, block, 0, s>>>(a);
    else if (a.hd <= 192) delta_steps_kernel<T, 12, 6><<<grid, block, 0, s>>>(a);
    else delta_steps_kernel<T, 16, 8><<<grid, block, 0, s>>>(a);
    return raven_host::check_launch("delta_rule (steps)");
}

}  // namespace raven

extern "C" size_t raven_delta_rule_workspace_bytes(int32_t B, int32_t S, int32_t n_heads, int32_t head_dim) {
    (void)B; (void)S; (void)n_heads; (void)head_dim;
    return 0;
}

extern "C" int raven_delta_rule(const float* z, int32_t ldz, const float* decay_logits, const float* a_bias, const float* norm, float* state,
                                void* y, int32_t B, int32_t S, int32_t pos0, const int32_t* pos_dev, int32_t n_heads, int32_t dim,
                                int32_t head_dim, float eps, int32_t dtype, void* workspace, size_t workspace_bytes, void* stream) {
    using namespace raven;
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "delta_rule: unknown dtype %d", dtype);
    RAVEN_REQUIRE(B >= 0 && B <= 65535 && S >= 0 && pos0 >= 0 && n_heads > 0 && n_heads <= 65535, "delta_rule: bad B=%d S=%d pos0=%d n_heads=%d", B, S,
                  pos0, n_heads);
    RAVEN_REQUIRE(dim > 0 && dim <= head_dim && head_dim % 8 == 0 && head_dim <= 256, "delta_rule: dim %d / head_dim %d (a multiple of 8 up to 256)",
                  dim, head_dim);
    RAVEN_REQUIRE(ldz >= 5 * n_heads * head_dim, "delta_rule: rows of %d elements hold less than five sections", ldz);
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(z && decay_logits && a_bias && norm && state && y, "delta_rule: null pointer");
    DeltaArgs a{};
    a.z = z; a.decay = decay_logits; a.a_bias = a_bias; a.norm = norm; a.state = state; a.y = y;
    a.H = n_heads; a.dim = dim; a.hd = head_dim; a.ldz = ldz; a.S = S; a.pos0 = pos0; a.pos_dev = pos_dev; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    return dtype == RAVEN_BF16 ? launch_delta_steps<bf16>(a, B, s) : launch_delta_steps<float>(a, B, s);
}
