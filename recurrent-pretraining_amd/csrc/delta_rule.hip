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
//
//   Long chunks run in blocks of 16 tokens.  With g_t the products of the block's decays up to token t (per key channel), S the
//   state in front of the block, G = g_16, and rows
//       U_t = u_t g_(t-1),  R_t = r_t g_t,  b_t = a_t u_t,  K_t = k_t / g_t,  B_t = b_t / g_t
//   the removals p_t = u_t^T S_(t-1) of all 16 tokens solve one unit lower triangular system:
//       (I + L) P = U S + M V,   L = stril(U B^T),  M = stril(U K^T)
//       O = R S - tril(R B^T) P + tril(R K^T) V
//       S' = G (S - B^T P + K^T V)
//   (g stays above exp(-16 exp(-1/2)) = 6e-5, so the quotients are harmless in fp32.)  Everything but S and P is independent
//   of the state:
//   delta_block_kernel   one workgroup per (block, head, sequence): the four 16 x 16 products, T = (I + L)^-1 by forward
//       substitution, T U and T M; operands of the next kernel to the workspace.
//   delta_scan_kernel    walks the blocks: one workgroup per 16 columns of a head's state, one wave per 16 rows, the wave's
//       16 x 16 piece of S in four registers per lane for the whole walk (the accumulator layout of the fp32 MFMA read as
//       the B operand of the next product with the k slots permuted accordingly, so S and P never change layout).  The
//       waves exchange their partial sums of P once per block, one barrier; partial sums of O ride along one block later.
//       Operands are requested four blocks ahead.
//   delta_output_kernel  the output stage.
//   All matrix products are fp32 MFMA (16 x 16 x 4).

#include <math.h>

#include "raven_common.h"

namespace raven {

struct DeltaArgs {
    const float* z;       // [M, ldz]: r | k | v | g | a
    const float* decay;   // [M, inner] logits, or null: w_decay tanh(low) + decay_bias, low = z's columns 5 * inner .. + rank - 1
    const void* w_decay;  // [inner, rank] of T
    const float* decay_bias;  // [inner]
    int rank;
    const float* a_bias;  // [inner]
    const float* norm;    // [inner]
    float* state;         // [batch, H, hd columns, hd rows]
    void* y;              // [M, inner]
    int H, dim, hd, ldz, S, pos0;
    const int* pos_dev;
    float eps;
};

constexpr int kDeltaTile = 8;  // tokens prepared together = waves of the workgroup
constexpr int kMaxRank = 256;  // of the decay projection, where the kernel forms it

__device__ __forceinline__ float delta_decay(float logit) { return expf(-0.60653065971263342f * sigmoid_f32(logit)); }

// RPL rows per lane (16 * RPL >= hd), CP columns per lane group (32 * CP >= hd)
template <typename T, int RPL, int CP>
__global__ __launch_bounds__(512) void delta_steps_kernel(DeltaArgs a) {
    constexpr int R = 16 * RPL;       // rows held, the last ones zero
    constexpr int KEEP = (R + 63) / 64;
    __shared__ __align__(16) float sw[kDeltaTile][R], su[kDeltaTile][R], sb[kDeltaTile][R], sk[kDeltaTile][R], sr[kDeltaTile][R];
    __shared__ __align__(16) float sv[kDeltaTile][32 * CP], so[kDeltaTile][32 * CP];
    __shared__ __align__(16) float slow[kDeltaTile][kMaxRank];
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
            float k[KEEP], r[KEEP], v[KEEP], al[KEEP], dl[KEEP], kk = 0.f;
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {  // every load unconditional, so that all are in flight together
                const int c = min(lane + 64 * i, hd - 1);
                k[i] = z[inner + c];
                r[i] = z[c];
                v[i] = z[2 * inner + c];
                g[i] = z[3 * inner + c];
                al[i] = z[4 * inner + c] + a.a_bias[h * hd + c];
                dl[i] = a.decay ? a.decay[m * inner + h * hd + c] : a.decay_bias[h * hd + c];
            }
            if (!a.decay) {
                for (int c = lane; c < a.rank; c += 64) slow[wave][c] = tanhf(a.z[m * a.ldz + 5 * inner + c]);
                __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
                __builtin_amdgcn_wave_barrier();
                __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
                constexpr int E = Chunk<T>::N;
#pragma unroll
                for (int i = 0; i < KEEP; ++i) {
                    const T* w = static_cast<const T*>(a.w_decay) + (int64_t)(h * hd + min(lane + 64 * i, hd - 1)) * a.rank;
                    for (int c = 0; c < a.rank; c += E) {
                        const Chunk<T> x = load_chunk(w + c);
#pragma unroll
                        for (int e = 0; e < E; ++e) dl[i] = __builtin_fmaf(to_f32(x.v[e]), slow[wave][c + e], dl[i]);
                    }
                }
            }
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {
                if (lane + 64 * i >= hd) k[i] = 0.f;
                kk = __builtin_fmaf(k[i], k[i], kk);
            }
            const float inv = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
#pragma unroll
            for (int i = 0; i < KEEP; ++i) {
                const int c = lane + 64 * i;
                if (c >= R) continue;
                const bool in = c < hd;
                const float u = k[i] * inv;
                sk[wave][c] = k[i];
                su[wave][c] = u;
                sb[wave][c] = in ? sigmoid_f32(al[i]) * u : 0.f;
                sw[wave][c] = in ? delta_decay(dl[i]) : 0.f;
                sr[wave][c] = in ? r[i] : 0.f;
                if (in) sv[wave][c] = v[i];
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

// ---- blocks of 16 tokens ----------------------------------------------------------------------------------------
constexpr int kBlk = 16;
constexpr int kScanAhead = 4;        // blocks whose operands are in flight
constexpr int kSegment = 256;        // most blocks per (block, scan) launch pair: bounds the workspace.  A pair costs about 13 us beside its
                                     // blocks (4096 tokens, 32 heads of 64: 307 us in segments of 64 blocks, 281 of 128)
constexpr int kMinBlocked = 48;      // shorter chunks walk token by token
constexpr int kMaxBlockedDim = 128;  // and so do wider heads (the scan's operands would not fit a wave's registers)

// workspace of one (sequence, head, block), in floats; R = rows rounded up to 16
__host__ __device__ constexpr int blk_floats(int R) { return 65 * R + 3 * kBlk * kBlk; }
//   T U [16][R] | R [16][R] | -B^T G [R][16] | K^T G [R][16] | T M [16][16] | -tril(R B^T) | tril(R K^T) | G [R]

struct DeltaBlockArgs {
    DeltaArgs d;
    float* ws;
    float* o;         // [B, H, o_rows, R]: token t of the chunk in row 16 + t, columns past the head unused
    int64_t o_rows;
    int stride;       // blocks the workspace holds per (sequence, head)
    int first;        // first block of the segment
    int n_blocks;     // blocks of the segment, a multiple of kScanAhead (those past the chunk are empty)
};

// a 16 x 16 product over the channels of two row sets in LDS: acc[v] = X[4 q + v] . Y[l16]
template <int R>
__device__ __forceinline__ f32x4 block_product(const float (*X)[R + 4], const float (*Y)[R + 4], int l16, int q) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < R / 16; ++kk) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(&X[l16][16 * kk + 4 * q]);
        const f32x4 y = *reinterpret_cast<const f32x4*>(&Y[l16][16 * kk + 4 * q]);
#pragma unroll
        for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[i], y[i], acc, 0, 0, 0);
    }
    return acc;
}

template <int R>
__global__ __launch_bounds__(256, R <= 64 ? 4 : 2) void delta_block_kernel(DeltaBlockArgs p) {
    constexpr int KEEP = (R + 63) / 64;
    __shared__ __align__(16) float U[kBlk][R + 4], Rt[kBlk][R + 4], Bt[kBlk][R + 4], Kt[kBlk][R + 4];
    __shared__ float part[4][R];                            // each wave's sum of log decays
    __shared__ __align__(16) float L[kBlk][kBlk], Mm[kBlk][kBlk], Ti[kBlk][kBlk + 4];
    const DeltaArgs& a = p.d;
    const int blk = blockIdx.x, h = blockIdx.y, b = blockIdx.z;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, q = lane >> 4;
    const int hd = a.hd, inner = a.H * hd;
    const int t0 = (p.first + blk) * kBlk;
    float* ws = p.ws + (((int64_t)b * a.H + h) * p.stride + blk) * blk_floats(R);
    float *wTU = ws, *wR = ws + 16 * R, *wB = ws + 32 * R, *wK = ws + 48 * R, *wTM = ws + 64 * R, *wRB = wTM + 256, *wRK = wRB + 256, *wG = wRK + 256;

    // this wave's four tokens, channels lane, lane + 64, ...; every load is unconditional (a clamped address, the value dropped)
    // so that all of them are in flight together
    float lw[4][KEEP], u[4][KEEP], bb[4][KEEP], k[4][KEEP], r[4][KEEP], ab[KEEP];
#pragma unroll
    for (int i = 0; i < KEEP; ++i) ab[i] = a.a_bias[h * hd + min(lane + 64 * i, hd - 1)];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int64_t m = (int64_t)b * a.S + min(t0 + 4 * wave + j, a.S - 1);
        const float* z = a.z + m * a.ldz + h * hd;
        const float* dl = a.decay + m * inner + h * hd;
#pragma unroll
        for (int i = 0; i < KEEP; ++i) {
            const int c = min(lane + 64 * i, hd - 1);
            k[j][i] = z[inner + c];
            r[j][i] = z[c];
            bb[j][i] = z[4 * inner + c];
            lw[j][i] = dl[c];
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const bool live = t0 + 4 * wave + j < a.S;  // tokens past the chunk change nothing: zero rows, decay one
        float kk = 0.f;
#pragma unroll
        for (int i = 0; i < KEEP; ++i) {
            const bool in = live && lane + 64 * i < hd;
            k[j][i] = in ? k[j][i] : 0.f;
            r[j][i] = in ? r[j][i] : 0.f;
            bb[j][i] = in ? sigmoid_f32(bb[j][i] + ab[i]) : 0.f;
            lw[j][i] = in ? -0.60653065971263342f * sigmoid_f32(lw[j][i]) : 0.f;
            kk = __builtin_fmaf(k[j][i], k[j][i], kk);
        }
        const float inv = 1.0f / sqrtf(wave_sum(kk) + 1e-6f);
#pragma unroll
        for (int i = 0; i < KEEP; ++i) {
            u[j][i] = k[j][i] * inv;
            bb[j][i] *= u[j][i];
        }
    }
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const int c = lane + 64 * i;
        if (c < R) part[wave][c] = (lw[0][i] + lw[1][i]) + (lw[2][i] + lw[3][i]);
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
        const int c = lane + 64 * i;
        if (c >= R) continue;
        float before = 0.f, total = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
            const float x = part[w][c];
            if (w < wave) before += x;
            total += x;
        }
        f32x4 bo, ko;
        float log_g = before;  // of the token before
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int t = 4 * wave + j;
            U[t][c] = u[j][i] * expf(log_g);
            log_g += lw[j][i];
            const float g = expf(log_g), rest = expf(total - log_g), back = expf(-log_g);
            const float rr = r[j][i] * g;
            Rt[t][c] = rr;
            wR[t * R + c] = rr;
            Bt[t][c] = bb[j][i] * back;
            Kt[t][c] = k[j][i] * back;
            bo[j] = -bb[j][i] * rest;
            ko[j] = k[j][i] * rest;
        }
        *reinterpret_cast<f32x4*>(wB + c * 16 + 4 * wave) = bo;
        *reinterpret_cast<f32x4*>(wK + c * 16 + 4 * wave) = ko;
        if (wave == 3) wG[c] = expf(total);
    }
    __syncthreads();
    // one of the four products per wave; rows are the later token, columns the earlier one
    const f32x4 acc = block_product<R>(wave < 2 ? U : Rt, (wave & 1) ? Kt : Bt, l16, q);
#pragma unroll
    for (int v = 0; v < 4; ++v) {
        const int t = 4 * q + v;
        if (wave == 0) L[t][l16] = l16 < t ? acc[v] : 0.f;
        else if (wave == 1) Mm[t][l16] = l16 < t ? acc[v] : 0.f;
        else if (wave == 2) wRB[t * 16 + l16] = l16 <= t ? -acc[v] : 0.f;
        else wRK[t * 16 + l16] = l16 <= t ? acc[v] : 0.f;
    }
    __syncthreads();
    if (wave == 0) {  // column l16 of T, top down
        float col[kBlk];
#pragma unroll
        for (int t = 0; t < kBlk; ++t) {
            float x = t == l16 ? 1.f : 0.f;
#pragma unroll
            for (int i = 0; i < t; ++i) x = __builtin_fmaf(-L[t][i], col[i], x);
            col[t] = x;
        }
#pragma unroll
        for (int t = 0; t < kBlk; ++t)
            if (q == (t & 3)) Ti[t][l16] = col[t];
    }
    __syncthreads();
    const f32x4 ti = *reinterpret_cast<const f32x4*>(&Ti[l16][4 * q]);
    for (int tile = wave; tile <= R / 16; tile += 4) {  // the column tiles of T U, then T M
        f32x4 x = {0.f, 0.f, 0.f, 0.f};
        const bool last = tile == R / 16;
#pragma unroll
        for (int i = 0; i < 4; ++i)
            x = __builtin_amdgcn_mfma_f32_16x16x4f32(ti[i], last ? Mm[4 * q + i][l16] : U[4 * q + i][(last ? 0 : 16 * tile) + l16], x, 0, 0, 0);
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            if (last) wTM[(4 * q + v) * 16 + l16] = x[v];
            else wTU[(4 * q + v) * R + 16 * tile + l16] = x[v];
        }
    }
}

template <int NB>  // waves = blocks of 16 rows
__global__ __launch_bounds__(64 * NB) void delta_scan_kernel(DeltaBlockArgs p) {
    constexpr int R = 16 * NB;
    __shared__ __align__(16) f32x4 xp[2][NB][64], xo[2][NB][64];
    const DeltaArgs& a = p.d;
    // workgroups go round the eight XCDs: the column tiles of one head, which read the same operands, land on one of them
    const int tiles = (p.d.hd + 15) / 16, n_wgs = tiles * p.d.H;
    const int logical = ((int)blockIdx.x & 7) * ((n_wgs + 7) >> 3) + ((int)blockIdx.x >> 3);
    if (logical >= n_wgs) return;
    const int tile = logical % tiles, h = logical / tiles, b = blockIdx.y;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l16 = lane & 15, q = lane >> 4;
    const int hd = a.hd, inner = a.H * hd;
    const int col = 16 * tile + l16, row = 16 * wave + 4 * q;
    const bool col_ok = col < hd, mine = col_ok && row < hd;  // hd is a multiple of 8: four rows exist together
    const bool fresh = p.first == 0 && (a.pos_dev ? *a.pos_dev : a.pos0) == 0;
    float* state = a.state + (((int64_t)b * a.H + h) * hd + min(col, hd - 1)) * hd + (row < hd ? row : 0);
    const float* ws = p.ws + ((int64_t)b * a.H + h) * p.stride * blk_floats(R);
    const char* vbase = reinterpret_cast<const char*>(a.z + (int64_t)b * a.S * a.ldz + 2 * inner + h * hd);
    // byte offsets below 2^32 (the host checks): uniform bases plus 32-bit lane offsets keep the address arithmetic off the loop
    const unsigned vcol = 4u * min(col, hd - 1), vrow = 4u * a.ldz, vlast = (a.S - 1) * vrow;
    const unsigned at_row = 4u * (l16 * R + row), at_tok = 4u * ((16 * wave + l16) * 16 + 4 * q), at_sq = 4u * (l16 * 16 + 4 * q), at_g = 4u * row;
    float* orow = p.o + (((int64_t)b * a.H + h) * p.o_rows) * R + 16 * tile + l16;
    constexpr int wGV = 0, wRKV = NB - 1, wRBP = NB / 2;  // which wave adds the 16 x 16 products

    f32x4 S = {0.f, 0.f, 0.f, 0.f};
    if (!fresh && mine) S = *reinterpret_cast<const f32x4*>(state);

    struct Set {
        f32x4 tu, r, bt, kt, g, tm, rb, rk;
        float v[4];
    };
    Set st[kScanAhead];
    auto fetch = [&](int c, Set& s) {
        const int cc = min(c, p.n_blocks - 1);
        const char* w = reinterpret_cast<const char*>(ws + (int64_t)cc * blk_floats(R));
        auto at = [&](int floats, unsigned off) { return *reinterpret_cast<const f32x4*>(w + 4 * floats + off); };
        s.tu = at(0, at_row);
        s.r = at(16 * R, at_row);
        s.bt = at(32 * R, at_tok);
        s.kt = at(48 * R, at_tok);
        s.tm = at(64 * R, at_sq);
        s.rb = at(64 * R + 256, at_sq);
        s.rk = at(64 * R + 512, at_sq);
        s.g = at(64 * R + 768, at_g);
        const unsigned first = (unsigned)((p.first + cc) * kBlk) * vrow;  // rows past the chunk repeat its last one: they meet zero factors
#pragma unroll
        for (int i = 0; i < 4; ++i) s.v[i] = *reinterpret_cast<const float*>(vbase + (min(first + (4 * q + i) * vrow, vlast) + vcol));
    };
    auto mac4 = [](const f32x4& x, const float* y, f32x4 acc) {
#pragma unroll
        for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x[i], y[i], acc, 0, 0, 0);
        return acc;
    };
    auto arr = [](const f32x4& x, float* y) {
#pragma unroll
        for (int i = 0; i < 4; ++i) y[i] = x[i];
    };
    // Sums of the O parts that block c's barrier has published: block c - 1's, one of the four rows of a lane per wave (with more
    // than four waves some store the same value twice), to rows 16 c' .. of the walk-through numbering that has an empty block
    // in front.  No condition anywhere: the stores and loads of an iteration can then be counted exactly.
    auto store_o = [&](int buf, float* dst) {
#pragma unroll
        for (int n = 0; n < (4 + NB - 1) / NB; ++n) {
            const int v = (wave + NB * n) & 3;
            float sum = 0.f;
#pragma unroll
            for (int w = 0; w < NB; ++w) sum += reinterpret_cast<const float*>(&xo[buf][w][lane])[v];
            dst[(4 * q + v) * R] = sum;
        }
    };
#pragma unroll
    for (int d = 0; d < kScanAhead; ++d) fetch(d, st[d]);
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    f32x4 O = zero, rb = zero;             // of the block before: its outputs so far, its -tril(R B^T) ...
    float pv[4] = {0.f, 0.f, 0.f, 0.f};    // ... and its removals
    f32x4 P = wave == wGV ? mac4(st[0].tm, st[0].v, zero) : zero;
    for (int c0 = 0; c0 < p.n_blocks; c0 += kScanAhead) {
#pragma unroll
        for (int d = 0; d < kScanAhead; ++d) {
            const int c = c0 + d;
            Set& s = st[d];
            const Set& next = st[(d + 1) % kScanAhead];
            const int buf = d & 1;
            float sv[4];
            arr(S, sv);
            // the chain from block to block: P -> exchange -> S.  Everything else fills the time between P's products and the
            // barrier (the fences keep it there)
            P = mac4(s.tu, sv, P);
            S = mac4(s.kt, s.v, S * s.g);
            xp[buf][wave][lane] = P;
            if (wave == wRBP) O = mac4(rb, pv, O);
            __builtin_amdgcn_sched_barrier(0);
            f32x4 O_next = wave == wRKV ? mac4(s.rk, s.v, zero) : zero;
            O_next = mac4(s.r, sv, O_next);
            xo[buf][wave][lane] = O;
            P = wave == wGV ? mac4(next.tm, next.v, zero) : zero;
            rb = s.rb;
            __builtin_amdgcn_sched_barrier(0);
            __syncthreads();
            f32x4 sum = xp[buf][0][lane];
#pragma unroll
            for (int w = 1; w < NB; ++w) sum += xp[buf][w][lane];
            arr(sum, pv);
            S = mac4(s.bt, pv, S);
            // the first block of a segment has nothing to publish: it writes to the empty block in front
            store_o(buf, orow + (int64_t)(c > 0 ? p.first + c : 0) * kBlk * R);
            O = O_next;
            fetch(c + kScanAhead, s);
        }
    }
    if (wave == wRBP) O = mac4(rb, pv, O);
    __syncthreads();
    xo[0][wave][lane] = O;
    __syncthreads();
    store_o(0, orow + (int64_t)(p.first + p.n_blocks) * kBlk * R);
    if (mine) *reinterpret_cast<f32x4*>(state) = S;
}

// y = T(o / rms(o) * norm * sigmoid(g)); 16 lanes per (row, head), four channels per lane and round
template <typename T, int J>
__global__ __launch_bounds__(256) void delta_output_kernel(DeltaBlockArgs p, int R, int64_t pairs) {
    const DeltaArgs& a = p.d;
    const int64_t i = (int64_t)blockIdx.x * 16 + (threadIdx.x >> 4);
    const int l16 = threadIdx.x & 15;
    const bool ok = i < pairs;
    const int64_t pair = ok ? i : pairs - 1;
    const int h = (int)(pair % a.H);
    const int64_t m = pair / a.H;
    const int b = (int)(m / a.S), t = (int)(m % a.S);
    const int inner = a.H * a.hd;
    const float* row = p.o + (((int64_t)b * a.H + h) * p.o_rows + kBlk + t) * R;
    const float* gate = a.z + m * a.ldz + 3 * inner + h * a.hd;
    f32x4 x[J], g[J], w[J];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int c = 4 * l16 + 64 * j, cc = min(c, a.hd - 4);
        x[j] = *reinterpret_cast<const f32x4*>(row + cc);
        g[j] = *reinterpret_cast<const f32x4*>(gate + cc);
        w[j] = *reinterpret_cast<const f32x4*>(a.norm + h * a.hd + cc);
    }
#pragma unroll
    for (int j = 0; j < J; ++j)
        if (4 * l16 + 64 * j < a.hd) ss += x[j][0] * x[j][0] + x[j][1] * x[j][1] + x[j][2] * x[j][2] + x[j][3] * x[j][3];
    const float inv = 1.0f / sqrtf(row16_sum(ss) / (float)a.dim + a.eps);
    T* y = static_cast<T*>(a.y) + m * inner + h * a.hd;
#pragma unroll
    for (int j = 0; j < J; ++j) {
        const int c = 4 * l16 + 64 * j;
        if (!ok || c >= a.hd) continue;
        T o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = from_f32<T>(x[j][e] * inv * w[j][e] * sigmoid_f32(g[j][e]));
        if constexpr (sizeof(T) == 4) *reinterpret_cast<f32x4*>(y + c) = *reinterpret_cast<const f32x4*>(o);
        else *reinterpret_cast<uint2*>(y + c) = *reinterpret_cast<const uint2*>(o);
    }
}

static int scan_rows(int hd) {  // rows the block kernels are compiled for
    return hd <= 32 ? 32 : hd <= 48 ? 48 : hd <= 64 ? 64 : hd <= 96 ? 96 : 128;
}
static int64_t blocked_o_rows(int S) {  // an empty block in front, the chunk in whole rounds of blocks behind it
    const int round = kBlk * kScanAhead;
    return kBlk + (int64_t)(S + round - 1) / round * round;
}
static int blocked_stride(int S) {
    const int64_t blocks = (blocked_o_rows(S) - kBlk) / kBlk;
    return blocks < kSegment ? (int)blocks : kSegment;
}
static size_t blocked_ws_floats(int B, int S, int H, int hd) {
    const int R = scan_rows(hd);
    return (size_t)B * H * blocked_stride(S) * blk_floats(R) + (size_t)B * H * blocked_o_rows(S) * R;
}

template <int R>
static int launch_delta_segment(const DeltaBlockArgs& p, int B, hipStream_t s) {
    delta_block_kernel<R><<<dim3(p.n_blocks, p.d.H, B), dim3(256), 0, s>>>(p);
    if (const int rc = raven_host::check_launch("delta_rule (blocks)")) return rc;
    delta_scan_kernel<R / 16><<<dim3(((p.d.hd + 15) / 16 * p.d.H + 7) / 8 * 8, B), dim3(4 * R), 0, s>>>(p);
    return raven_host::check_launch("delta_rule (scan)");
}

template <typename T>
static int launch_delta_blocked(const DeltaArgs& a, int B, float* ws, hipStream_t s) {
    DeltaBlockArgs p{};
    p.d = a;
    p.ws = ws;
    p.stride = blocked_stride(a.S);
    p.o = ws + (size_t)B * a.H * p.stride * blk_floats(scan_rows(a.hd));
    p.o_rows = blocked_o_rows(a.S);
    const int blocks = (int)((p.o_rows - kBlk) / kBlk);
    for (p.first = 0; p.first < blocks; p.first += kSegment) {
        p.n_blocks = blocks - p.first < kSegment ? blocks - p.first : kSegment;
        int rc;
        switch (scan_rows(a.hd)) {
            case 32: rc = launch_delta_segment<32>(p, B, s); break;
            case 48: rc = launch_delta_segment<48>(p, B, s); break;
            case 64: rc = launch_delta_segment<64>(p, B, s); break;
            case 96: rc = launch_delta_segment<96>(p, B, s); break;
            default: rc = launch_delta_segment<128>(p, B, s); break;
        }
        if (rc) return rc;
    }
    const int64_t pairs = (int64_t)B * a.S * a.H;
    const dim3 grid((unsigned)((pairs + 15) / 16));
    if (a.hd <= 64) delta_output_kernel<T, 1><<<grid, dim3(256), 0, s>>>(p, scan_rows(a.hd), pairs);
    else delta_output_kernel<T, 2><<<grid, dim3(256), 0, s>>>(p, scan_rows(a.hd), pairs);
    return raven_host::check_launch("delta_rule (output)");
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
    if (B <= 0 || S < raven::kMinBlocked || n_heads <= 0 || head_dim <= 0 || head_dim > raven::kMaxBlockedDim) return 0;
    return raven_host::align_up(raven::blocked_ws_floats(B, S, n_heads, head_dim) * sizeof(float));
}

extern "C" int raven_delta_rule(const float* z, int32_t ldz, const float* decay_logits, const void* w_decay, const float* decay_bias,
                                int32_t rank, const float* a_bias, const float* norm, float* state, void* y, int32_t B, int32_t S, int32_t pos0, const int32_t* pos_dev, int32_t n_heads, int32_t dim,
                                int32_t head_dim, float eps, int32_t dtype, void* workspace, size_t workspace_bytes, void* stream) {
    using namespace raven;
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "delta_rule: unknown dtype %d", dtype);
    RAVEN_REQUIRE(B >= 0 && B <= 65535 && S >= 0 && pos0 >= 0 && n_heads > 0 && n_heads <= 65535, "delta_rule: bad B=%d S=%d pos0=%d n_heads=%d", B, S,
                  pos0, n_heads);
    RAVEN_REQUIRE(dim > 0 && dim <= head_dim && head_dim % 8 == 0 && head_dim <= 256, "delta_rule: dim %d / head_dim %d (a multiple of 8 up to 256)",
                  dim, head_dim);
    RAVEN_REQUIRE(ldz >= 5 * n_heads * head_dim, "delta_rule: rows of %d elements hold less than five sections", ldz);
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(z && a_bias && norm && state && y, "delta_rule: null pointer");
    RAVEN_REQUIRE(decay_logits || (w_decay && decay_bias && rank > 0 && rank % 8 == 0 && rank <= kMaxRank && S <= kDeltaTile && ldz >= 5 * n_heads * head_dim + rank),
                  "delta_rule: without decay logits it needs the low-rank product's operands (rank %d, ldz %d) and at most %d tokens, not %d", rank, ldz,
                  kDeltaTile, S);
    DeltaArgs a{};
    a.z = z; a.decay = decay_logits; a.w_decay = w_decay; a.decay_bias = decay_bias; a.rank = rank; a.a_bias = a_bias; a.norm = norm; a.state = state; a.y = y;
    a.H = n_heads; a.dim = dim; a.hd = head_dim; a.ldz = ldz; a.S = S; a.pos0 = pos0; a.pos_dev = pos_dev; a.eps = eps;
    hipStream_t s = static_cast<hipStream_t>(stream);
    const size_t need = raven_delta_rule_workspace_bytes(B, S, n_heads, head_dim);
    if (need && (int64_t)S * ldz < (1ll << 30) && workspace && need <= workspace_bytes) {
        RAVEN_REQUIRE(((uintptr_t)workspace & 15) == 0 && ((uintptr_t)state & 15) == 0, "delta_rule: workspace and state must be 16-byte aligned");
        float* ws = static_cast<float*>(workspace);
        return dtype == RAVEN_BF16 ? launch_delta_blocked<bf16>(a, B, ws, s) : launch_delta_blocked<float>(a, B, ws, s);
    }
    return dtype == RAVEN_BF16 ? launch_delta_steps<bf16>(a, B, s) : launch_delta_steps<float>(a, B, s);
}
