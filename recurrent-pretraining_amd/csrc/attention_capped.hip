// Attention with capped scores, a per-head distance bias, grouped query heads and keys that serve as values:
//     s_ij = cap * tanh(scale * q_i . k_j / cap) - r1_h * ln(1 + r2_h * (i - j)),   j <= i        (cap <= 0: no cap; r1 null: no bias)
//     y_i  = sum_j softmax_j(s_ij) k_j
// The rows q | k come out of one fused product ([M, (n_heads + n_kv_heads) * head_dim], heads of head_dim elements, zero
// past the head's true size); the cache holds keys only, [batch, n_kv_heads, t_max, head_dim] of T.
//
// Two kernels:
//   capped_attention_kernel          any T, any number of rows: a workgroup takes one row, one key head and up to four of the
//       query heads that read it, and a range of positions.  LPP lanes share a position (16 bytes each), so one 16-byte load
//       per lane serves the score AND the weighted sum of all those query heads -- a cached position is read once per key
//       head.  Ranges are merged by a second launch in range order.  A decode step reads its own position's key from
//       the fused row and appends it to the cache on the way.
//   capped_attention_prefill_kernel  bf16 chunks of 16 and more rows on the matrix cores (further down).

#include <math.h>

#include <type_traits>

#include "raven_common.h"

namespace raven {

// caps whose weights may be taken relative to the cap itself (see the chunk kernel)
static bool fixed_reference(float cap) { return cap > 0.f && cap <= 35.f; }

struct CappedArgs {
    const void* qk;   // [M, ldq]
    void* y;          // [M, ldy]
    void* kc;         // [batch, G, t_max, hd]
    int ldq, ldy;
    int H, G, hd, t_max, S, pos0;
    const int* pos_dev;
    float scale, cap;
    const float* r1;
    const float* r2;
    int append;       // S == 1: the row's own key comes from qk and goes to the cache
    int splits;
    float* part;      // [M, H, splits, hd + 2] when splits > 1
};

// The score behind the product, in natural-log units.  float: the library functions; bf16: hardware exp2 / log2 / reciprocal
// (1 ulp each; the absolute error of the tanh form, 1.2e-7 of the cap, is far below what a bf16 q or k leaves in the product).
template <typename T>
__device__ __forceinline__ float capped_score(float dot, float scale, float cap, float inv_cap, float r1, float r2, float dist) {
    float s = dot * scale;
    if constexpr (sizeof(T) == 4) {
        if (cap > 0.f) s = cap * tanhf(s / cap);
        if (r1 != 0.f) s -= r1 * log1pf(r2 * dist);
    } else {
        if (cap > 0.f) s = cap * (1.0f - 2.0f * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(s * inv_cap * 2.8853900817779268f)));
        if (r1 != 0.f) s -= r1 * 0.69314718055994531f * __builtin_amdgcn_logf(1.0f + r2 * dist);
    }
    return s;
}
template <typename T>
__device__ __forceinline__ float exp_weight(float x) {
    if constexpr (sizeof(T) == 4) return expf(x);
    else return __builtin_amdgcn_exp2f(x * 1.4426950408889634f);
}

template <int LPP>
__device__ __forceinline__ float lanes_sum(float v) {  // over groups of LPP neighbouring lanes
    v += dpp_f<0xB1>(v);
    v += dpp_f<0x4E>(v);
    if (LPP >= 8) v += dpp_f<0x141>(v);
    if (LPP >= 16) v += dpp_f<0x140>(v);
    if (LPP >= 32) v += __shfl_xor(v, 16, 64);
    if (LPP >= 64) v += __shfl_xor(v, 32, 64);
    return v;
}

// FIXED (bf16, caps up to 35): weights are taken relative to the constant +cap, as in the chunk kernel below (its comment says why
// that is safe): no maximum, no rescaling, and ranges merge by plain sums.  The lanes that share a position then also share
// the work behind the product: each turns NQ * U / LPP of the NQ * U scores into weights and hands them round.
template <typename T, int LPP, int NQ, bool FIXED>
__global__ __launch_bounds__(256) void capped_attention_kernel(CappedArgs a) {
    constexpr int E = Chunk<T>::N;
    constexpr int U = 4;                 // positions in flight per lane group
    constexpr int GPW = 64 / LPP, NG = 4 * GPW;
    __shared__ float sm[NG][NQ], sl[NG][NQ];
    __shared__ __align__(16) float so[NG][NQ][LPP * E];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int grp = wave * GPW + lane / LPP, c = lane % LPP;
    const int group = a.H / a.G;
    const int sub = (group + NQ - 1) / NQ;           // workgroups per key head
    const int g = blockIdx.y / sub, q0 = (blockIdx.y % sub) * NQ;
    const int m = blockIdx.z, b = m / a.S, s = m % a.S;
    const int pos = (a.pos_dev ? *a.pos_dev : a.pos0) + s;
    const int n_pos = pos + 1;
    const int span = (n_pos + a.splits - 1) / a.splits;
    const int lo = (int)blockIdx.x * span, hi = min(n_pos, lo + span);
    const bool active = c * E < a.hd;
    const int cc = active ? c : 0;

    const T* row = static_cast<const T*>(a.qk) + (int64_t)m * a.ldq;
    T* keys = static_cast<T*>(a.kc) + ((int64_t)b * a.G + g) * a.t_max * a.hd;
    Chunk<T> q[NQ];
    float r1[NQ], r2[NQ], mx[NQ], l[NQ], acc[NQ][E];
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        const int h = g * group + min(q0 + i, group - 1);
        q[i] = active ? load_chunk(row + h * a.hd + c * E) : zero_chunk<T>();
        r1[i] = a.r1 ? a.r1[h] : 0.f;
        r2[i] = a.r1 ? a.r2[h] : 0.f;
        mx[i] = -INFINITY;
        l[i] = 0.f;
#pragma unroll
        for (int e = 0; e < E; ++e) acc[i][e] = 0.f;
    }
    const float inv_cap = a.cap > 0.f ? 1.0f / a.cap : 0.f;

    // U positions: their scores, one rescaling, their weighted sum
    auto take = [&](const Chunk<T>* k, const int* p, const bool* ok) {
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            float sc[U], top = mx[i];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const float d = lanes_sum<LPP>(dot_chunk(q[i], k[u], 0.f));
                sc[u] = ok[u] ? capped_score<T>(d, a.scale, a.cap, inv_cap, r1[i], r2[i], (float)(pos - p[u])) : -INFINITY;
                top = fmaxf(top, sc[u]);
            }
            const float ref = top == -INFINITY ? 0.f : top;
            const float corr = exp_weight<T>(mx[i] - ref);
            mx[i] = top;
            l[i] *= corr;
#pragma unroll
            for (int e = 0; e < E; ++e) acc[i][e] *= corr;
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const float w = exp_weight<T>(sc[u] - ref);
                l[i] += w;
#pragma unroll
                for (int e = 0; e < E; ++e) acc[i][e] = __builtin_fmaf(w, to_f32(k[u].v[e]), acc[i][e]);
            }
        }
    };
    // FIXED: this lane's pairs (query head, position of the round): pair = c + LPP * j
    constexpr int NP = NQ * U, PER = (NP + LPP - 1) / LPP;
    float pr1[PER], pr2[PER];
    if constexpr (FIXED) {
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            const int i = min((c + LPP * j) / U, NQ - 1);
            pr1[j] = r1[0];
            pr2[j] = r2[0];
#pragma unroll
            for (int k = 1; k < NQ; ++k) {
                pr1[j] = i == k ? r1[k] : pr1[j];
                pr2[j] = i == k ? r2[k] : pr2[j];
            }
        }
    }
    const float in_scale = 2.8853900817779268f * a.scale * inv_cap, drop = -2.8853900817779268f * a.cap;
    auto take_fixed = [&](const Chunk<T>* k, int p0) {
        float d[NP];
#pragma unroll
        for (int n = 0; n < NP; ++n) d[n] = lanes_sum<LPP>(dot_chunk(q[n / U], k[n % U], 0.f));
        float w[PER];
#pragma unroll
        for (int j = 0; j < PER; ++j) {
            float x = d[LPP * j < NP ? LPP * j : 0];
#pragma unroll
            for (int n = 1; n < LPP; ++n)
                if (LPP * j + n < NP) x = c == n ? d[LPP * j + n] : x;
            const int p = p0 + ((c + LPP * j) % U) * NG + grp;
            const float e = drop * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(x * in_scale)) -
                            pr1[j] * __builtin_amdgcn_logf(1.f + pr2[j] * fmaxf((float)(pos - p), 0.f));
            w[j] = p < hi ? __builtin_amdgcn_exp2f(e) : 0.f;
        }
#pragma unroll
        for (int n = 0; n < NP; ++n) {
            const float wn = __shfl(w[n / LPP], (lane & ~(LPP - 1)) | (n % LPP), 64);
            l[n / U] += wn;
#pragma unroll
            for (int e = 0; e < E; ++e) acc[n / U][e] = __builtin_fmaf(wn, to_f32(k[n % U].v[e]), acc[n / U][e]);
        }
    };
    const T* own = row + (int64_t)(a.H + g) * a.hd;  // a decode step's own key is still in its fused row
    for (int p0 = lo; p0 < hi; p0 += NG * U) {
        Chunk<T> k[U];
        int p[U];
        bool ok[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            p[u] = p0 + u * NG + grp;
            ok[u] = p[u] < hi;
            const int at = min(p[u], hi - 1);  // hi > lo >= 0 here
            k[u] = load_chunk((a.append && at == pos ? own : keys + (int64_t)at * a.hd) + cc * E);
        }
        if constexpr (FIXED) take_fixed(k, p0);
        else take(k, p, ok);
    }
    if (a.append && (int)blockIdx.x == a.splits - 1 && q0 == 0 && grp == 0 && active && pos < a.t_max)
        store_chunk(keys + (int64_t)pos * a.hd + c * E, load_chunk(own + c * E));

#pragma unroll
    for (int i = 0; i < NQ; ++i) {
        if (c == 0) {
            sm[grp][i] = FIXED ? 1.f : mx[i];
            sl[grp][i] = l[i];
        }
#pragma unroll
        for (int e = 0; e < E; e += 4) *reinterpret_cast<f32x4*>(&so[grp][i][c * E + e]) = f32x4{acc[i][e], acc[i][e + 1], acc[i][e + 2], acc[i][e + 3]};
    }
    __syncthreads();
    // merge: the groups' factors first (group-major threads), then every output is one dot product over the groups
    float top[NQ];
#pragma unroll
    for (int i = 0; i < NQ; ++i) top[i] = 0.f;
    if constexpr (!FIXED) {
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            float x = -INFINITY;
            for (int n = lane; n < NG; n += 64) x = fmaxf(x, sm[n][i]);
            top[i] = wave_max(x);
        }
        __syncthreads();
        for (int t = threadIdx.x; t < NG * NQ; t += 256) {
            const int n = t / NQ, i = t % NQ;
            float ref = top[0];
#pragma unroll
            for (int k = 1; k < NQ; ++k) ref = i == k ? top[k] : ref;
            sm[n][i] = exp_weight<T>(sm[n][i] - (ref == -INFINITY ? 0.f : ref));
        }
        __syncthreads();
    }
    for (int t = threadIdx.x; t < NQ * a.hd; t += 256) {
        const int i = t / a.hd, col = t - i * a.hd;
        if (q0 + i >= group) break;
        float sum = 0.f, o = 0.f;
#pragma unroll 8
        for (int n = 0; n < NG; ++n) {
            const float w = FIXED ? 1.f : sm[n][i];
            sum = __builtin_fmaf(w, sl[n][i], sum);
            o = __builtin_fmaf(w, so[n][i][col], o);
        }
        const int h = g * group + q0 + i;
        if (a.splits == 1) {
            static_cast<T*>(a.y)[(int64_t)m * a.ldy + h * a.hd + col] = from_f32<T>(o / sum);
        } else {
            float* p = a.part + (((int64_t)m * a.H + h) * a.splits + blockIdx.x) * (a.hd + 2);
            float ref = top[0];
#pragma unroll
            for (int k = 1; k < NQ; ++k) ref = i == k ? top[k] : ref;
            p[2 + col] = o;
            if (col == 0) {
                p[0] = ref;
                p[1] = sum;
            }
        }
    }
}

// Lane n holds range n's reference and sum (at most 32 ranges); the columns then add eight ranges' partials per round, all
// requested before the first is used.
template <typename T>
__global__ __launch_bounds__(64) void capped_combine_kernel(CappedArgs a) {
    const int h = blockIdx.x, m = blockIdx.y, lane = threadIdx.x;
    const int ld = a.hd + 2;
    const float* p = a.part + ((int64_t)m * a.H + h) * a.splits * ld;
    const int mine = min(lane, a.splits - 1);
    const float ref = p[(int64_t)mine * ld], sum = p[(int64_t)mine * ld + 1];
    const float top = wave_max(ref);  // some range always holds a position, so it is finite
    const float w = lane < a.splits ? exp_weight<T>(ref - top) : 0.f;
    const float inv = 1.0f / wave_sum(w * sum);
    for (int c0 = 0; c0 < a.hd; c0 += 64) {
        const int col = min(c0 + lane, a.hd - 1);
        float o = 0.f;
        for (int n0 = 0; n0 < a.splits; n0 += 8) {
            float x[8];
#pragma unroll
            for (int n = 0; n < 8; ++n) x[n] = p[(int64_t)min(n0 + n, a.splits - 1) * ld + 2 + col];
#pragma unroll
            for (int n = 0; n < 8; ++n) o = __builtin_fmaf(__shfl(w, n0 + n, 64), x[n], o);  // lanes past the last range hold 0
        }
        if (c0 + lane < a.hd) static_cast<T*>(a.y)[(int64_t)m * a.ldy + h * a.hd + c0 + lane] = from_f32<T>(o * inv);
    }
}

// keys of the fused rows -> cache positions pos0 .. pos0 + S - 1
template <typename T>
__global__ __launch_bounds__(256) void key_append_kernel(CappedArgs a, int M) {
    constexpr int E = Chunk<T>::N;
    const int cpr = a.hd / E;
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= (int64_t)M * a.G * cpr) return;
    const int c = (int)(i % cpr), g = (int)(i / cpr % a.G), m = (int)(i / cpr / a.G);
    const int b = m / a.S, pos = (a.pos_dev ? *a.pos_dev : a.pos0) + m % a.S;
    if (pos >= a.t_max) return;
    store_chunk(static_cast<T*>(a.kc) + (((int64_t)b * a.G + g) * a.t_max + pos) * a.hd + c * E,
                load_chunk(static_cast<const T*>(a.qk) + (int64_t)m * a.ldq + (int64_t)(a.H + g) * a.hd + c * E));
}

// ------------------------------------------------------------------------------------------------
// bf16 chunks on the matrix cores, the scheme of attention_prefill.hip: a wave owns RG groups of 16 query rows and walks tiles
// of 64 keys; S^T = K Q^T leaves a lane with the scores of 16 keys of ONE query per group, in the layout the A operand of
// P V wants; the weights' row sums come from one more product against ones; the reference maximum moves only when a tile
// exceeds it by 2^8.  Keys are values, so ONE staged tile serves both products: read by rows for the scores and
// through the transposing loads for P V.  Heads of up to HD channels (multiples of 8) sit zero-padded in the tile.
//
// A score costs four quarter-rate instructions (exp2 and reciprocal for the cap, log2 for the distance, exp2 for the weight)
// where plain attention has one: the kernel is bound by vector work, not by the products.  The FIXED variant saves one of them
// and the running maximum:
//   * a capped score lies in [-cap, cap] and a row always sees its own position, whose bias is ln 1 = 0, so weights relative
//     to the constant +cap never lose the row's sum below exp(-2 cap): for caps up to 35 (2^-101) nothing that matters
//     underflows and no maximum is needed;
//   * exp(-bias) = (1 + r2 d)^-r1 multiplies the weight and depends on the distance alone: the workgroup tabulates its tile's
//     ROWS + 63 distances once per tile, zero for keys behind the query, which is the causal mask.  A lane's four
//     consecutive keys are one 16-byte read; the table is stored four times, shifted by one element each, so that the
//     read is aligned whatever the lane's query.
// ------------------------------------------------------------------------------------------------
constexpr int kCpKeys = 64;

template <int HD, int RG, bool FIXED>
__global__ __launch_bounds__(256, 2) void capped_attention_prefill_kernel(CappedArgs a) {
    constexpr int KS = HD / 32, NT = HD / 16;
    constexpr int KP = HD + 16;          // an odd multiple of 8 banks: the transposing reads of 8 key rows hit 64 banks
    constexpr int WR = 16 * RG, ROWS = 4 * WR;
    constexpr int CPR = HD / 8, KCH = kCpKeys * CPR / 256;
    static_assert(kCpKeys * CPR % 256 == 0, "staging shape");
    __shared__ __align__(16) bf16 sk[2][kCpKeys][KP];
    constexpr int NE = ROWS + kCpKeys - 1;   // distances a tile holds
    __shared__ __align__(16) float table[FIXED ? 2 : 1][FIXED ? 4 : 1][FIXED ? (NE + 7) / 4 * 4 : 1];
    typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
    typedef short s16x4 __attribute__((ext_vector_type(4)));

    const int qb = gridDim.x - 1 - blockIdx.x;  // the blocks with the most keys start first
    const int head = blockIdx.y, b = blockIdx.z, g = head / (a.H / a.G);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int qc = lane & 15, s4 = lane >> 4;
    const int pos0 = a.pos_dev ? *a.pos_dev : a.pos0;
    const int hd = a.hd, row0 = qb * ROWS + wave * WR;
    const bf16* keys = static_cast<const bf16*>(a.kc) + ((int64_t)b * a.G + g) * a.t_max * hd;
    const bf16* q = static_cast<const bf16*>(a.qk) + (int64_t)b * a.S * a.ldq + head * hd;

    bf16x8 qf[RG][KS];
    int my_pos[RG];
#pragma unroll
    for (int r = 0; r < RG; ++r) {
        const int row = row0 + 16 * r + qc;
        my_pos[r] = pos0 + row;
        const bf16* qp = q + (int64_t)min(row, a.S - 1) * a.ldq;
#pragma unroll
        for (int ks = 0; ks < KS; ++ks) {
            const int d = 32 * ks + 8 * s4;
            const u32x4 v = *reinterpret_cast<const u32x4*>(qp + (d < hd ? d : 0));
            qf[r][ks] = __builtin_bit_cast(bf16x8, d < hd ? v : u32x4{0, 0, 0, 0});
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
    // scores in log2 units: with a cap, cap2 - 2 cap2 / (1 + exp2(x in_scale)) and in_scale = 2 log2(e) scale / cap
    const float log2e = 1.4426950408889634f;
    const bool capped = a.cap > 0.f;
    const float in_scale = capped ? 2.f * log2e * a.scale / a.cap : a.scale * log2e;
    const float cap2 = a.cap * log2e;
    const bool biased = a.r1 != nullptr;
    const float r1 = biased ? a.r1[head] : 0.f, r2 = biased ? a.r2[head] : 0.f;

    const int n_keys = min(pos0 + min(qb * ROWS + ROWS, a.S), a.t_max);
    const int wave_last = pos0 + row0 + WR - 1;
    u32x4 reg[KCH];
    auto fetch = [&](int kt) {
#pragma unroll
        for (int i = 0; i < KCH; ++i) {
            const int c = threadIdx.x + 256 * i;
            const int key = min(kt + c / CPR, a.t_max - 1), d = (c % CPR) * 8;
            const u32x4 v = *reinterpret_cast<const u32x4*>(keys + (int64_t)key * hd + (d < hd ? d : 0));
            reg[i] = d < hd ? v : u32x4{0, 0, 0, 0};
        }
    };
    // keys past the last row's own position may never have been written: weight 0 times whatever lies there must stay 0
    auto park = [&](int kt, int buf) {
#pragma unroll
        for (int i = 0; i < KCH; ++i) {
            const int c = threadIdx.x + 256 * i;
            *reinterpret_cast<u32x4*>(&sk[buf][c / CPR][(c % CPR) * 8]) = kt + c / CPR < n_keys ? reg[i] : u32x4{0, 0, 0, 0};
        }
    };

    // entry e: the key of distance d = (first row's position) - kt + ROWS - 1 - e; copy c holds entry e at place e - c
    auto tabulate = [&](int kt, int buf) {
        if constexpr (FIXED) {
            const int e = threadIdx.x;
            if (e < NE) {
                const int d = pos0 + qb * ROWS - kt + ROWS - 1 - e;
                float w = 1.f;
                if (biased) w = __builtin_amdgcn_exp2f(-r1 * __builtin_amdgcn_logf(__builtin_fmaf(r2, (float)d, 1.f)));
                if (d < 0) w = 0.f;
#pragma unroll
                for (int c = 0; c < 4; ++c)
                    if (e >= c) table[buf][c][e - c] = w;
            }
        }
    };

    auto tile = [&](int kt, int buf, bool masked) {
        f32x4 sc[RG][4];
#pragma unroll
        for (int r = 0; r < RG; ++r)
#pragma unroll
            for (int t = 0; t < 4; ++t) sc[r][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const bf16x8 kf = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(&sk[buf][16 * t + qc][32 * ks + 8 * s4]));
#pragma unroll
                for (int r = 0; r < RG; ++r) sc[r][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[r][ks], sc[r][t], 0, 0, 0);
            }
        if constexpr (FIXED) {
#pragma unroll
            for (int r = 0; r < RG; ++r) {
                const int e0 = ROWS - 1 - (wave * WR + 16 * r + qc) + 4 * s4, shift = (3 - qc) & 3;  // e0 = shift mod 4
                const float* fac = &table[buf][shift][e0 - shift];
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    const f32x4 w = *reinterpret_cast<const f32x4*>(fac + 16 * t);
#pragma unroll
                    for (int v = 0; v < 4; ++v)
                        sc[r][t][v] = w[v] * __builtin_amdgcn_exp2f(-2.f * cap2 * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(sc[r][t][v] * in_scale)));
                }
            }
        }
        bool moved = false;
        float next[RG];
#pragma unroll
        for (int r = 0; r < RG && !FIXED; ++r) {
            const float d0 = (float)(my_pos[r] - kt - 4 * s4);
            float mx = -INFINITY;
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int v = 0; v < 4; ++v) {
                    float s = sc[r][t][v] * in_scale;
                    if (capped) s = __builtin_fmaf(-2.f * cap2, __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(s)), cap2);
                    // a key behind the query has a negative distance: clamped, and hidden below
                    if (biased) s = __builtin_fmaf(-r1, __builtin_amdgcn_logf(__builtin_fmaf(r2, fmaxf(d0 - (float)(16 * t + v), 0.f), 1.f)), s);
                    if (masked && kt + 16 * t + 4 * s4 + v > my_pos[r]) s = -INFINITY;
                    sc[r][t][v] = s;
                    mx = fmaxf(mx, s);
                }
            mx = max_over_quarters(mx);
            const bool up = mx > ref[r] + 8.f;
            next[r] = up ? mx : ref[r];
            moved |= up;
        }
        if (!FIXED && __builtin_amdgcn_ballot_w64(moved) != 0) {
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
        const bf16* vtr = &sk[buf][4 * s4 + (qc >> 2)][4 * (qc & 3)];
#pragma unroll
        for (int c = 0; c < 2; ++c) {
            bf16x8 pf[RG];
#pragma unroll
            for (int r = 0; r < RG; ++r) {
                const float m = ref[r] == -INFINITY ? 0.f : ref[r];
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const float x = sc[r][2 * c + e / 4][e % 4];
                    pf[r][e] = static_cast<bf16>(FIXED ? x : __builtin_amdgcn_exp2f(x - m));
                }
            }
#pragma unroll
            for (int nt = 0; nt < NT; ++nt) {
                const bf16* p0 = vtr + (32 * c) * KP + 16 * nt;
                const s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3)))*)(p0));
                const s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((s16x4 __attribute__((address_space(3)))*)(p0 + 16 * KP));
                const bf16x8 vf = __builtin_bit_cast(bf16x8, __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
                for (int r = 0; r < RG; ++r) o[r][nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[r], vf, o[r][nt], 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < RG; ++r) o[r][NT] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[r], ones, o[r][NT], 0, 0, 0);
        }
    };

    fetch(0);
    park(0, 0);
    tabulate(0, 0);
    if (kCpKeys < n_keys) fetch(kCpKeys);
    __syncthreads();
    int buf = 0;
    for (int kt = 0; kt < n_keys; kt += kCpKeys, buf ^= 1) {
        if (kt + kCpKeys - 1 <= pos0 + row0) tile(kt, buf, false);
        else if (kt <= wave_last) tile(kt, buf, true);
        if (kt + kCpKeys < n_keys) {
            tabulate(kt + kCpKeys, buf ^ 1);
            park(kt + kCpKeys, buf ^ 1);  // last read two tiles ago; every wave has passed the barrier since
            if (kt + 2 * kCpKeys < n_keys) fetch(kt + 2 * kCpKeys);
        }
        __syncthreads();
    }

    // rows leave through LDS (free after the last barrier) as 16-byte pieces; each wave has its own 16 rows
    bf16* ot = &sk[0][0][0] + wave * (16 * KP);
    static_assert(2 * kCpKeys >= 4 * 16, "the output pass fits the staging buffers");
    bf16* y = static_cast<bf16*>(a.y) + (int64_t)b * a.S * a.ldy + head * hd;
#pragma unroll
    for (int r = 0; r < RG; ++r) {
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const float inv = 1.0f / o[r][NT][v];
#pragma unroll
            for (int nt = 0; nt < NT; ++nt) ot[(4 * s4 + v) * KP + 16 * nt + qc] = from_f32<bf16>(o[r][nt][v] * inv);
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        for (int c = lane; c < 16 * CPR; c += 64) {
            const int rr = c / CPR, d = (c % CPR) * 8, row = row0 + 16 * r + rr;
            if (row < a.S && d < hd) *reinterpret_cast<u32x4*>(y + (int64_t)row * a.ldy + d) = *reinterpret_cast<const u32x4*>(ot + rr * KP + d);
        }
        __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
        __builtin_amdgcn_wave_barrier();
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    }
}

template <int HD>
static int launch_capped_prefill(const CappedArgs& a, int B, hipStream_t s) {
    const int rg = (int64_t)((a.S + 127) / 128) * a.H * B >= 512 ? 2 : 1;
    const dim3 grid((a.S + 64 * rg - 1) / (64 * rg), a.H, B);
    const bool fixed = fixed_reference(a.cap);
    if (rg == 2) {
        if (fixed) capped_attention_prefill_kernel<HD, 2, true><<<grid, dim3(256), 0, s>>>(a);
        else capped_attention_prefill_kernel<HD, 2, false><<<grid, dim3(256), 0, s>>>(a);
    } else {
        if (fixed) capped_attention_prefill_kernel<HD, 1, true><<<grid, dim3(256), 0, s>>>(a);
        else capped_attention_prefill_kernel<HD, 1, false><<<grid, dim3(256), 0, s>>>(a);
    }
    return raven_host::check_launch("capped_attention (prefill)");
}

constexpr int kCpMinRows = 16;  // fewer new rows per sequence go to the row kernel

static int run_capped_prefill(const CappedArgs& a, int B, hipStream_t s) {
    const int64_t n = (int64_t)B * a.S * a.G * (a.hd / 8);
    key_append_kernel<bf16><<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s>>>(a, B * a.S);
    if (const int rc = raven_host::check_launch("capped_attention (append)")) return rc;
    if (a.hd <= 32) return launch_capped_prefill<32>(a, B, s);
    if (a.hd <= 64) return launch_capped_prefill<64>(a, B, s);
    if (a.hd <= 96) return launch_capped_prefill<96>(a, B, s);
    return launch_capped_prefill<128>(a, B, s);
}

static int capped_nq(int group) { return group >= 4 ? 4 : group >= 2 ? 2 : 1; }

// position ranges per (row, key head): enough workgroups for the chip, at least 128 positions each
static int capped_splits(int rows, int H, int G, int n_pos) {
    const int group = H / G, nq = capped_nq(group);
    const int64_t wgs = (int64_t)rows * G * ((group + nq - 1) / nq);
    int64_t n = (512 + wgs - 1) / wgs;
    if (n > (n_pos + 127) / 128) n = (n_pos + 127) / 128;
    if (n > 32) n = 32;
    return n < 1 ? 1 : (int)n;
}

template <typename T, int LPP>
static int launch_capped(const CappedArgs& a, int M, hipStream_t s) {
    const int group = a.H / a.G, nq = capped_nq(group);
    const dim3 grid(a.splits, a.G * ((group + nq - 1) / nq), M);
    auto run = [&](auto fixed) {
        constexpr bool F = decltype(fixed)::value;
        if (nq == 4) capped_attention_kernel<T, LPP, 4, F><<<grid, dim3(256), 0, s>>>(a);
        else if (nq == 2) capped_attention_kernel<T, LPP, 2, F><<<grid, dim3(256), 0, s>>>(a);
        else capped_attention_kernel<T, LPP, 1, F><<<grid, dim3(256), 0, s>>>(a);
    };
    if constexpr (sizeof(T) == 2) {
        if (fixed_reference(a.cap)) run(std::true_type{});
        else run(std::false_type{});
    } else {
        run(std::false_type{});
    }
    if (a.splits > 1) capped_combine_kernel<T><<<dim3(a.H, M), dim3(64), 0, s>>>(a);
    return raven_host::check_launch("capped_attention");
}

template <typename T>
static int run_capped(CappedArgs a, int M, hipStream_t s) {
    constexpr int E = Chunk<T>::N;
    if (!a.append) {
        const int64_t n = (int64_t)M * a.G * (a.hd / E);
        key_append_kernel<T><<<dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s>>>(a, M);
        if (const int rc = raven_host::check_launch("capped_attention (append)")) return rc;
    }
    const int chunks = a.hd / E;
    if (chunks <= 4) return launch_capped<T, 4>(a, M, s);
    if (chunks <= 8) return launch_capped<T, 8>(a, M, s);
    if (chunks <= 16) return launch_capped<T, 16>(a, M, s);
    if (chunks <= 32) return launch_capped<T, 32>(a, M, s);
    return launch_capped<T, 64>(a, M, s);
}

}  // namespace raven

extern "C" size_t raven_capped_attention_workspace_bytes(int32_t M, int32_t n_heads, int32_t n_kv_heads, int32_t head_dim) {
    if (M <= 0 || n_heads <= 0 || n_kv_heads <= 0 || head_dim <= 0) return 0;
    const int splits = raven::capped_splits(M, n_heads, n_kv_heads, 1 << 30);
    return splits > 1 ? raven_host::align_up((size_t)M * n_heads * splits * (head_dim + 2) * sizeof(float)) : 0;
}

extern "C" int raven_capped_attention(const void* qk, void* y, const raven_key_cache* cache, const raven_score* score, int32_t B, int32_t S,
                                      int32_t pos0, const int32_t* pos_dev, int32_t n_heads, int32_t dtype, void* workspace,
                                      size_t workspace_bytes, void* stream) {
    using namespace raven;
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "capped_attention: unknown dtype %d", dtype);
    RAVEN_REQUIRE(cache && score && cache->k, "capped_attention: null pointer");
    RAVEN_REQUIRE(B >= 0 && S >= 0 && pos0 >= 0 && n_heads > 0, "capped_attention: bad B=%d S=%d pos0=%d", B, S, pos0);
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(qk && y, "capped_attention: null pointer");
    RAVEN_REQUIRE(B <= cache->batch, "capped_attention: batch %d exceeds the cache's %d", B, cache->batch);
    RAVEN_REQUIRE(cache->n_kv_heads > 0 && n_heads % cache->n_kv_heads == 0, "capped_attention: %d query heads for %d key heads", n_heads,
                  cache->n_kv_heads);
    RAVEN_REQUIRE(cache->head_dim > 0 && cache->head_dim % 8 == 0 && cache->head_dim <= 256, "capped_attention: head_dim %d is not a multiple of 8 up to 256",
                  cache->head_dim);
    RAVEN_REQUIRE(pos0 + S <= cache->t_max, "capped_attention: positions up to %d exceed the cache length %d", pos0 + S - 1, cache->t_max);
    RAVEN_REQUIRE((score->r1 == nullptr) == (score->r2 == nullptr), "capped_attention: r1 and r2 must be given together");
    CappedArgs a{};
    a.qk = qk; a.y = y; a.kc = cache->k;
    a.H = n_heads; a.G = cache->n_kv_heads; a.hd = cache->head_dim; a.t_max = cache->t_max; a.S = S; a.pos0 = pos0; a.pos_dev = pos_dev;
    a.ldq = (a.H + a.G) * a.hd; a.ldy = a.H * a.hd;
    a.scale = score->scale; a.cap = score->softcap; a.r1 = score->r1; a.r2 = score->r2;
    a.append = S == 1;
    const int M = B * S;
    hipStream_t s = static_cast<hipStream_t>(stream);
    if (dtype == RAVEN_BF16 && S >= kCpMinRows && a.hd <= 128) {
        RAVEN_REQUIRE(B <= 65535 && a.H <= 65535, "capped_attention: grid too large");
        return run_capped_prefill(a, B, s);
    }
    RAVEN_REQUIRE((int64_t)B * S <= 65535, "capped_attention: %d x %d rows in one call", B, S);
    a.splits = capped_splits(M, a.H, a.G, pos0 + S);
    while (a.splits > 1 && (workspace == nullptr || (size_t)M * a.H * a.splits * (a.hd + 2) * sizeof(float) > workspace_bytes)) --a.splits;
    a.part = static_cast<float*>(workspace);
    return dtype == RAVEN_BF16 ? run_capped<bf16>(a, M, s) : run_capped<float>(a, M, s);
}
