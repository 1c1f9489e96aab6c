// Mixture of gated experts over an fp32 stream (raven_moe_forward):
//     x += sum over the chosen experts of W_down ( silu(s W_gate h) * (s W_up h) )  +  sigmoid(g) W_down' ( silu(W_gate' h) * (W_up' h) )
// s = sigmoid(router logit): the factor of an expert's input is applied to the sums of its first two products, which is the same.
//
// Few rows (and fp32): moe_up_kernel forms the gated activations of a row's experts and of the shared one side by side, moe_down_kernel
// multiplies them by the down matrices and adds to the stream.  The first picks the row's experts itself from its logits -- a handful
// of wave reductions -- so no routing launch stands in between; for a single row it also takes the norm of the stream as a prologue.
// bf16 chunks: the rows are sorted by expert (moe_pick_kernel, moe_sort_kernel) and the experts run as one grouped product on the
// matrix cores (gemm_tiled.hip), rows gathered through the sorted list; every (token, expert) pair has a slot of its own, and
// moe_combine_kernel adds a token's slots and its shared expert to the stream in a fixed order.

#include "row_helpers.h"

namespace raven {

int grouped_gemm(const void* x, int x_rows, const void* w, int64_t w_stride, void* y, int rows, int N, int K, int swiglu, const int* group_of,
                 const int* group_row, const int* group_end, int n_tiles, int tile_rows, const int* x_row, const float* x_scale, hipStream_t s);

constexpr int kMaxExperts = 1024, kMaxTop = 32;
constexpr int kBigTileRows = 320;  // rows per expert from which the grouped products take 256-row tiles
constexpr int kPickRows = 32;  // tokens a workgroup of the two sorting kernels owns

struct MoeArgs {
    const void *h, *up, *down, *shared_up, *shared_down;
    const float* logits;
    float* x;
    const float* norm;      // h null (one row): the norm of x that gives it, with its true width and eps
    int dim;
    float eps;
    void* act;              // few rows: [M, top * ff + shared_ff] of T
    int M, ld, ldl, experts, top, ff, sff;
    // chunks
    int* pick;              // [M, top]: expert
    float* pick_scale;      // [M, top]: its score
    int *slot_of;           // [M, top]: row of the grouped product
    int *slot_row;          // [M * top]: token of a slot
    float* slot_scale;      // [M * top]
    int *group_of, *group_row, *group_end;
    int n_tiles, tile_rows;
    int* block_count;       // [ceil(M / kPickRows), experts]: pairs of a workgroup's tokens
    const bf16* y;          // [M * top, ld]
    const float* ys;        // [M, ld] or null
};

// one wave: the `top` experts of largest logit (lower index first among equals); lane k holds the k-th one and its score
__device__ __forceinline__ void pick_experts(const float* logits, int experts, int top, int& mine, float& score) {
    const int lane = threadIdx.x & 63;
    float v[kMaxExperts / 64];
#pragma unroll
    for (int j = 0; j < kMaxExperts / 64; ++j) {
        v[j] = -INFINITY;
        if (64 * j < experts && lane + 64 * j < experts) v[j] = logits[lane + 64 * j];
    }
    mine = 0;
    float logit = 0.f;
    for (int k = 0; k < top; ++k) {
        float best = -INFINITY;
        int at = 0x7fffffff;
#pragma unroll
        for (int j = 0; j < kMaxExperts / 64; ++j)
            if (64 * j < experts && v[j] > best) {
                best = v[j];
                at = lane + 64 * j;
            }
        const float m = wave_max(best);
        int who = best == m ? at : 0x7fffffff;
#pragma unroll
        for (int d = 1; d < 64; d <<= 1) who = min(who, __shfl_xor(who, d, 64));
        who = min(who, experts - 1);  // all logits NaN: still an expert
        if (lane == k) {
            mine = who;
            logit = m;
        }
#pragma unroll
        for (int j = 0; j < kMaxExperts / 64; ++j)
            if (lane + 64 * j == who) v[j] = -INFINITY;
    }
    score = sigmoid_f32(logit);
}

// ---- few rows --------------------------------------------------------------------------------------------
// A wave per (gate, up) row pair, over the concatenation of the row's experts and the shared one
template <typename T>
__global__ __launch_bounds__(256) void moe_up_kernel(MoeArgs a) {
    constexpr int E = Chunk<T>::N, U = 4;
    extern __shared__ __align__(16) unsigned char smem_raw[];
    T* xs = reinterpret_cast<T*>(smem_raw);  // [ld]
    __shared__ int idx[kMaxTop];
    __shared__ float score[kMaxTop], red[4];
    const int m = blockIdx.y, nc = a.ld / E, total = a.top * a.ff + a.sff, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (a.h) {
        for (int i = threadIdx.x; i < nc; i += 256) store_chunk(xs + i * E, load_chunk(static_cast<const T*>(a.h) + (int64_t)m * a.ld + i * E));
    }
    if (wave == 0) {
        int e;
        float s;
        pick_experts(a.logits + (int64_t)m * a.ldl, a.experts, a.top, e, s);
        if (lane < a.top) {
            idx[lane] = e;
            score[lane] = s;
            if (blockIdx.x == 0) a.pick[(int64_t)m * a.top + lane] = e;
        }
    }
    if (!a.h) {
        const float* x = a.x + (int64_t)m * a.ld;
        float ss = 0.f;
        for (int i = 4 * threadIdx.x; i < a.ld; i += 1024) {
            const f32x4 v = load4(x + i);
            ss += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
        }
        ss = wave_sum(ss);
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.dim + a.eps);
        for (int i = 4 * threadIdx.x; i < a.ld; i += 1024) store4(xs + i, load4(x + i) * inv * load4(a.norm + i));
    }
    __syncthreads();
    const int p = blockIdx.x * 4 + wave;
    if (p >= total) return;
    const bool shared = p >= a.top * a.ff;
    const int slot = shared ? 0 : p / a.ff, r = shared ? p - a.top * a.ff : p - slot * a.ff;
    const T* g = shared ? static_cast<const T*>(a.shared_up) + (int64_t)r * a.ld
                        : static_cast<const T*>(a.up) + ((int64_t)idx[slot] * 2 * a.ff + r) * a.ld;
    const T* u = g + (int64_t)(shared ? a.sff : a.ff) * a.ld;
    float sg = 0.f, su = 0.f;
    for (int c0 = lane; c0 < nc; c0 += 64 * U) {
        Chunk<T> vg[U], vu[U];
#pragma unroll
        for (int j = 0; j < U; ++j) {
            const int c = min(c0 + 64 * j, nc - 1);
            vg[j] = load_chunk_stream(g + c * E);
            vu[j] = load_chunk_stream(u + c * E);
        }
#pragma unroll
        for (int j = 0; j < U; ++j) {
            if (c0 + 64 * j >= nc) break;
            const Chunk<T> x = load_chunk(xs + (c0 + 64 * j) * E);
            sg = dot_chunk(vg[j], x, sg);
            su = dot_chunk(vu[j], x, su);
        }
    }
    sg = wave_sum(sg);
    su = wave_sum(su);
    if (lane != 0) return;
    const float s = shared ? 1.f : score[slot];
    float v = silu_f32(s * sg) * (s * su);
    if (shared) v *= sigmoid_f32(a.logits[(int64_t)m * a.ldl + a.experts]);
    static_cast<T*>(a.act)[(int64_t)m * total + p] = from_f32<T>(v);
}

// a wave per output channel: its row of every chosen down matrix and of the shared one, as one long row
template <typename T>
__global__ __launch_bounds__(256) void moe_down_kernel(MoeArgs a) {
    constexpr int E = Chunk<T>::N, U = 6;
    const int m = blockIdx.y, n = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (n >= a.ld) return;
    const int* pick = a.pick + (int64_t)m * a.top;
    const float x = a.x[(int64_t)m * a.ld + n];
    const int nf = a.ff / E, nr = a.top * nf, nc = nr + a.sff / E;
    const T* act = static_cast<const T*>(a.act) + (int64_t)m * nc * E;
    const T* down = static_cast<const T*>(a.down);
    const T* sdown = static_cast<const T*>(a.shared_down);
    float sum = 0.f;
    for (int c0 = lane; c0 < nc; c0 += 64 * U) {
        Chunk<T> w[U], v[U];
        int e[U];
#pragma unroll
        for (int j = 0; j < U; ++j) {
            const int c = min(c0 + 64 * j, nc - 1);
            v[j] = load_chunk(act + c * E);
            e[j] = c < nr ? pick[c / nf] : 0;
        }
#pragma unroll
        for (int j = 0; j < U; ++j) {
            const int c = min(c0 + 64 * j, nc - 1);
            w[j] = load_chunk_stream(c < nr ? down + ((int64_t)e[j] * a.ld + n) * a.ff + (c % nf) * E : sdown + (int64_t)n * a.sff + (c - nr) * E);
        }
#pragma unroll
        for (int j = 0; j < U; ++j)
            if (c0 + 64 * j < nc) sum = dot_chunk(w[j], v[j], sum);
    }
    sum = wave_sum(sum);
    if (lane == 0) a.x[(int64_t)m * a.ld + n] = x + sum;
}

// ---- chunks ----------------------------------------------------------------------------------------------
// Both sorting kernels give kPickRows tokens to a workgroup.  The first picks their experts (a wave per token in turn) and counts
// its pairs per expert; the second adds the counts up -- every workgroup for itself: they are few --, so that it knows where each
// expert's rows start and which of them are its own, and puts its pairs there.  Inside a workgroup's share of an expert the order is
// whatever the counters give: no result depends on it.
__global__ __launch_bounds__(1024) void moe_pick_kernel(MoeArgs a) {
    __shared__ int count[kMaxExperts];
    const int m0 = blockIdx.x * kPickRows, wave = threadIdx.x >> 6;
    for (int e = threadIdx.x; e < a.experts; e += 1024) count[e] = 0;
    __syncthreads();
    for (int i = wave; i < kPickRows && m0 + i < a.M; i += 16) {
        const int64_t m = m0 + i;
        const int lane = threadIdx.x & 63;
        int e;
        float s;
        pick_experts(a.logits + m * a.ldl, a.experts, a.top, e, s);
        if (lane < a.top) {
            a.pick[m * a.top + lane] = e;
            a.pick_scale[m * a.top + lane] = s;
            atomicAdd(&count[e], 1);
        }
    }
    __syncthreads();
    for (int e = threadIdx.x; e < a.experts; e += 1024) a.block_count[(int64_t)blockIdx.x * a.experts + e] = count[e];
}

__global__ __launch_bounds__(1024) void moe_sort_kernel(MoeArgs a) {
    __shared__ int before[kMaxExperts], total[kMaxExperts], wave_sums[2][16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, blocks = gridDim.x, me = blockIdx.x;
    before[tid] = total[tid] = 0;
    __syncthreads();
    const int counts = blocks * a.experts;
    for (int i0 = tid; i0 < counts; i0 += 4096) {
        int v[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = i0 + 1024 * j < counts ? a.block_count[i0 + 1024 * j] : 0;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (v[j] == 0) continue;
            const int i = i0 + 1024 * j, b = i / a.experts, e = i - b * a.experts;
            atomicAdd(&total[e], v[j]);
            if (b < me) atomicAdd(&before[e], v[j]);
        }
    }
    __syncthreads();
    // running sums over the experts of rows and of tile rows
    const int rows = total[tid], tiles = (rows + a.tile_rows - 1) / a.tile_rows;
    int r = rows, t = tiles;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
        const int pr = __shfl_up(r, d, 64), pt = __shfl_up(t, d, 64);
        if (lane >= d) {
            r += pr;
            t += pt;
        }
    }
    if (lane == 63) {
        wave_sums[0][wave] = r;
        wave_sums[1][wave] = t;
    }
    __syncthreads();
    for (int w = 0; w < wave; ++w) {
        r += wave_sums[0][w];
        t += wave_sums[1][w];
    }
    const int first = r - rows, first_tile = t - tiles;
    before[tid] += first;  // where this workgroup's rows of expert tid start
    if (me == 0) {
        for (int i = 0; i < tiles; ++i) {
            a.group_of[first_tile + i] = tid;
            a.group_row[first_tile + i] = first + i * a.tile_rows;
            a.group_end[first_tile + i] = min(first + (i + 1) * a.tile_rows, first + rows);
        }
        int used = 0;
        for (int w = 0; w < 16; ++w) used += wave_sums[1][w];
        for (int i = used + tid; i < a.n_tiles; i += 1024) a.group_of[i] = -1;
    }
    __syncthreads();
    const int lo = me * kPickRows * a.top, hi = min(a.M, (me + 1) * kPickRows) * a.top;
    for (int i = lo + tid; i < hi; i += 1024) {
        const int slot = atomicAdd(&before[a.pick[i]], 1);
        a.slot_of[i] = slot;
        a.slot_row[slot] = i / a.top;
        a.slot_scale[slot] = a.pick_scale[i];
    }
}

__global__ __launch_bounds__(256) void moe_combine_kernel(MoeArgs a) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    const int per = a.ld / 4;
    if (i >= (int64_t)a.M * per) return;
    const int m = (int)(i / per), c = 4 * (int)(i % per);
    f32x4 x = load4(a.x + (int64_t)m * a.ld + c);
    for (int k0 = 0; k0 < a.top; k0 += 4) {
        f32x4 v[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) v[k] = load4(a.y + (int64_t)a.slot_of[m * a.top + min(k0 + k, a.top - 1)] * a.ld + c);
#pragma unroll
        for (int k = 0; k < 4; ++k)
            if (k0 + k < a.top) x += v[k];
    }
    if (a.ys) x += load4(a.ys + (int64_t)m * a.ld + c) * sigmoid_f32(a.logits[(int64_t)m * a.ldl + a.experts]);
    store4(a.x + (int64_t)m * a.ld + c, x);
}

// rows from which a chunk's experts run as a grouped product: once they share weights (or there are enough rows anyway)
static bool moe_grouped(const raven_moe* m, int M, int dtype) {
    return dtype == RAVEN_BF16 && M > 8 && ((int64_t)M * m->top >= 2 * m->experts || M > 128);
}

struct MoeChunk {
    int *pick, *slot_of, *slot_row, *group_of, *group_row, *group_end, *block_count;
    bf16* y;
    float *pick_scale, *slot_scale, *ys;
    char *act, *sact, *lin;
    size_t lin_bytes;
    int n_tiles, tile_rows;
};
static size_t carve_moe(const raven_moe* m, int M, int ld, int dtype, char* base, MoeChunk* out) {
    const size_t es = raven_host::elt_size(dtype), pairs = (size_t)M * m->top;
    size_t off = 0;
    auto take = [&](size_t bytes) {
        char* p = base ? base + off : nullptr;
        off += raven_host::align_up(bytes);
        return p;
    };
    MoeChunk c{};
    if (!moe_grouped(m, M, dtype)) {
        c.act = take((size_t)M * (m->top * (size_t)m->ff + m->shared_ff) * es);
        c.pick = (int*)take(pairs * 4);
    } else {
        // 256-row tiles (twice the speed per row) once an expert fills most of two of them on average
        c.tile_rows = pairs >= (size_t)kBigTileRows * m->experts ? 256 : 128;
        c.n_tiles = (int)(pairs / c.tile_rows) + m->experts;
        c.pick = (int*)take(pairs * 4);
        c.pick_scale = (float*)take(pairs * 4);
        c.slot_of = (int*)take(pairs * 4);
        c.slot_row = (int*)take(pairs * 4);
        c.slot_scale = (float*)take(pairs * 4);
        c.group_of = (int*)take((size_t)c.n_tiles * 4);
        c.group_row = (int*)take((size_t)c.n_tiles * 4);
        c.group_end = (int*)take((size_t)c.n_tiles * 4);
        c.block_count = (int*)take((size_t)((M + kPickRows - 1) / kPickRows) * m->experts * 4);
        c.act = take(pairs * m->ff * es);
        c.y = (bf16*)take(pairs * ld * sizeof(bf16));
        if (m->shared_up) {
            c.sact = take((size_t)M * m->shared_ff * es);
            c.ys = (float*)take((size_t)M * ld * sizeof(float));
            c.lin_bytes = raven_linear_workspace_bytes(M, ld > 2 * m->shared_ff ? ld : 2 * m->shared_ff);
            c.lin = take(c.lin_bytes);
        }
    }
    if (out) *out = c;
    return off;
}

static int check_moe(const char* who, const raven_moe* m, int M, int ld, int dtype) {
    RAVEN_REQUIRE(dtype == RAVEN_F32 || dtype == RAVEN_BF16, "%s: unknown dtype %d", who, dtype);
    RAVEN_REQUIRE(m && m->experts > 0 && m->experts <= kMaxExperts && m->top > 0 && m->top <= m->experts && m->top <= kMaxTop, "%s: bad experts / top", who);
    RAVEN_REQUIRE(m->ff > 0 && m->ff % 8 == 0 && m->shared_ff >= 0 && m->shared_ff % 8 == 0 && ld > 0 && ld % 8 == 0 && M >= 0, "%s: bad sizes", who);
    RAVEN_REQUIRE(m->logit_ld >= m->experts + (m->shared_up ? 1 : 0), "%s: bad logit pitch %d", who, m->logit_ld);
    RAVEN_REQUIRE((m->shared_up == nullptr) == (m->shared_ff == 0) && (m->shared_up == nullptr) == (m->shared_down == nullptr), "%s: incomplete shared expert", who);
    return 0;
}

template <typename T>
static int run_moe_rows(const MoeArgs& a, hipStream_t s) {
    const size_t lds = (size_t)a.ld * sizeof(T);
    RAVEN_REQUIRE(lds <= 64 * 1024 - 1024, "moe: rows of %d channels do not fit the LDS", a.ld);
    const int total = a.top * a.ff + a.sff;
    moe_up_kernel<T><<<dim3((total + 3) / 4, a.M), dim3(256), lds, s>>>(a);
    moe_down_kernel<T><<<dim3((a.ld + 3) / 4, a.M), dim3(256), 0, s>>>(a);
    return raven_host::check_launch("moe (rows)");
}

}  // namespace raven

extern "C" size_t raven_moe_workspace_bytes(const raven_moe* m, int32_t M, int32_t ld, int32_t dtype) {
    if (raven::check_moe("moe_workspace_bytes", m, M, ld, dtype) || M == 0) return 0;
    return raven::carve_moe(m, M, ld, dtype, nullptr, nullptr);
}

namespace raven {
// h null (one row): moe_up_kernel norms the row of x itself
int moe_forward(const raven_moe* m, const void* h, const float* norm, int dim, float eps, const float* logits, float* x, int M, int ld, int dtype,
                void* workspace, size_t workspace_bytes, hipStream_t s) {
    if (const int rc = check_moe("moe", m, M, ld, dtype)) return rc;
    if (M == 0) return 0;
    RAVEN_REQUIRE(m->up && m->down && (h || (norm && M == 1)) && logits && x, "moe: null pointer");
    RAVEN_REQUIRE(workspace && ((uintptr_t)workspace & 255) == 0 && carve_moe(m, M, ld, dtype, nullptr, nullptr) <= workspace_bytes,
                  "moe: workspace of %zu bytes is too small or unaligned", workspace_bytes);
    MoeChunk c;
    carve_moe(m, M, ld, dtype, static_cast<char*>(workspace), &c);
    MoeArgs a{};
    a.h = h; a.up = m->up; a.down = m->down; a.shared_up = m->shared_up; a.shared_down = m->shared_down;
    a.logits = logits; a.x = x; a.act = c.act; a.norm = norm; a.dim = dim; a.eps = eps; a.pick = c.pick;
    a.M = M; a.ld = ld; a.ldl = m->logit_ld; a.experts = m->experts; a.top = m->top; a.ff = m->ff; a.sff = m->shared_ff;
    if (!moe_grouped(m, M, dtype)) {
        RAVEN_REQUIRE(M <= 65535, "moe: %d rows in one call", M);
        return dtype == RAVEN_BF16 ? run_moe_rows<bf16>(a, s) : run_moe_rows<float>(a, s);
    }
    const int pairs = M * m->top, blocks = (M + kPickRows - 1) / kPickRows;
    a.pick_scale = c.pick_scale; a.slot_of = c.slot_of; a.slot_row = c.slot_row; a.slot_scale = c.slot_scale;
    a.group_of = c.group_of; a.group_row = c.group_row; a.group_end = c.group_end; a.n_tiles = c.n_tiles; a.tile_rows = c.tile_rows; a.block_count = c.block_count;
    a.y = c.y; a.ys = c.ys;
    moe_pick_kernel<<<dim3(blocks), dim3(1024), 0, s>>>(a);
    moe_sort_kernel<<<dim3(blocks), dim3(1024), 0, s>>>(a);
    if (const int rc = raven_host::check_launch("moe (sort)")) return rc;
    if (const int rc = grouped_gemm(h, M, m->up, (int64_t)2 * m->ff * ld, c.act, pairs, m->ff, ld, 1, c.group_of, c.group_row, c.group_end, c.n_tiles, c.tile_rows, c.slot_row,
                                    c.slot_scale, s)) return rc;
    if (const int rc = grouped_gemm(c.act, pairs, m->down, (int64_t)ld * m->ff, c.y, pairs, ld, m->ff, 0, c.group_of, c.group_row, c.group_end, c.n_tiles, c.tile_rows, nullptr,
                                    nullptr, s)) return rc;
    if (m->shared_up) {
        raven_epilogue e{};
        e.scale = 1.f; e.out_f32 = 1;
        if (const int rc = raven_linear(h, nullptr, m->shared_up, nullptr, c.sact, M, m->shared_ff, ld, 0, 1, 0, dtype, c.lin, c.lin_bytes, s)) return rc;
        if (const int rc = raven_linear_epilogue(c.sact, nullptr, m->shared_down, c.ys, M, ld, m->shared_ff, 0, &e, dtype, c.lin, c.lin_bytes, s)) return rc;
    }
    moe_combine_kernel<<<dim3((unsigned)(((int64_t)M * (ld / 4) + 255) / 256)), dim3(256), 0, s>>>(a);
    return raven_host::check_launch("moe (combine)");
}
}  // namespace raven

extern "C" int raven_moe_forward(const raven_moe* m, const void* h, const float* logits, float* x, int32_t M, int32_t ld, int32_t dtype,
                                 void* workspace, size_t workspace_bytes, void* stream) {
    RAVEN_REQUIRE(h || M == 0, "moe: null pointer");
    return raven::moe_forward(m, h, nullptr, 0, 0.f, logits, x, M, ld, dtype, workspace, workspace_bytes, static_cast<hipStream_t>(stream));
}
