// One pre-norm layer of a decoder with an fp32 residual stream and a choice of mixers, as a sequence of this library's kernels
// on one stream: norm (+ convolution) -> fused input projection -> mixer -> output projection added to the stream ->
// norm -> up + gelu -> down added to the stream.  The residual adds and the activation ride in the products' epilogues.

#include "raven_common.h"

namespace raven {

struct MixerScratch {
    char *h, *z, *low, *y, *ff;
    float* decay;
    char *attn_ws, *delta_ws, *lin_ws;
    size_t attn_ws_bytes, delta_ws_bytes, lin_ws_bytes;
};

bool gemv1_stream_fits(int K, int dtype);
int gemv1_stream(const float* x, const float* norm, int dim, float eps, const void* w, void* y, int N, int K, const raven_epilogue& epi, int dtype,
                 hipStream_t s);

static size_t carve_mixer(const raven_stream_dims* d, const raven_mixer_layer* l, int B, int S, char* base, MixerScratch* out) {
    const size_t es = raven_host::elt_size(d->dtype);
    const size_t M = (size_t)B * S;
    const size_t inner = (size_t)l->heads * l->head_dim;
    const bool delta = l->mixer == RAVEN_MIXER_GENERAL_DELTA;
    size_t off = 0;
    auto take = [&](size_t bytes) {
        char* p = base ? base + off : nullptr;
        off += raven_host::align_up(bytes);
        return p;
    };
    MixerScratch s{};
    s.h = take(M * d->ld * es);
    s.z = take(delta ? M * (5 * inner + l->rank) * sizeof(float) : M * (l->heads + l->kv_heads) * l->head_dim * es);
    s.low = take(delta ? M * l->rank * es : 0);
    s.decay = reinterpret_cast<float*>(take(delta ? M * inner * sizeof(float) : 0));
    s.y = take(M * inner * es);
    s.ff = take(l->up ? M * l->ff * es : 0);
    s.attn_ws_bytes = delta ? 0 : raven_capped_attention_workspace_bytes((int)M, l->heads, l->kv_heads, l->head_dim);
    s.attn_ws = take(s.attn_ws_bytes);
    s.delta_ws_bytes = delta ? raven_delta_rule_workspace_bytes(B, S, l->heads, l->head_dim) : 0;
    s.delta_ws = take(s.delta_ws_bytes);
    size_t widest = delta ? 5 * inner + l->rank : (size_t)(l->heads + l->kv_heads) * l->head_dim;
    if ((size_t)d->ld > widest) widest = d->ld;
    if (l->up && (size_t)l->ff > widest) widest = l->ff;
    s.lin_ws_bytes = M > 1 ? raven_linear_workspace_bytes((int)M, (int)widest) : 0;
    s.lin_ws = take(s.lin_ws_bytes);
    if (out) *out = s;
    return off;
}

static int check_mixer_layer(const char* who, const raven_stream_dims* d, const raven_mixer_layer* l) {
    RAVEN_REQUIRE(d && l, "%s: null pointer", who);
    RAVEN_REQUIRE(d->dtype == RAVEN_F32 || d->dtype == RAVEN_BF16, "%s: unknown dtype %d", who, d->dtype);
    RAVEN_REQUIRE(d->width > 0 && d->ld >= d->width && d->ld % 8 == 0, "%s: bad width %d / ld %d", who, d->width, d->ld);
    RAVEN_REQUIRE(l->mixer == RAVEN_MIXER_ATTENTION || l->mixer == RAVEN_MIXER_GENERAL_DELTA, "%s: unknown mixer %d", who, l->mixer);
    RAVEN_REQUIRE(l->heads > 0 && l->dim > 0 && l->head_dim >= l->dim && l->head_dim % 8 == 0, "%s: bad heads %d / dim %d / head_dim %d", who, l->heads,
                  l->dim, l->head_dim);
    RAVEN_REQUIRE(l->norm1 && l->w_in && l->w_out, "%s: null weight", who);
    if (l->mixer == RAVEN_MIXER_GENERAL_DELTA)
        RAVEN_REQUIRE(l->w_decay && l->decay_bias && l->a_bias && l->out_norm && l->rank > 0 && l->rank % 8 == 0,
                      "%s: the delta rule needs its decay and output weights (rank %d)", who, l->rank);
    RAVEN_REQUIRE((l->up == nullptr) == (l->down == nullptr) && (l->up == nullptr || (l->norm2 && l->ff > 0 && l->ff % 8 == 0)),
                  "%s: a feed-forward needs norm2, up, down and ff a multiple of 8 (ff %d)", who, l->ff);
    return 0;
}

}  // namespace raven

extern "C" size_t raven_mixer_layer_workspace_bytes(const raven_stream_dims* dims, const raven_mixer_layer* layer, int32_t B, int32_t S) {
    if (B <= 0 || S <= 0 || raven::check_mixer_layer("mixer_layer_workspace_bytes", dims, layer)) return 0;
    return raven::carve_mixer(dims, layer, B, S, nullptr, nullptr);
}

extern "C" int raven_mixer_layer_forward(const raven_stream_dims* dims, const raven_mixer_layer* layer, const raven_mixer_state* state, float* x,
                                         int32_t B, int32_t S, int32_t pos0, const int32_t* pos_dev, void* workspace,
                                         size_t workspace_bytes, void* stream) {
    using namespace raven;
    if (const int rc = check_mixer_layer("mixer_layer", dims, layer)) return rc;
    RAVEN_REQUIRE(B >= 0 && S >= 0 && (int64_t)B * S < (1 << 30), "mixer_layer: bad B=%d S=%d", B, S);
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(state && x && workspace && ((uintptr_t)workspace & 255) == 0, "mixer_layer: null pointer or unaligned workspace");
    RAVEN_REQUIRE(carve_mixer(dims, layer, B, S, nullptr, nullptr) <= workspace_bytes, "mixer_layer: workspace of %zu bytes is too small",
                  workspace_bytes);
    MixerScratch w;
    carve_mixer(dims, layer, B, S, static_cast<char*>(workspace), &w);
    const raven_mixer_layer& l = *layer;
    const int M = B * S, dt = dims->dtype, ld = dims->ld, inner = l.heads * l.head_dim;

    auto product = [&](const void* in, const void* wt, void* y, int N, int K, int act, const float* bias, const float* residual, int out_f32) {
        raven_epilogue e{};
        e.bias = bias; e.residual = residual; e.scale = 1.f; e.act = act; e.out_f32 = out_f32;
        return raven_linear_epilogue(in, nullptr, wt, y, M, N, K, 0, &e, dt, w.lin_ws, w.lin_ws_bytes, stream);
    };
    if (int rc = raven_norm_conv(x, l.norm1, l.conv, state->ring, w.h, B, S, dims->width, ld, l.taps, dims->eps, pos0, pos_dev, dt, stream)) return rc;
    if (l.mixer == RAVEN_MIXER_ATTENTION) {
        if (int rc = product(w.h, l.w_in, w.z, (l.heads + l.kv_heads) * l.head_dim, ld, RAVEN_ACT_NONE, nullptr, nullptr, 0)) return rc;
        if (int rc = raven_capped_attention(w.z, w.y, &state->keys, &l.score, B, S, pos0, pos_dev, l.heads, dt, w.attn_ws, w.attn_ws_bytes, stream)) return rc;
    } else {
        // a few tokens: the low-rank rows ride in the fused projection and the recurrence's kernel forms the decay logits;
        // more: two small products of their own
        const bool few = S <= 8 && l.rank <= 256;
        const int ldz = 5 * inner + (few ? l.rank : 0);
        if (int rc = product(w.h, l.w_in, w.z, ldz, ld, RAVEN_ACT_NONE, nullptr, nullptr, 1)) return rc;
        if (!few) {
            const char* w_low = static_cast<const char*>(l.w_in) + (size_t)5 * inner * ld * raven_host::elt_size(dt);
            if (int rc = product(w.h, w_low, w.low, l.rank, ld, RAVEN_ACT_TANH, nullptr, nullptr, 0)) return rc;
            if (int rc = product(w.low, l.w_decay, w.decay, inner, l.rank, RAVEN_ACT_NONE, l.decay_bias, nullptr, 1)) return rc;
        }
        if (int rc = raven_delta_rule(reinterpret_cast<float*>(w.z), ldz, few ? nullptr : w.decay, l.w_decay, l.decay_bias, l.rank, l.a_bias,
                                      l.out_norm, state->state, w.y, B, S, pos0, pos_dev, l.heads, l.dim, l.head_dim, dims->eps, dt, w.delta_ws,
                                      w.delta_ws_bytes, stream)) return rc;
    }
    if (int rc = product(w.y, l.w_out, x, ld, inner, RAVEN_ACT_NONE, nullptr, x, 1)) return rc;
    if (l.up && M == 1 && gemv1_stream_fits(ld, dt)) {  // the norm rides in the product's prologue
        raven_epilogue e{};
        e.scale = 1.f; e.act = RAVEN_ACT_GELU;
        if (int rc = gemv1_stream(x, l.norm2, dims->width, dims->eps, l.up, w.ff, l.ff, ld, e, dt, static_cast<hipStream_t>(stream))) return rc;
        if (int rc = product(w.ff, l.down, x, ld, l.ff, RAVEN_ACT_NONE, nullptr, x, 1)) return rc;
    } else if (l.up) {
        if (int rc = raven_norm_conv(x, l.norm2, nullptr, nullptr, w.h, B, S, dims->width, ld, 1, dims->eps, pos0, pos_dev, dt, stream)) return rc;
        if (int rc = product(w.h, l.up, w.ff, l.ff, ld, RAVEN_ACT_GELU, nullptr, nullptr, 0)) return rc;
        if (int rc = product(w.ff, l.down, x, ld, l.ff, RAVEN_ACT_NONE, nullptr, x, 1)) return rc;
    }
    return 0;
}
