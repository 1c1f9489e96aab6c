// One pre-norm layer of a decoder with an fp32 residual stream and a choice of mixers and feed-forwards, as a sequence of this
// library's kernels on one stream: norm (+ convolution) -> fused input projection -> mixer -> output projection added to the
// stream -> norm -> feed-forward added to the stream.  Residual adds and activations ride in the products' epilogues, norms of a
// single row in their prologues.
//
// The mixers' entry points are referenced weakly: a build of one model family's kernels links without the others', and a layer
// that needs a missing one is refused.

#include "raven_common.h"

#define RAVEN_WEAK __attribute__((weak))
extern "C" {
RAVEN_WEAK decltype(raven_capped_attention_workspace_bytes) raven_capped_attention_workspace_bytes;
RAVEN_WEAK decltype(raven_capped_attention) raven_capped_attention;
RAVEN_WEAK decltype(raven_delta_rule_workspace_bytes) raven_delta_rule_workspace_bytes;
RAVEN_WEAK decltype(raven_delta_rule) raven_delta_rule;
RAVEN_WEAK decltype(raven_latent_rows) raven_latent_rows;
RAVEN_WEAK decltype(raven_latent_attention_workspace_bytes) raven_latent_attention_workspace_bytes;
RAVEN_WEAK decltype(raven_rglru_workspace_bytes) raven_rglru_workspace_bytes;
RAVEN_WEAK decltype(raven_rglru_forward) raven_rglru_forward;
RAVEN_WEAK decltype(raven_moe_workspace_bytes) raven_moe_workspace_bytes;
}

namespace raven {

RAVEN_WEAK int latent_attention(const raven_latent* l, const void* q, const void* z, int ldz, int z_f32, const raven_latent_cache* cache, void* y, int B,
                                int S, int pos0, const int* pos_dev, int append, int dtype, void* workspace, size_t workspace_bytes, hipStream_t s);

RAVEN_WEAK int moe_forward(const raven_moe* m, const void* h, const float* norm, int dim, float eps, const float* logits, float* x, int M, int ld, int dtype,
                           void* workspace, size_t workspace_bytes, hipStream_t s);

bool gemv1_stream_fits(int K, int dtype);
int gemv1_stream(const float* x, const float* norm, int dim, float eps, const void* w, void* y, int N, int K, const raven_epilogue& epi, int dtype,
                 hipStream_t s);
int gemv1_stream_swiglu(const float* x, const float* norm, int dim, float eps, const void* w, void* y, int N, int K, int dtype, hipStream_t s);

struct MixerScratch {
    char *h, *z, *low, *y, *ff;  // low: the decay's low-rank rows / the normed query latents
    char* q;
    float *decay, *logits;
    char *mix_ws, *ff_ws, *lin_ws;
    size_t mix_ws_bytes, ff_ws_bytes, lin_ws_bytes;
};

// columns of the fused input projection
static int input_columns(const raven_mixer_layer* l) {
    switch (l->mixer) {
        case RAVEN_MIXER_ATTENTION: return (l->heads + l->kv_heads) * l->head_dim;
        case RAVEN_MIXER_GENERAL_DELTA: return 5 * l->heads * l->head_dim + l->rank;
        case RAVEN_MIXER_LATENT: return l->latent->q_rank + (l->latent->own_kv ? l->latent->kv_rank + l->latent->rot : 0) + l->latent->heads * l->latent->vdim;
        default: return 2 * l->rglru->width;
    }
}

static size_t carve_mixer(const raven_stream_dims* d, const raven_mixer_layer* l, int B, int S, int pos0, char* base, MixerScratch* out) {
    const size_t es = raven_host::elt_size(d->dtype);
    const size_t M = (size_t)B * S;
    const size_t inner = (size_t)l->heads * l->head_dim, z_cols = input_columns(l);
    const bool delta = l->mixer == RAVEN_MIXER_GENERAL_DELTA, latent = l->mixer == RAVEN_MIXER_LATENT;
    const bool moe = l->ff_kind == RAVEN_FF_MOE && l->moe, ff = !moe && l->up;
    size_t off = 0;
    auto take = [&](size_t bytes) {
        char* p = base ? base + off : nullptr;
        off += raven_host::align_up(bytes);
        return p;
    };
    const size_t q_cols = latent ? (size_t)l->latent->heads * (l->latent->nope + l->latent->rot) : 0;
    MixerScratch s{};
    s.h = take(M * d->ld * es);
    s.z = take(M * z_cols * (delta || (latent && M == 1) ? sizeof(float) : es));
    s.low = take(delta ? M * l->rank * es : latent ? M * l->latent->q_rank * es : 0);
    s.q = take(M * q_cols * es);
    s.decay = reinterpret_cast<float*>(take(delta ? M * inner * sizeof(float) : 0));
    s.y = take(M * inner * es);
    s.ff = take(ff ? M * l->ff * es : 0);
    s.logits = reinterpret_cast<float*>(take(moe ? M * l->moe->logit_ld * sizeof(float) : 0));
    switch (l->mixer) {
        case RAVEN_MIXER_ATTENTION: s.mix_ws_bytes = raven_capped_attention_workspace_bytes((int)M, l->heads, l->kv_heads, l->head_dim); break;
        case RAVEN_MIXER_GENERAL_DELTA: s.mix_ws_bytes = raven_delta_rule_workspace_bytes(B, S, l->heads, l->head_dim); break;
        case RAVEN_MIXER_LATENT: s.mix_ws_bytes = raven_latent_attention_workspace_bytes(l->latent, B, S, pos0, d->dtype); break;
        default: s.mix_ws_bytes = raven_rglru_workspace_bytes(l->rglru, B, S, d->dtype);
    }
    s.mix_ws = take(s.mix_ws_bytes);
    s.ff_ws_bytes = moe ? raven_moe_workspace_bytes(l->moe, (int)M, d->ld, d->dtype) : 0;
    s.ff_ws = take(s.ff_ws_bytes);
    size_t widest = z_cols > q_cols ? z_cols : q_cols;
    if ((size_t)d->ld > widest) widest = d->ld;
    if (ff && (size_t)l->ff * 2 > widest) widest = (size_t)l->ff * 2;
    if (moe && (size_t)l->moe->logit_ld > widest) widest = l->moe->logit_ld;
    s.lin_ws_bytes = M > 1 ? raven_linear_workspace_bytes((int)M, (int)widest) : 0;
    s.lin_ws = take(s.lin_ws_bytes);
    if (out) *out = s;
    return off;
}

static int check_mixer_layer(const char* who, const raven_stream_dims* d, const raven_mixer_layer* l) {
    RAVEN_REQUIRE(d && l, "%s: null pointer", who);
    RAVEN_REQUIRE(d->dtype == RAVEN_F32 || d->dtype == RAVEN_BF16, "%s: unknown dtype %d", who, d->dtype);
    RAVEN_REQUIRE(d->width > 0 && d->ld >= d->width && d->ld % 8 == 0, "%s: bad width %d / ld %d", who, d->width, d->ld);
    RAVEN_REQUIRE(l->mixer >= RAVEN_MIXER_ATTENTION && l->mixer <= RAVEN_MIXER_RGLRU, "%s: unknown mixer %d", who, l->mixer);
    RAVEN_REQUIRE(l->heads > 0 && l->dim > 0 && l->head_dim >= l->dim && l->head_dim % 8 == 0, "%s: bad heads %d / dim %d / head_dim %d", who, l->heads,
                  l->dim, l->head_dim);
    RAVEN_REQUIRE(l->norm1 && l->w_in && l->w_out, "%s: null weight", who);
    switch (l->mixer) {
        case RAVEN_MIXER_ATTENTION: RAVEN_REQUIRE(&raven_capped_attention, "%s: this build lacks capped attention", who); break;
        case RAVEN_MIXER_GENERAL_DELTA:
            RAVEN_REQUIRE(&raven_delta_rule, "%s: this build lacks the delta rule", who);
            RAVEN_REQUIRE(l->w_decay && l->decay_bias && l->a_bias && l->out_norm && l->rank > 0 && l->rank % 8 == 0,
                          "%s: the delta rule needs its decay and output weights (rank %d)", who, l->rank);
            break;
        case RAVEN_MIXER_LATENT:
            RAVEN_REQUIRE(&raven_latent_rows && &latent_attention, "%s: this build lacks latent attention", who);
            RAVEN_REQUIRE(l->latent && l->latent->w_uq && l->heads == l->latent->heads && l->head_dim == l->latent->vdim, "%s: bad latent attention", who);
            break;
        default:
            RAVEN_REQUIRE(&raven_rglru_forward, "%s: this build lacks the recurrent unit", who);
            RAVEN_REQUIRE(l->rglru && l->in_bias && l->heads * l->head_dim == l->rglru->width, "%s: bad recurrent unit", who);
    }
    RAVEN_REQUIRE(l->ff_kind >= RAVEN_FF_GELU && l->ff_kind <= RAVEN_FF_MOE, "%s: unknown feed-forward %d", who, l->ff_kind);
    if (l->ff_kind == RAVEN_FF_MOE) {
        RAVEN_REQUIRE(&raven_moe_workspace_bytes && &moe_forward, "%s: this build lacks the mixture of experts", who);
        RAVEN_REQUIRE(l->moe && l->moe->router && l->norm2, "%s: bad mixture of experts", who);
    } else {
        RAVEN_REQUIRE((l->up == nullptr) == (l->down == nullptr) && (l->up == nullptr || (l->norm2 && l->ff > 0 && l->ff % 8 == 0)),
                      "%s: a feed-forward needs norm2, up, down and ff a multiple of 8 (ff %d)", who, l->ff);
    }
    return 0;
}

}  // namespace raven

extern "C" size_t raven_mixer_layer_workspace_bytes(const raven_stream_dims* dims, const raven_mixer_layer* layer, int32_t B, int32_t S, int32_t pos0) {
    if (B <= 0 || S <= 0 || raven::check_mixer_layer("mixer_layer_workspace_bytes", dims, layer)) return 0;
    return raven::carve_mixer(dims, layer, B, S, pos0, nullptr, nullptr);
}

extern "C" int raven_mixer_layer_forward(const raven_stream_dims* dims, const raven_mixer_layer* layer, const raven_mixer_state* state, float* x,
                                         int32_t B, int32_t S, int32_t pos0, const int32_t* pos_dev, void* workspace,
                                         size_t workspace_bytes, void* stream) {
    using namespace raven;
    if (const int rc = check_mixer_layer("mixer_layer", dims, layer)) return rc;
    RAVEN_REQUIRE(B >= 0 && S >= 0 && (int64_t)B * S < (1 << 30), "mixer_layer: bad B=%d S=%d", B, S);
    if (B == 0 || S == 0) return 0;
    RAVEN_REQUIRE(state && x && workspace && ((uintptr_t)workspace & 255) == 0, "mixer_layer: null pointer or unaligned workspace");
    RAVEN_REQUIRE(carve_mixer(dims, layer, B, S, pos0, nullptr, nullptr) <= workspace_bytes, "mixer_layer: workspace of %zu bytes is too small",
                  workspace_bytes);
    MixerScratch w;
    carve_mixer(dims, layer, B, S, pos0, static_cast<char*>(workspace), &w);
    const raven_mixer_layer& l = *layer;
    const int M = B * S, dt = dims->dtype, ld = dims->ld, inner = l.heads * l.head_dim;
    hipStream_t s = static_cast<hipStream_t>(stream);

    auto product = [&](const void* in, const void* wt, void* y, int N, int K, int act, const float* bias, const float* residual, int out_f32) {
        raven_epilogue e{};
        e.bias = bias; e.residual = residual; e.scale = 1.f; e.act = act; e.out_f32 = out_f32;
        return raven_linear_epilogue(in, nullptr, wt, y, M, N, K, 0, &e, dt, w.lin_ws, w.lin_ws_bytes, stream);
    };
    const bool one_row = M == 1 && gemv1_stream_fits(ld, dt);
    // a product behind an RMSNorm of the stream: one row takes the norm as its prologue, more go through w.h
    auto normed_product = [&](const float* norm, const void* wt, void* y, int N, int act, const float* bias, int out_f32) {
        if (one_row) {
            raven_epilogue e{};
            e.bias = bias; e.scale = 1.f; e.act = act; e.out_f32 = out_f32;
            return gemv1_stream(x, norm, dims->width, dims->eps, wt, y, N, ld, e, dt, s);
        }
        if (int rc = raven_norm_conv(x, norm, nullptr, nullptr, w.h, B, S, dims->width, ld, 1, dims->eps, pos0, pos_dev, dt, stream)) return rc;
        return product(w.h, wt, y, N, ld, act, bias, nullptr, out_f32);
    };

    if (l.mixer == RAVEN_MIXER_ATTENTION) {
        if (int rc = raven_norm_conv(x, l.norm1, l.conv, state->ring, w.h, B, S, dims->width, ld, l.taps, dims->eps, pos0, pos_dev, dt, stream)) return rc;
        if (int rc = product(w.h, l.w_in, w.z, (l.heads + l.kv_heads) * l.head_dim, ld, RAVEN_ACT_NONE, nullptr, nullptr, 0)) return rc;
        if (int rc = raven_capped_attention(w.z, w.y, &state->keys, &l.score, B, S, pos0, pos_dev, l.heads, dt, w.mix_ws, w.mix_ws_bytes, stream)) return rc;
    } else if (l.mixer == RAVEN_MIXER_GENERAL_DELTA) {
        if (int rc = raven_norm_conv(x, l.norm1, l.conv, state->ring, w.h, B, S, dims->width, ld, l.taps, dims->eps, pos0, pos_dev, dt, stream)) return rc;
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
                                      l.out_norm, state->state, w.y, B, S, pos0, pos_dev, l.heads, l.dim, l.head_dim, dims->eps, dt, w.mix_ws,
                                      w.mix_ws_bytes, stream)) return rc;
    } else if (l.mixer == RAVEN_MIXER_LATENT) {
        const raven_latent& a = *l.latent;
        const int ldz = input_columns(layer), q_cols = a.heads * (a.nope + a.rot), z_f32 = M == 1 || dt == RAVEN_F32;
        if (int rc = normed_product(l.norm1, l.w_in, w.z, ldz, RAVEN_ACT_NONE, nullptr, z_f32)) return rc;
        const bool fold = M == 1 && gemv1_stream_fits(a.q_rank, dt);  // the query latent's norm rides in W_uq, the cache entry in the attention
        if (fold) {
            raven_epilogue e{};
            e.scale = 1.f;
            if (int rc = gemv1_stream(reinterpret_cast<float*>(w.z), a.q_norm, a.q_dim, a.eps, a.w_uq, w.q, q_cols, a.q_rank, e, dt, s)) return rc;
        } else {
            if (int rc = raven_latent_rows(&a, w.z, ldz, z_f32, &state->latent, w.low, B, S, pos0, pos_dev, dt, stream)) return rc;
            if (int rc = product(w.low, a.w_uq, w.q, q_cols, a.q_rank, RAVEN_ACT_NONE, nullptr, nullptr, 0)) return rc;
        }
        if (int rc = latent_attention(&a, w.q, w.z, ldz, z_f32, &state->latent, w.y, B, S, pos0, pos_dev, fold, dt, w.mix_ws, w.mix_ws_bytes, s)) return rc;
    } else {
        if (int rc = normed_product(l.norm1, l.w_in, w.z, 2 * inner, RAVEN_ACT_NONE, l.in_bias, 0)) return rc;
        if (int rc = raven_rglru_forward(l.rglru, w.z, state->ring, state->state, w.y, B, S, pos0, pos_dev, dt, w.mix_ws, w.mix_ws_bytes, stream)) return rc;
    }
    if (int rc = product(w.y, l.w_out, x, ld, inner, RAVEN_ACT_NONE, nullptr, x, 1)) return rc;

    if (l.ff_kind == RAVEN_FF_MOE) {
        // (one row: the norm rides in the router's product and again in the experts' first one; else it lies in w.h)
        if (int rc = normed_product(l.norm2, l.moe->router, w.logits, l.moe->logit_ld, RAVEN_ACT_NONE, nullptr, 1)) return rc;
        return moe_forward(l.moe, one_row ? nullptr : w.h, l.norm2, dims->width, dims->eps, w.logits, x, M, ld, dt, w.ff_ws, w.ff_ws_bytes, s);
    }
    if (!l.up) return 0;
    if (l.ff_kind == RAVEN_FF_SWIGLU) {
        if (one_row) {
            if (int rc = gemv1_stream_swiglu(x, l.norm2, dims->width, dims->eps, l.up, w.ff, l.ff, ld, dt, s)) return rc;
        } else {
            if (int rc = raven_norm_conv(x, l.norm2, nullptr, nullptr, w.h, B, S, dims->width, ld, 1, dims->eps, pos0, pos_dev, dt, stream)) return rc;
            if (int rc = raven_linear(w.h, nullptr, l.up, nullptr, w.ff, M, l.ff, ld, 0, 1, 0, dt, w.lin_ws, w.lin_ws_bytes, stream)) return rc;
        }
    } else {
        if (int rc = normed_product(l.norm2, l.up, w.ff, l.ff, RAVEN_ACT_GELU, nullptr, 0)) return rc;
    }
    return product(w.ff, l.down, x, ld, l.ff, RAVEN_ACT_NONE, nullptr, x, 1);
}
