// The Suvazen decoder: a residual stream in f32 into which every sublayer's result enters through a layer norm of its
// own, windowed attention whose values are the unrotated keys, a squared-ReLU feed-forward, and a range of layers that
// runs several times with the same weights (a cache for each pass).  The norms between two sublayers are one launch
// (prompts, f32) or the prologue of the next contraction (bfloat16 decode step).  Step, prompt, cache and generation
// around the layers: decoder.hip.
#include <algorithm>
#include <cstring>
#include <vector>

#include "decoder.h"
#include "dense.h"

struct candy_hip_suvazen final : candy_hip_decoder {
    candy_hip_suvazen_config cfg{};
    struct Layer {
        candy_hip_suvazen_layer c{};
        const candy_hip_dense *qk = nullptr, *o = nullptr, *up = nullptr, *down = nullptr;
        float *norm[8] = {};   // in the order of enum candy_hip_suvazen_vector
        float *sink = nullptr;
        const float *cos_t = nullptr, *sin_t = nullptr;
        int n_splits = 1;
    };
    struct Run {               // one pass through one layer; run r has cache part r
        int layer;
        int step;              // row added in front of it, or -1
    };
    std::vector<Layer> layers;
    std::vector<Run> runs;
    std::vector<float *> steps;
    float *final_w = nullptr, *final_b = nullptr;
    const candy_hip_dense *head = nullptr, *embed_w = nullptr;
    bool f32 = false;
    int max_qk = 0, max_att = 0, max_ff = 0, max_q = 0;   // widest rows over the layers, padded
    size_t max_part = 0;

    struct Buffers {           // n rows each
        float *x = nullptr, *x2 = nullptr, *x3 = nullptr, *qk = nullptr, *y = nullptr;
        void *act = nullptr, *q = nullptr, *att = nullptr, *ff = nullptr;
        float *part = nullptr;
    };
    Buffers dec, pf;
    int *row_ids = nullptr;    // rows a prompt pass wants logits of
    size_t row_ids_cap = 0;

    size_t act_bytes() const { return f32 ? 4 : 2; }
    int check_complete() const override;
    bool has_embedding() const override { return embed_w != nullptr; }
    int embed(const int64_t *dev_ids, int64_t n, float *out) override {
        return candy::launch_dense_gather(dev, embed_w, dev_ids, n, out, width_pad);
    }
    int enqueue_step() override;
    int reserve_prompt(int n) override;
    int enqueue_prompt(int n, int pos0) override;
    const float *prompt_hidden() const override { return pf.x; }
    int enqueue_head() override;
    int enqueue_head_rows(const int32_t *rows, int n_rows, float *out) override;

    template <class Alloc>
    int alloc_buffers(Buffers &B, int n, Alloc alloc);
    candy::NormArgs norm_args(Buffers &B, int n) const;
    candy::WindowAttn attn_args(Buffers &B, int run) const;
    int layers_forward(Buffers &B, int n, int pos0, const int *pos_ptr, float *x_final, const candy::DenseLaunch *last);
    candy::DenseLaunch head_launch(const void *x, int n, float *out) const;
};

using namespace candy;

template <class Alloc>
int candy_hip_suvazen::alloc_buffers(Buffers &B, int n, Alloc alloc) {
    const size_t N = (size_t)n, es = act_bytes();
    auto bytes = [&](void **p, size_t b) {
        uint8_t *t = nullptr;
        const int rc = alloc(&t, b);
        *p = t;
        return rc;
    };
    int rc = CANDY_HIP_OK;
    const bool step = &B == &dec;
    if (!step && !rc) rc = bytes((void **)&B.x, N * width_pad * 4);
    if (step && !rc) rc = bytes((void **)&B.x2, N * width_pad * 4);
    if (step && !rc) rc = bytes((void **)&B.x3, N * width_pad * 4);
    if (!rc) rc = bytes((void **)&B.qk, N * max_qk * 4);
    if (!rc) rc = bytes((void **)&B.y, N * width_pad * 4);
    if (!rc) rc = bytes(&B.act, N * width_pad * es);
    if (!rc) rc = bytes(&B.q, N * max_q * es);
    if (!rc) rc = bytes(&B.att, N * max_att * es);
    if (!rc) rc = bytes(&B.ff, N * std::max(max_ff, 64) * es);
    if (step && !rc) rc = bytes((void **)&B.part, max_part * 4);
    return rc;
}

int candy_hip_suvazen::reserve_prompt(int n) {
    return alloc_buffers(pf, n, [this](uint8_t **p, size_t b) { return prompt_alloc(this, p, b); });
}

NormArgs candy_hip_suvazen::norm_args(Buffers &B, int n) const {
    NormArgs A;
    A.x = B.x; A.ldx = width_pad; A.eps = cfg.norm_eps; A.rows = n; A.cols = width; A.f32 = f32;
    A.out = B.act; A.ldo = width_pad; A.mult = cfg.residual_mult;
    return A;
}

WindowAttn candy_hip_suvazen::attn_args(Buffers &B, int run) const {
    const Layer &L = layers[(size_t)runs[(size_t)run].layer];
    WindowAttn A;
    A.s = L.c.attn;
    A.row = candy_hip_attn_row(A.s.head_dim);
    A.max_pos = max_pos; A.f32 = f32;
    A.cos_t = L.cos_t; A.sin_t = L.sin_t; A.sink = L.c.has_sink ? L.sink : nullptr;
    A.k_cache = cache.k_of(run); A.v_cache = cache.v_of(run);
    A.q = B.q; A.part = B.part; A.n_splits = L.n_splits;
    A.out = B.att; A.ldo = L.o->ld; A.out_cols = (int)L.o->ld;
    return A;
}

// The layers over n rows whose residual stream is in B.x; it ends in x_final, and `last`, if any, contracts the final
// norm of it.  pos_ptr: one token, its position in device memory; otherwise positions pos0 ...  The result of a
// contraction enters the residual sum in the norm that follows it.
int candy_hip_suvazen::layers_forward(Buffers &B, int n, int pos0, const int *pos_ptr, float *x_final, const DenseLaunch *last) {
    int rc;
    // what the next norm still has to add: a projection's result and the norm it passes through
    Partial pending;
    const float *post_w = nullptr, *post_b = nullptr;
    const bool fuse = pos_ptr && !f32;  // decode step: the norms in the contraction's prologue
    float *const own[2] = {B.x2, B.x3};   // decode: the stream alternates between these two
    auto elsewhere = [&] { return fuse ? own[B.x == own[0]] : B.x; };
    // x <- x + (pending) + step, written to `to` if anything is added; then `next` contracts the norm of it
    auto norm_then = [&](const float *w, const float *b, const float *step, const DenseLaunch *next, float *to) -> int {
        NormArgs A = norm_args(B, n);
        if (pending.p) { A.y = pending; A.post_w = post_w; A.post_b = post_b; }
        A.step = step;
        if (pending.p || step) A.x_out = to;
        A.pre_w = w; A.pre_b = b;
        if (!w) A.out = nullptr;
        pending = Partial{};
        int e = CANDY_HIP_ERR_UNSUPPORTED;
        // every workgroup of the fused launch reads the old row: the new one goes elsewhere
        if (next && fuse && A.x_out != A.x) e = launch_dense_norm(dev, *next, A);
        if (e == CANDY_HIP_ERR_UNSUPPORTED) {
            e = A.out || A.x_out ? launch_norm_chain(dev, A) : CANDY_HIP_OK;
            if (!e && next) e = launch_dense(dev, *next);
        }
        if (A.x_out) B.x = A.x_out;
        return e;
    };
    auto linear = [&](const candy_hip_dense *w, const void *x, int64_t ldx, int epi, void *y, int64_t ldy, Partial *partial) {
        DenseLaunch D;
        D.w = w; D.x = x; D.ldx = ldx; D.f32 = f32; D.m = n; D.epi = epi; D.y = y; D.ldy = ldy; D.n_store = w->rows_pad;
        D.partial = partial;
        return D;
    };
    for (size_t r = 0; r < runs.size(); ++r) {
        const Layer &L = layers[(size_t)runs[r].layer];
        const float *step = runs[r].step >= 0 ? steps[(size_t)runs[r].step] : nullptr;
        WindowAttn A = attn_args(B, (int)r);
        DenseLaunch D = linear(L.qk, B.act, width_pad, CANDY_HIP_EPI_NONE, B.qk, L.qk->rows_pad, &A.qk);
        if ((rc = norm_then(L.norm[0], L.norm[1], step, &D, elsewhere()))) return rc;
        if ((rc = pos_ptr ? launch_window_decode(dev, A, pos_ptr) : launch_window_prompt(dev, A, n, pos0))) return rc;
        if ((rc = launch_dense(dev, linear(L.o, B.att, L.o->ld, CANDY_HIP_EPI_NONE, B.y, width_pad, &pending)))) return rc;
        post_w = L.norm[2]; post_b = L.norm[3];
        if (L.c.d_ffn == 0) continue;
        D = linear(L.up, B.act, width_pad, CANDY_HIP_EPI_SQUARED_RELU, B.ff, L.down->ld, nullptr);
        if ((rc = norm_then(L.norm[4], L.norm[5], nullptr, &D, elsewhere()))) return rc;
        if ((rc = launch_dense(dev, linear(L.down, B.ff, L.down->ld, CANDY_HIP_EPI_NONE, B.y, width_pad, &pending)))) return rc;
        post_w = L.norm[6]; post_b = L.norm[7];
    }
    return norm_then(last ? final_w : nullptr, last ? final_b : nullptr, nullptr, last, x_final);
}

DenseLaunch candy_hip_suvazen::head_launch(const void *x, int n, float *out) const {
    DenseLaunch D;
    D.w = head; D.x = x; D.ldx = width_pad; D.f32 = f32; D.m = n; D.epi = CANDY_HIP_EPI_SOFTCAP;
    D.scale = cfg.logit_scale; D.cap = cfg.logit_softcap; D.y = out; D.ldy = D.n_store = vocab;
    return D;
}

int candy_hip_suvazen::enqueue_head() {
    NormArgs A = norm_args(dec, 1);
    A.x = h;
    A.pre_w = final_w; A.pre_b = final_b;
    if (int rc = launch_norm_chain(dev, A)) return rc;
    return launch_dense(dev, head_launch(dec.act, 1, logits));
}

int candy_hip_suvazen::enqueue_step() {
    Buffers B = dec;
    B.x = h;
    const DenseLaunch D = head_launch(B.act, 1, logits);
    if (int rc = layers_forward(B, 1, 0, d_pos, h, &D)) return rc;
    return launch_argmax_key(dev, logits, vocab, next_key);
}

int candy_hip_suvazen::enqueue_prompt(int n, int pos0) {
    if (int rc = embed(prompt_ids, n, pf.x)) return rc;
    Buffers B = pf;
    return layers_forward(B, n, pos0, nullptr, pf.x, nullptr);
}

int candy_hip_suvazen::enqueue_head_rows(const int32_t *rows, int n_rows, float *out) {
    if ((size_t)n_rows > row_ids_cap) {
        CANDY_HIP_TRY(hipStreamSynchronize(dev->stream));
        row_ids = nullptr;  // the old list stays owned by the model until it is freed
        if (int rc = decoder_alloc(this, &row_ids, (size_t)n_rows)) return rc;
        row_ids_cap = (size_t)n_rows;
    }
    if (int rc = candy_hip_h2d(dev, row_ids, rows, (size_t)n_rows * sizeof(int))) return rc;
    for (int r0 = 0; r0 < n_rows; r0 += prompt_cap) {  // the activations have room for one prompt's rows
        const int part = std::min(prompt_cap, n_rows - r0);
        NormArgs A = norm_args(pf, part);
        A.pre_w = final_w; A.pre_b = final_b; A.row_ids = row_ids + r0;
        if (int rc = launch_norm_chain(dev, A)) return rc;
        if (int rc = launch_dense(dev, head_launch(pf.act, part, out + (size_t)r0 * vocab))) return rc;
    }
    return CANDY_HIP_OK;
}

int candy_hip_suvazen::check_complete() const {
    CANDY_REQUIRE(head && final_w && final_b, "final norm / head not set");
    for (size_t l = 0; l < layers.size(); ++l) {
        const Layer &L = layers[l];
        CANDY_REQUIRE(L.qk && L.o && (!L.c.has_sink || L.sink) && (L.c.d_ffn == 0 || (L.up && L.down)), "layer %zu is missing weights", l);
        for (int i = 0; i < (L.c.d_ffn ? 8 : 4); ++i) CANDY_REQUIRE(L.norm[i], "layer %zu is missing norms", l);
    }
    for (size_t t = 0; t < steps.size(); ++t) CANDY_REQUIRE(steps[t], "the row of pass %zu is missing", t);
    return CANDY_HIP_OK;
}

extern "C" {

int candy_hip_suvazen_create(candy_hip_device *dev, const candy_hip_suvazen_config *cfg, const candy_hip_suvazen_layer *layers,
                             candy_hip_suvazen **out) {
    CANDY_REQUIRE(out, "out is nil");
    *out = nullptr;
    CANDY_REQUIRE(dev && cfg && layers, "nil argument");
    const candy_hip_suvazen_config &c = *cfg;
    CANDY_REQUIRE(c.n_layers > 0 && c.d_model > 0 && c.d_model <= 16384 && c.vocab > 0 && c.max_pos > 0,
                  "every size in the config must be positive (d_model at most 16384)");
    CANDY_REQUIRE(c.act == CANDY_HIP_ACT_BF16 || c.act == CANDY_HIP_ACT_F32, "unknown activation format %d", c.act);
    CANDY_REQUIRE(c.loop_times >= 0 && (c.loop_times == 0 || (c.loop_start >= 0 && c.loop_start < c.loop_stop && c.loop_stop <= c.n_layers)),
                  "loop %d .. %d does not lie inside %d layers", c.loop_start, c.loop_stop, c.n_layers);
    CANDY_REQUIRE(c.norm_eps >= 0 && c.logit_softcap >= 0, "negative constant in the config");
    for (int l = 0; l < c.n_layers; ++l) {
        if (int rc = check_attn_spec(layers[l].attn)) return rc;
        CANDY_REQUIRE(layers[l].d_ffn >= 0, "layer %d: negative feed-forward width", l);
    }
    if (int rc = use_device(dev)) return rc;
    candy_hip_suvazen *m = new candy_hip_suvazen();
    m->dev = dev;
    m->cfg = c;
    m->f32 = c.act == CANDY_HIP_ACT_F32;
    m->width = c.d_model;
    m->width_pad = (int)pad64(c.d_model);
    m->vocab = c.vocab;
    m->max_pos = m->cache.max_pos = c.max_pos;
    m->cache.elem_bytes = m->f32 ? 4 : 2;
    m->layers.resize((size_t)c.n_layers);
    const int loop_start = c.loop_times ? c.loop_start : 0, loop_stop = c.loop_times ? c.loop_stop : 0;
    for (int l = 0; l < loop_start; ++l) m->runs.push_back({l, -1});
    for (int t = 0; t < c.loop_times; ++t)
        for (int l = loop_start; l < loop_stop; ++l) m->runs.push_back({l, l == loop_start ? t : -1});
    for (int l = loop_stop; l < c.n_layers; ++l) m->runs.push_back({l, -1});
    m->steps.resize((size_t)c.loop_times, nullptr);
    int rc = CANDY_HIP_OK;
    for (int l = 0; l < c.n_layers; ++l) {
        candy_hip_suvazen::Layer &L = m->layers[(size_t)l];
        L.c = layers[l];
        const candy_hip_attn_spec &s = L.c.attn;
        L.n_splits = window_splits(dev, s, c.max_pos);
        m->max_part = std::max(m->max_part, window_scratch_floats(s, L.n_splits));
        m->max_qk = std::max(m->max_qk, (int)pad64((int64_t)(s.n_heads + s.n_kv_heads) * s.head_dim));
        m->max_att = std::max(m->max_att, (int)pad64((int64_t)s.n_heads * s.head_dim));
        m->max_q = std::max(m->max_q, s.n_heads * candy_hip_attn_row(s.head_dim));
        m->max_ff = std::max(m->max_ff, (int)pad64(L.c.d_ffn));
        // layers with the same rotation share its tables
        for (int k = 0; k < l && !L.cos_t; ++k) {
            const candy_hip_attn_spec &o = m->layers[(size_t)k].c.attn;
            if (o.rope_dims == s.rope_dims && o.rope_base == s.rope_base && o.rope_original == s.rope_original &&
                o.rope_factor == s.rope_factor && o.rope_low == s.rope_low && o.rope_high == s.rope_high) {
                L.cos_t = m->layers[(size_t)k].cos_t;
                L.sin_t = m->layers[(size_t)k].sin_t;
            }
        }
        if (!L.cos_t && s.rope_dims > 0 && !rc) {
            const size_t count = (size_t)c.max_pos * (s.rope_dims / 2);
            std::vector<float> hc(count), hs(count);
            fill_rope_tables(s, c.max_pos, hc.data(), hs.data());
            float *ct = nullptr, *st = nullptr;
            rc = decoder_alloc(m, &ct, count);
            if (!rc) rc = decoder_alloc(m, &st, count);
            if (!rc) rc = candy_hip_h2d(dev, ct, hc.data(), count * sizeof(float));
            if (!rc) rc = candy_hip_h2d(dev, st, hs.data(), count * sizeof(float));
            L.cos_t = ct;
            L.sin_t = st;
        }
    }
    for (const candy_hip_suvazen::Run &r : m->runs) {
        const candy_hip_attn_spec &s = m->layers[(size_t)r.layer].c.attn;
        m->cache.add_layer(s.n_kv_heads, candy_hip_attn_row(s.head_dim));
    }
    if (!rc) rc = decoder_init(m);
    if (!rc) rc = m->alloc_buffers(m->dec, 1, [m](uint8_t **p, size_t b) { return decoder_alloc(m, p, b); });
    if (rc) {
        candy_hip_decoder_free(m);
        return rc;
    }
    *out = m;
    return CANDY_HIP_OK;
}

candy_hip_decoder *candy_hip_suvazen_decoder(candy_hip_suvazen *m) { return m; }

int candy_hip_suvazen_set_matrix(candy_hip_suvazen *m, int which, int layer, const candy_hip_dense *w) {
    CANDY_REQUIRE(m && w, "nil argument");
    CANDY_REQUIRE(w->dev == m->dev, "weight lives on another device");
    const bool global = which == CANDY_HIP_SV_HEAD || which == CANDY_HIP_SV_EMBED;
    CANDY_REQUIRE(which >= CANDY_HIP_SV_QK && which <= CANDY_HIP_SV_EMBED, "unknown weight kind %d", which);
    CANDY_REQUIRE(global || (layer >= 0 && layer < m->cfg.n_layers), "layer %d out of range", layer);
    candy_hip_suvazen::Layer *L = global ? nullptr : &m->layers[(size_t)layer];
    const int64_t d = m->cfg.d_model;
    int64_t rows = m->cfg.vocab, cols = d;
    const candy_hip_dense **slot = which == CANDY_HIP_SV_HEAD ? &m->head : &m->embed_w;
    switch (which) {
    case CANDY_HIP_SV_QK: slot = &L->qk; rows = (int64_t)(L->c.attn.n_heads + L->c.attn.n_kv_heads) * L->c.attn.head_dim; break;
    case CANDY_HIP_SV_O: slot = &L->o; rows = d; cols = (int64_t)L->c.attn.n_heads * L->c.attn.head_dim; break;
    case CANDY_HIP_SV_UP: slot = &L->up; rows = L->c.d_ffn; break;
    case CANDY_HIP_SV_DOWN: slot = &L->down; rows = d; cols = L->c.d_ffn; break;
    }
    CANDY_REQUIRE(w->rows == rows && w->cols == cols, "weight kind %d must be %lld x %lld, got %lld x %lld", which, (long long)rows,
                  (long long)cols, (long long)w->rows, (long long)w->cols);
    *slot = w;
    m->graph_dirty = true;
    return CANDY_HIP_OK;
}

int candy_hip_suvazen_set_vector(candy_hip_suvazen *m, int which, int layer, const float *host, int64_t count) {
    CANDY_REQUIRE(m && host, "nil argument");
    const bool final_norm = which == CANDY_HIP_SV_FINAL || which == CANDY_HIP_SV_FINAL_BIAS;
    CANDY_REQUIRE(which >= CANDY_HIP_SV_NORM1 && which <= CANDY_HIP_SV_FINAL_BIAS, "unknown vector kind %d", which);
    const int limit = which == CANDY_HIP_SV_STEP ? m->cfg.loop_times : m->cfg.n_layers;
    CANDY_REQUIRE(final_norm || (layer >= 0 && layer < limit), "layer %d out of range", layer);
    int64_t want = m->cfg.d_model;
    float **slot;
    if (final_norm) slot = which == CANDY_HIP_SV_FINAL ? &m->final_w : &m->final_b;
    else if (which == CANDY_HIP_SV_STEP) slot = &m->steps[(size_t)layer];
    else if (which == CANDY_HIP_SV_SINK) {
        slot = &m->layers[(size_t)layer].sink;
        want = m->layers[(size_t)layer].c.attn.n_heads;
    } else slot = &m->layers[(size_t)layer].norm[which];
    CANDY_REQUIRE(count == want, "vector kind %d has %lld values, got %lld", which, (long long)want, (long long)count);
    if (int rc = use_device(m->dev)) return rc;
    std::vector<float> padded((size_t)pad64(want), 0.0f);
    memcpy(padded.data(), host, (size_t)want * sizeof(float));
    if (!*slot)
        if (int rc = decoder_alloc(m, slot, padded.size())) return rc;
    m->graph_dirty = true;
    return candy_hip_h2d(m->dev, *slot, padded.data(), padded.size() * sizeof(float));
}

}  // extern "C"
