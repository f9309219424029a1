// The Gulisun decoder: a residual stream in f32 that the sublayers read as it is and into which their results enter
// through an RMS norm; mixers are latent attention (over a cache of its own or an earlier layer's) or a real-gated linear
// recurrent unit, feed-forwards are routed experts beside a shared one.  Norm and residual sum are one launch (prompts,
// f32) or the prologue of the next contraction (bfloat16 decode step).  Step, prompt, cache, state and generation around
// the layers: decoder.hip.
#include <algorithm>
#include <cstring>
#include <vector>

#include "decoder.h"
#include "dense.h"

struct candy_hip_gulisun final : candy_hip_decoder {
    candy_hip_gulisun_config cfg{};
    struct Layer {
        candy_hip_gulisun_layer c{};
        const candy_hip_dense *w[CANDY_HIP_GL_EMBED] = {};   // in the order of enum candy_hip_gulisun_matrix
        float *v[CANDY_HIP_GL_FINAL] = {};                   // enum candy_hip_gulisun_vector
        const float *cos_t = nullptr, *sin_t = nullptr;
        int n_splits = 1;
        int part = 0;                                        // of the cache, or of the recurrent state

        bool latent() const { return c.mixer == CANDY_HIP_GL_LATENT; }
        bool own_cache() const { return c.kv_from < 0; }
        bool experts() const { return c.experts.n_experts > 0; }
    };
    std::vector<Layer> layers;
    float *final_w = nullptr;
    const candy_hip_dense *embed_w = nullptr;
    bool f32 = false;
    // widest rows over the layers
    int64_t max_z = 0, max_cq = 0, max_q = 0, max_att = 0, max_u = 0, max_kv = 0, max_top = 0, max_act = 0, max_row_act = 0, max_shared = 0,
            max_logits = 0;
    size_t max_qa = 0, max_part = 0, max_scan = 0;

    struct Buffers {                                         // n rows each
        float *x = nullptr, *x2 = nullptr, *x3 = nullptr, *z = nullptr, *q = nullptr, *y = nullptr, *part = nullptr, *logits = nullptr,
              *g = nullptr, *scan = nullptr, *weights = nullptr, *slots = nullptr;
        void *act = nullptr, *cq = nullptr, *att = nullptr, *qa = nullptr, *u = nullptr, *eact = nullptr, *sact = nullptr;
        int *ids = nullptr, *list = nullptr;
    };
    Buffers dec, pf;
    void *kv = nullptr;        // keys and values of every head and position, for the layer a prompt pass is in
    int *row_ids = nullptr;    // rows a prompt pass wants logits of
    size_t row_ids_cap = 0;

    size_t act_bytes() const { return f32 ? 4 : 2; }
    int check_complete() const override;
    bool has_embedding() const override { return embed_w != nullptr; }
    int embed(const int64_t *dev_ids, int64_t n, float *out) override {
        return candy::launch_dense_gather(dev, embed_w, dev_ids, n, out, width_pad, cfg.embed_scale);
    }
    int enqueue_step() override;
    int reserve_prompt(int n) override;
    int enqueue_prompt(int n, int pos0) override;
    const float *prompt_hidden() const override { return pf.x; }
    int enqueue_head() override;
    int enqueue_head_rows(const int32_t *rows, int n_rows, float *out) override;

    template <class Alloc>
    int alloc_buffers(Buffers &B, int n, Alloc alloc);
    candy::NormArgs norm_args(const Buffers &B, int n) const;
    candy::LatentAttn latent_args(const Buffers &B, const Layer &L) const;
    candy::LruLayer lru_args(const Buffers &B, const Layer &L) const;
    candy::ExpertLayer expert_args(const Buffers &B, const Layer &L) const;
    int layers_forward(Buffers &B, int n, int pos0, const int *pos_ptr, float *x_final, const candy::DenseLaunch *last);
    candy::DenseLaunch head_launch(const void *x, int n, float *out) const;
};

using namespace candy;

template <class Alloc>
int candy_hip_gulisun::alloc_buffers(Buffers &B, int n, Alloc alloc) {
    const size_t N = (size_t)n, es = act_bytes(), W = (size_t)width_pad;
    const bool step = &B == &dec;
    int rc = CANDY_HIP_OK;
    auto bytes = [&](auto **p, size_t b) {
        uint8_t *t = nullptr;
        if (!rc && b) rc = alloc(&t, b);
        *p = (std::remove_reference_t<decltype(*p)>)t;
    };
    if (!step) bytes(&B.x, N * W * 4);
    bytes(&B.z, N * max_z * 4);
    bytes(&B.q, N * max_q * 4);
    bytes(&B.y, N * W * 4);
    bytes(&B.act, N * W * es);
    bytes(&B.cq, N * max_cq * es);
    bytes(&B.att, N * max_att * es);
    bytes(&B.ids, N * max_top * 4);
    if (step) {
        bytes(&B.x2, W * 4);
        bytes(&B.x3, W * 4);
        bytes(&B.qa, max_qa);
        bytes(&B.part, max_part * 4);
        bytes(&B.logits, max_logits * 4);
        bytes(&B.eact, max_row_act * es);
    } else {
        bytes(&B.u, N * max_u * es);
        bytes(&B.g, N * max_u * 2 * 4);
        bytes(&B.scan, max_scan * 4);
        bytes(&B.weights, N * max_top * 4);
        bytes(&B.eact, N * max_act * es);
        bytes(&B.sact, N * max_shared * es);
        bytes(&B.slots, N * max_top * W * 4);
        size_t list = 0;
        for (const Layer &L : layers)
            if (L.experts()) list = std::max(list, expert_list_ints(L.c.experts, n));
        bytes(&B.list, list * 4);
    }
    return rc;
}

int candy_hip_gulisun::reserve_prompt(int n) {
    if (!kv && max_kv) {
        uint8_t *t = nullptr;
        if (int rc = decoder_alloc(this, &t, (size_t)max_pos * max_kv * act_bytes())) return rc;
        kv = t;
    }
    return alloc_buffers(pf, n, [this](uint8_t **p, size_t b) { return prompt_alloc(this, p, b); });
}

NormArgs candy_hip_gulisun::norm_args(const Buffers &B, int n) const {
    NormArgs A;
    A.x = B.x; A.ldx = width_pad; A.eps = cfg.norm_eps; A.rows = n; A.cols = width; A.f32 = f32; A.rms = true;
    A.out = B.act; A.ldo = width_pad;
    return A;
}

LatentAttn candy_hip_gulisun::latent_args(const Buffers &B, const Layer &L) const {
    LatentAttn A;
    A.s = L.c.latent;
    A.max_pos = max_pos; A.f32 = f32; A.eps = cfg.norm_eps;
    A.cos_t = L.cos_t; A.sin_t = L.sin_t; A.sink = L.c.has_sink ? L.v[CANDY_HIP_GL_SINK] : nullptr;
    A.q_norm = L.v[CANDY_HIP_GL_Q_NORM]; A.kv_norm = L.v[CANDY_HIP_GL_KV_NORM];
    A.cache = cache.k_of(L.part); A.own = L.own_cache();
    A.ukv = L.w[CANDY_HIP_GL_UKV]; A.ukt = L.w[CANDY_HIP_GL_UKT];
    A.cq = B.cq; A.kv = kv; A.qa = B.qa; A.part = B.part; A.n_splits = L.n_splits;
    A.out = B.att; A.ldo = L.w[CANDY_HIP_GL_O]->ld; A.out_cols = (int)A.ldo;
    return A;
}

LruLayer candy_hip_gulisun::lru_args(const Buffers &B, const Layer &L) const {
    LruLayer A;
    A.s = L.c.lru;
    A.p = candy_hip_lru_params{L.v[CANDY_HIP_GL_Y_BIAS], L.v[CANDY_HIP_GL_X_BIAS], L.v[CANDY_HIP_GL_CONV], L.v[CANDY_HIP_GL_CONV_BIAS],
                               L.v[CANDY_HIP_GL_RA_BIAS], L.v[CANDY_HIP_GL_RI_BIAS], L.v[CANDY_HIP_GL_LAM]};
    A.gates = L.w[CANDY_HIP_GL_GATES]; A.f32 = f32; A.state = state.of(L.part);
    A.u = B.u; A.g = B.g; A.scan = B.scan;
    A.out = B.att; A.ldo = L.w[CANDY_HIP_GL_O]->ld; A.out_cols = (int)A.ldo;
    return A;
}

ExpertLayer candy_hip_gulisun::expert_args(const Buffers &B, const Layer &L) const {
    ExpertLayer A;
    A.s = L.c.experts;
    A.w = candy_hip_expert_weights{L.w[CANDY_HIP_GL_ROUTER], L.w[CANDY_HIP_GL_UP], L.w[CANDY_HIP_GL_DOWN], L.w[CANDY_HIP_GL_SHARED_UP],
                                   L.w[CANDY_HIP_GL_SHARED_DOWN]};
    A.d = width; A.f32 = f32;
    A.x = B.x; A.ldx = width_pad; A.x_act = B.act; A.ld_act = width_pad;
    A.logits = B.logits; A.ids = B.ids; A.weights = B.weights; A.act = B.eact; A.shared_act = B.sact; A.list = B.list; A.slots = B.slots;
    A.y = B.y; A.ldy = width_pad;
    return A;
}

// The layers over n rows whose residual stream is in B.x; it ends in x_final, and `last`, if any, contracts the final
// norm of it.  pos_ptr: one token, its position in device memory; otherwise positions pos0 ...  A sublayer's result
// enters the residual sum in front of the next contraction.
int candy_hip_gulisun::layers_forward(Buffers &B, int n, int pos0, const int *pos_ptr, float *x_final, const DenseLaunch *last) {
    int rc;
    NormArgs pending;                                  // y / slots and post_w of a result not yet added
    bool is_pending = false;
    const bool step = pos_ptr != nullptr, fuse = step && !f32;
    float *const own[2] = {B.x2, B.x3};                // fused: the stream alternates between these two
    auto elsewhere = [&] { return fuse ? own[B.x == own[0]] : B.x; };
    // x <- x + norm(pending), written to `to`; then `next` contracts it (with w: its norm).  What is made of the sum beside
    // that: activations, nothing, or nothing because `next` takes the f32 sum itself
    enum Make { ACT, NOTHING, WIDE };
    auto add_then = [&](DenseLaunch *next, float *to, Make make, const float *w = nullptr) -> int {
        NormArgs A = norm_args(B, n);
        if (is_pending) {
            A.y = pending.y; A.slots = pending.slots; A.slot_weight = pending.slot_weight; A.slot_ld = pending.slot_ld; A.top = pending.top;
            A.post_w = pending.post_w; A.x_out = to;
        }
        is_pending = false;
        A.pre_w = w;
        if (make != ACT) A.out = nullptr;
        int e = CANDY_HIP_ERR_UNSUPPORTED;
        // every workgroup of the fused launch reads the old row: the new one goes elsewhere
        if (next && fuse && A.x_out != A.x) e = launch_dense_norm(dev, *next, A);
        if (e == CANDY_HIP_ERR_UNSUPPORTED) {
            e = A.out || A.x_out ? launch_norm_chain(dev, A) : CANDY_HIP_OK;
            if (next && make == WIDE) next->x = A.x_out ? A.x_out : B.x;
            if (!e && next) e = launch_dense(dev, *next);
        }
        if (A.x_out) B.x = A.x_out;
        return e;
    };
    auto linear = [&](const candy_hip_dense *w, const void *x, int64_t ldx, void *y, int64_t ldy, Partial *partial) {
        DenseLaunch D;
        D.w = w; D.x = x; D.ldx = ldx; D.f32 = f32; D.m = n; D.y = y; D.ldy = ldy; D.n_store = w->rows_pad; D.partial = partial;
        return D;
    };
    for (const Layer &L : layers) {
        const candy_hip_dense *in = L.w[CANDY_HIP_GL_IN], *o = L.w[CANDY_HIP_GL_O];
        Partial z;
        DenseLaunch D = linear(in, B.act, width_pad, B.z, in->rows_pad, &z);
        if ((rc = add_then(&D, elsewhere(), ACT))) return rc;
        if (L.latent()) {
            LatentAttn A = latent_args(B, L);
            const candy_hip_dense *uq = L.w[CANDY_HIP_GL_UQ];
            A.down = z;
            D = linear(uq, B.cq, uq->ld, B.q, uq->rows_pad, &A.q);
            rc = CANDY_HIP_ERR_UNSUPPORTED;
            if (fuse) {                                // the query latent's norm in the contraction's prologue
                NormArgs N;
                N.x = z.p; N.ldx = z.ld; N.eps = cfg.norm_eps; N.rows = 1; N.cols = A.s.q_rank; N.rms = true; N.pre_w = A.q_norm;
                N.out = B.cq; N.ldo = uq->ld;
                rc = launch_dense_norm(dev, D, N);
            }
            if (rc == CANDY_HIP_ERR_UNSUPPORTED) {
                LatentAttn R = A;
                if (step) R.own = false;               // the decode kernels append the row themselves
                if ((rc = launch_latent_rows(dev, R, n, pos0, pos_ptr))) return rc;
                rc = launch_dense(dev, D);
            }
            if (rc) return rc;
            rc = step ? launch_latent_decode(dev, A, pos_ptr) : launch_latent_prompt(dev, A, n, pos0);
        } else {
            LruLayer A = lru_args(B, L);
            A.z = z;
            rc = step ? launch_lru_step(dev, A, pos_ptr) : launch_lru_prompt(dev, A, n, pos0);
        }
        if (rc) return rc;
        pending = NormArgs{};
        if ((rc = launch_dense(dev, linear(o, B.att, o->ld, B.y, width_pad, &pending.y)))) return rc;
        pending.post_w = L.v[CANDY_HIP_GL_NORM1];
        is_pending = true;
        if (!L.experts()) continue;
        if (step) {
            const candy_hip_dense *router = L.w[CANDY_HIP_GL_ROUTER];
            D = linear(router, nullptr, width_pad, B.logits, router->rows_pad, nullptr);
            D.f32 = true;
            if ((rc = add_then(&D, elsewhere(), WIDE))) return rc;
            if ((rc = launch_experts_row(dev, expert_args(B, L)))) return rc;
            pending = NormArgs{};
            pending.y = Partial{B.y, 1, 0, width_pad};
        } else {
            if ((rc = add_then(nullptr, B.x, ACT))) return rc;
            pending = NormArgs{};
            ExpertLayer A = expert_args(B, L);
            A.shared = &pending.y;
            if ((rc = launch_experts_prompt(dev, A, n))) return rc;
            pending.slots = B.slots; pending.slot_weight = B.weights; pending.slot_ld = width_pad; pending.top = L.c.experts.top;
        }
        pending.post_w = L.v[CANDY_HIP_GL_NORM2];
        is_pending = true;
    }
    DenseLaunch head;
    if (last) head = *last;
    return add_then(last ? &head : nullptr, x_final, last ? ACT : NOTHING, last ? final_w : nullptr);
}

DenseLaunch candy_hip_gulisun::head_launch(const void *x, int n, float *out) const {
    DenseLaunch D;
    D.w = embed_w; D.x = x; D.ldx = width_pad; D.f32 = f32; D.m = n; D.y = out; D.ldy = D.n_store = vocab;
    return D;
}

int candy_hip_gulisun::enqueue_head() {
    NormArgs A = norm_args(dec, 1);
    A.x = h;
    A.pre_w = final_w;
    if (int rc = launch_norm_chain(dev, A)) return rc;
    return launch_dense(dev, head_launch(dec.act, 1, logits));
}

int candy_hip_gulisun::enqueue_step() {
    Buffers B = dec;
    B.x = h;
    const DenseLaunch D = head_launch(B.act, 1, logits);
    if (int rc = layers_forward(B, 1, 0, d_pos, h, &D)) return rc;
    return launch_argmax_key(dev, logits, vocab, next_key);
}

int candy_hip_gulisun::enqueue_prompt(int n, int pos0) {
    if (int rc = embed(prompt_ids, n, pf.x)) return rc;
    Buffers B = pf;
    return layers_forward(B, n, pos0, nullptr, pf.x, nullptr);
}

int candy_hip_gulisun::enqueue_head_rows(const int32_t *rows, int n_rows, float *out) {
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
        A.pre_w = final_w; A.row_ids = row_ids + r0;
        if (int rc = launch_norm_chain(dev, A)) return rc;
        if (int rc = launch_dense(dev, head_launch(pf.act, part, out + (size_t)r0 * vocab))) return rc;
    }
    return CANDY_HIP_OK;
}

namespace {

// rows x cols a layer's matrix must have as given, {0, 0}: the layer has none of the kind
struct Shape {
    int64_t rows, cols;
};

Shape matrix_shape(const candy_hip_gulisun_layer &c, int64_t d, int which) {
    const candy_hip_latent_spec &a = c.latent;
    const candy_hip_lru_spec &u = c.lru;
    const candy_hip_expert_spec &e = c.experts;
    const bool attn = c.mixer == CANDY_HIP_GL_LATENT;
    const int64_t H = a.n_heads, dim = pad32(a.dim), rot = pad32(a.rot_dim), vdim = pad32(a.vdim), kv = pad64(a.kv_rank);
    switch (which) {
    case CANDY_HIP_GL_IN: return attn ? Shape{pad64(a.q_rank) + (c.kv_from < 0 ? kv + rot : 0), d} : Shape{2 * pad64(u.width), d};
    case CANDY_HIP_GL_O: return attn ? Shape{d, H * vdim} : Shape{d, u.width};
    case CANDY_HIP_GL_UQ: return attn ? Shape{H * (dim + rot), a.q_rank} : Shape{0, 0};
    case CANDY_HIP_GL_UKV: return attn ? Shape{H * (dim + vdim), a.kv_rank} : Shape{0, 0};
    case CANDY_HIP_GL_UKT: return attn ? Shape{H * kv, a.dim} : Shape{0, 0};
    case CANDY_HIP_GL_GATES: return attn ? Shape{0, 0} : Shape{lru_gate_rows(u), u.width / u.blocks};
    default: break;
    }
    if (!e.n_experts) return {0, 0};
    switch (which) {
    case CANDY_HIP_GL_ROUTER: return {e.n_experts, d};
    case CANDY_HIP_GL_UP: return {e.n_experts * pad64(e.d_ff), d};
    case CANDY_HIP_GL_DOWN: return {e.n_experts * pad64(d), e.d_ff};
    case CANDY_HIP_GL_SHARED_UP: return e.shared_ff ? Shape{e.shared_ff, d} : Shape{0, 0};
    case CANDY_HIP_GL_SHARED_DOWN: return e.shared_ff ? Shape{d, e.shared_ff} : Shape{0, 0};
    default: return {0, 0};
    }
}

// values of a layer's vector, in `rows` rows that are each padded on the device
Shape vector_shape(const candy_hip_gulisun_layer &c, int64_t d, int which) {
    const bool attn = c.mixer == CANDY_HIP_GL_LATENT;
    switch (which) {
    case CANDY_HIP_GL_NORM1: return {1, d};
    case CANDY_HIP_GL_NORM2: return c.experts.n_experts ? Shape{1, d} : Shape{0, 0};
    case CANDY_HIP_GL_Q_NORM: return attn ? Shape{1, c.latent.q_rank} : Shape{0, 0};
    case CANDY_HIP_GL_KV_NORM: return attn && c.kv_from < 0 ? Shape{1, c.latent.kv_rank} : Shape{0, 0};
    case CANDY_HIP_GL_SINK: return attn && c.has_sink ? Shape{1, c.latent.n_heads} : Shape{0, 0};
    case CANDY_HIP_GL_CONV: return attn ? Shape{0, 0} : Shape{c.lru.taps, c.lru.width};
    default: return attn ? Shape{0, 0} : Shape{1, c.lru.width};
    }
}

}  // namespace

int candy_hip_gulisun::check_complete() const {
    CANDY_REQUIRE(embed_w && final_w, "embedding / final norm not set");
    for (size_t l = 0; l < layers.size(); ++l) {
        const Layer &L = layers[l];
        for (int k = 0; k < CANDY_HIP_GL_EMBED; ++k)
            CANDY_REQUIRE(L.w[k] || matrix_shape(L.c, width, k).rows == 0, "layer %zu is missing matrix %d", l, k);
        for (int k = 0; k < CANDY_HIP_GL_FINAL; ++k)
            CANDY_REQUIRE(L.v[k] || vector_shape(L.c, width, k).rows == 0, "layer %zu is missing vector %d", l, k);
    }
    return CANDY_HIP_OK;
}

static int check_layer(const candy_hip_gulisun_layer *layers, int l, int d) {
    const candy_hip_gulisun_layer &c = layers[l];
    CANDY_REQUIRE(c.mixer == CANDY_HIP_GL_LATENT || c.mixer == CANDY_HIP_GL_LRU, "layer %d: unknown mixer %d", l, c.mixer);
    if (c.mixer == CANDY_HIP_GL_LRU) {
        if (int rc = check_lru_spec(c.lru)) return rc;
    } else {
        if (int rc = check_latent_spec(c.latent)) return rc;
        if (c.kv_from >= 0) {
            CANDY_REQUIRE(c.kv_from < l, "layer %d reads the cache of layer %d, which does not run before it", l, c.kv_from);
            const candy_hip_gulisun_layer &j = layers[c.kv_from];
            CANDY_REQUIRE(j.mixer == CANDY_HIP_GL_LATENT && j.kv_from < 0, "layer %d: layer %d has no cache of its own", l, c.kv_from);
            CANDY_REQUIRE(j.latent.kv_rank == c.latent.kv_rank && j.latent.rot_dim == c.latent.rot_dim && j.latent.rope_base == c.latent.rope_base,
                          "layer %d: the cache of layer %d has other sizes or another rotation", l, c.kv_from);
        }
    }
    CANDY_REQUIRE(c.experts.n_experts >= 0, "layer %d: negative number of experts", l);
    return c.experts.n_experts ? check_expert_spec(c.experts, d) : CANDY_HIP_OK;
}

// Rotation tables of layer l, shared with the layers that turn alike.
static int rope_tables(candy_hip_gulisun *m, size_t l) {
    candy_hip_gulisun::Layer &L = m->layers[l];
    const candy_hip_latent_spec &s = L.c.latent;
    for (size_t k = 0; k < l && !L.cos_t; ++k) {
        const candy_hip_gulisun::Layer &o = m->layers[k];
        if (o.latent() && o.c.latent.rot_dim == s.rot_dim && o.c.latent.rope_base == s.rope_base) {
            L.cos_t = o.cos_t;
            L.sin_t = o.sin_t;
        }
    }
    if (L.cos_t || s.rot_dim == 0) return CANDY_HIP_OK;
    candy_hip_attn_spec turn{};
    turn.rope_dims = s.rot_dim;
    turn.rope_base = s.rope_base;
    const size_t count = (size_t)m->max_pos * (s.rot_dim / 2);
    std::vector<float> hc(count), hs(count);
    fill_rope_tables(turn, m->max_pos, hc.data(), hs.data());
    float *ct = nullptr, *st = nullptr;
    if (int rc = decoder_alloc(m, &ct, count)) return rc;
    if (int rc = decoder_alloc(m, &st, count)) return rc;
    if (int rc = candy_hip_h2d(m->dev, ct, hc.data(), count * sizeof(float))) return rc;
    L.cos_t = ct;
    L.sin_t = st;
    return candy_hip_h2d(m->dev, st, hs.data(), count * sizeof(float));
}

extern "C" {

int candy_hip_gulisun_create(candy_hip_device *dev, const candy_hip_gulisun_config *cfg, const candy_hip_gulisun_layer *layers,
                             candy_hip_gulisun **out) {
    CANDY_REQUIRE(out, "out is nil");
    *out = nullptr;
    CANDY_REQUIRE(dev && cfg && layers, "nil argument");
    const candy_hip_gulisun_config &c = *cfg;
    CANDY_REQUIRE(c.n_layers > 0 && c.d_model > 0 && c.d_model <= 16384 && c.vocab > 0 && c.max_pos > 0,
                  "every size in the config must be positive (d_model at most 16384)");
    CANDY_REQUIRE(c.act == CANDY_HIP_ACT_BF16 || c.act == CANDY_HIP_ACT_F32, "unknown activation format %d", c.act);
    CANDY_REQUIRE(c.norm_eps >= 0, "negative constant in the config");
    for (int l = 0; l < c.n_layers; ++l)
        if (int rc = check_layer(layers, l, c.d_model)) return rc;
    if (int rc = use_device(dev)) return rc;
    candy_hip_gulisun *m = new candy_hip_gulisun();
    m->dev = dev;
    m->cfg = c;
    m->f32 = c.act == CANDY_HIP_ACT_F32;
    m->width = c.d_model;
    m->width_pad = (int)pad64(c.d_model);
    m->vocab = c.vocab;
    m->max_pos = m->cache.max_pos = c.max_pos;
    m->cache.elem_bytes = m->f32 ? 4 : 2;
    m->cache.one_array = true;
    m->layers.resize((size_t)c.n_layers);
    int rc = CANDY_HIP_OK;
    auto grow = [](int64_t &v, int64_t to) { v = std::max(v, to); };
    for (size_t l = 0; l < m->layers.size() && !rc; ++l) {
        candy_hip_gulisun::Layer &L = m->layers[l];
        L.c = layers[l];
        auto rows = [&](int which) { return pad64(matrix_shape(L.c, c.d_model, which).rows); };
        grow(m->max_z, rows(CANDY_HIP_GL_IN));
        grow(m->max_att, pad64(matrix_shape(L.c, c.d_model, CANDY_HIP_GL_O).cols));
        if (L.latent()) {
            const candy_hip_latent_spec &s = L.c.latent;
            if (L.own_cache()) {
                L.part = (int)m->cache.layers.size();
                m->cache.add_layer(1, candy_hip_latent_row(&s));
            } else {
                L.part = m->layers[(size_t)L.c.kv_from].part;
            }
            L.n_splits = latent_splits(dev, s, c.max_pos);
            grow(m->max_cq, pad64(s.q_rank));
            grow(m->max_q, rows(CANDY_HIP_GL_UQ));
            grow(m->max_kv, rows(CANDY_HIP_GL_UKV));
            m->max_qa = std::max(m->max_qa, latent_query_bytes(s));
            m->max_part = std::max(m->max_part, latent_scratch_floats(s, L.n_splits));
            rc = rope_tables(m, l);
        } else {
            L.part = m->state.add_layer(lru_state_floats(L.c.lru));
            grow(m->max_u, lru_gate_rows(L.c.lru) / 2);
            m->max_scan = std::max(m->max_scan, lru_scan_floats(L.c.lru));
        }
        if (L.experts()) {
            const candy_hip_expert_spec &e = L.c.experts;
            grow(m->max_top, e.top);
            grow(m->max_act, e.top * pad64(e.d_ff));
            grow(m->max_row_act, expert_row_values(e));
            grow(m->max_shared, pad64(e.shared_ff));
            grow(m->max_logits, rows(CANDY_HIP_GL_ROUTER));
        }
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

candy_hip_decoder *candy_hip_gulisun_decoder(candy_hip_gulisun *m) { return m; }

int candy_hip_gulisun_set_matrix(candy_hip_gulisun *m, int which, int layer, const candy_hip_dense *w) {
    CANDY_REQUIRE(m && w, "nil argument");
    CANDY_REQUIRE(w->dev == m->dev, "weight lives on another device");
    CANDY_REQUIRE(which >= 0 && which <= CANDY_HIP_GL_EMBED, "unknown weight kind %d", which);
    const bool global = which == CANDY_HIP_GL_EMBED;
    CANDY_REQUIRE(global || (layer >= 0 && layer < m->cfg.n_layers), "layer %d out of range", layer);
    const Shape s = global ? Shape{m->vocab, m->width} : matrix_shape(m->layers[(size_t)layer].c, m->width, which);
    CANDY_REQUIRE(s.rows > 0, "layer %d has no weight of kind %d", layer, which);
    CANDY_REQUIRE(w->rows == s.rows && w->cols == s.cols, "weight kind %d must be %lld x %lld, got %lld x %lld", which, (long long)s.rows,
                  (long long)s.cols, (long long)w->rows, (long long)w->cols);
    if (global) m->embed_w = w;
    else m->layers[(size_t)layer].w[which] = w;
    m->graph_dirty = true;
    return CANDY_HIP_OK;
}

int candy_hip_gulisun_set_vector(candy_hip_gulisun *m, int which, int layer, const float *host, int64_t count) {
    CANDY_REQUIRE(m && host, "nil argument");
    CANDY_REQUIRE(which >= 0 && which <= CANDY_HIP_GL_FINAL, "unknown vector kind %d", which);
    const bool global = which == CANDY_HIP_GL_FINAL;
    CANDY_REQUIRE(global || (layer >= 0 && layer < m->cfg.n_layers), "layer %d out of range", layer);
    const Shape s = global ? Shape{1, m->width} : vector_shape(m->layers[(size_t)layer].c, m->width, which);
    CANDY_REQUIRE(s.rows > 0, "layer %d has no vector of kind %d", layer, which);
    CANDY_REQUIRE(count == s.rows * s.cols, "vector kind %d has %lld values, got %lld", which, (long long)(s.rows * s.cols), (long long)count);
    if (int rc = use_device(m->dev)) return rc;
    const int64_t pitch = pad64(s.cols);
    std::vector<float> padded((size_t)(s.rows * pitch), 0.0f);
    for (int64_t r = 0; r < s.rows; ++r) memcpy(&padded[(size_t)(r * pitch)], host + r * s.cols, (size_t)s.cols * sizeof(float));
    float **slot = global ? &m->final_w : &m->layers[(size_t)layer].v[which];
    if (!*slot)
        if (int rc = decoder_alloc(m, slot, padded.size())) return rc;
    m->graph_dirty = true;
    return candy_hip_h2d(m->dev, *slot, padded.data(), padded.size() * sizeof(float));
}

}  // extern "C"
