// The part of a decoder that does not depend on its layers (decoder.h): one token through the captured step, a prompt
// in one pass, greedy generation without the host in the loop.
#include "decoder.h"

namespace candy {

// Parks the step's position and token id in device memory (read by the captured kernels).
__global__ void k_set_step(int *pos_dst, int pos, int64_t *tok_dst, int64_t tok, unsigned long long *key) {
    *pos_dst = pos;
    if (tok >= 0) *tok_dst = tok;
    *key = 0;  // the step's argmax folds into it
}

// Greedy generation without the host in the loop: the token the last step chose becomes the next step's input and
// is written to the list the caller gets at the end.
__global__ void k_chain_step(int *pos_dst, int pos, int64_t *tok_dst, unsigned long long *key, int32_t *list) {
    *pos_dst = pos;
    const uint32_t t = argmax_key_index(*key);
    *key = 0;
    *tok_dst = (int64_t)t;
    *list = (int32_t)t;
}

int decoder_init(candy_hip_decoder *m) {
    int rc = CANDY_HIP_OK;
    uint8_t *k = nullptr, *v = nullptr;
    if (!rc && m->cache.bytes()) rc = decoder_alloc(m, &k, m->cache.bytes());
    if (!rc && m->cache.bytes() && !m->cache.one_array) rc = decoder_alloc(m, &v, m->cache.bytes());
    m->cache.k = k;
    m->cache.v = v;
    if (!rc && k) rc = candy_hip_zero(m->dev, k, m->cache.bytes());
    if (!rc && v) rc = candy_hip_zero(m->dev, v, m->cache.bytes());
    if (!rc && m->state.floats) rc = decoder_alloc(m, &m->state.data, m->state.floats);
    if (!rc && m->state.floats) rc = candy_hip_zero(m->dev, m->state.data, m->state.floats * sizeof(float));
    if (!rc) rc = decoder_alloc(m, &m->h, (size_t)m->width_pad);
    if (!rc) rc = candy_hip_zero(m->dev, m->h, (size_t)m->width_pad * sizeof(float));  // what pads the row stays zero
    if (!rc) rc = decoder_alloc(m, &m->logits, (size_t)m->vocab + 4);  // the argmax kernel reads whole 16-byte pieces
    if (!rc) rc = decoder_alloc(m, &m->next_key, 1);
    if (!rc) rc = candy_hip_zero(m->dev, m->next_key, sizeof(unsigned long long));
    if (!rc) rc = decoder_alloc(m, &m->tok_id, 1);
    if (!rc) rc = decoder_alloc(m, &m->d_pos, 1);
    m->use_graph = m->dev->opt.llama_graph != 0;
    return rc;
}

}  // namespace candy

using namespace candy;

int candy_hip_decoder::enqueue_head_rows(const int32_t *rows, int n_rows, float *out) {
    for (int i = 0; i < n_rows; ++i) {
        if (int rc = candy_hip_d2d(dev, h, prompt_hidden() + (size_t)rows[i] * width_pad, (size_t)width_pad * sizeof(float)))
            return rc;
        if (int rc = enqueue_head()) return rc;
        if (int rc = candy_hip_d2d(dev, out + (size_t)i * vocab, logits, (size_t)vocab * sizeof(float))) return rc;
    }
    return CANDY_HIP_OK;
}

// Whether a call may feed position pos: recurrent state stands behind one position only.
static int check_order(const candy_hip_decoder *m, int32_t pos) {
    CANDY_REQUIRE(!m->state.floats || pos == 0 || pos == m->state.next, "position %d out of order: the recurrent state stands in front of %d",
                  pos, m->state.next);
    return CANDY_HIP_OK;
}

// chain_to: null, or where the token chosen by the previous step is recorded while it becomes this step's input
static int decoder_step(candy_hip_decoder *m, int32_t pos, int64_t token, const float *dev_hidden,
                        const float **dev_logits, int32_t *next_token, int32_t *chain_to = nullptr) {
    candy_hip_device *dev = m->dev;
    int rc;
    m->state.next = -1;
    if (chain_to)
        hipLaunchKernelGGL(k_chain_step, dim3(1), dim3(1), 0, dev->stream, m->d_pos, (int)pos, m->tok_id, m->next_key, chain_to);
    else
        hipLaunchKernelGGL(k_set_step, dim3(1), dim3(1), 0, dev->stream, m->d_pos, (int)pos, m->tok_id, token, m->next_key);
    CANDY_LAUNCH_CHECK();
    if (dev_hidden) {
        if ((rc = candy_hip_d2d(dev, m->h, dev_hidden, (size_t)m->width * sizeof(float)))) return rc;
    } else {
        if ((rc = m->embed(m->tok_id, 1, m->h))) return rc;
    }
    if (m->use_graph) {
        if (m->graph_epoch != dev->opt_epoch) m->graph_dirty = true;  // an option changed: other kernels may be due
        if (m->graph_dirty) {
            // a replay of the old graph may still be in flight (a caller that did not ask for the token): drain first
            if (m->graph_exec) CANDY_HIP_TRY(hipStreamSynchronize(dev->stream));
            if (m->graph_exec) CANDY_HIP_TRY(hipGraphExecDestroy(m->graph_exec));
            if (m->graph) CANDY_HIP_TRY(hipGraphDestroy(m->graph));
            m->graph_exec = nullptr;
            m->graph = nullptr;
            // kernels may count on their tickets being zero at launch and leave them so; a step that was cut short (an
            // error, a device reset) may not have: start every new graph from the initial state
            if ((rc = m->reset_step())) return rc;
            CANDY_HIP_TRY(hipStreamBeginCapture(dev->stream, hipStreamCaptureModeThreadLocal));
            rc = m->enqueue_step();
            hipError_t e = hipStreamEndCapture(dev->stream, &m->graph);
            if (rc) return rc;
            CANDY_HIP_TRY(e);
            CANDY_HIP_TRY(hipGraphInstantiate(&m->graph_exec, m->graph, nullptr, nullptr, 0));
            m->graph_dirty = false;
            m->graph_epoch = dev->opt_epoch;
        }
        CANDY_HIP_TRY(hipGraphLaunch(m->graph_exec, dev->stream));
    } else if ((rc = m->enqueue_step())) {
        (void)m->reset_step();  // see above
        return rc;
    }
    m->state.next = pos + 1;
    if (dev_logits) *dev_logits = m->logits;
    if (next_token) {
        unsigned long long key = 0;
        if ((rc = candy_hip_d2h(dev, &key, m->next_key, sizeof(key)))) return rc;
        *next_token = (int32_t)argmax_key_index(key);
    }
    return CANDY_HIP_OK;
}

// Everything of a prompt pass up to the residual stream behind the last layer.
static int decoder_feed(candy_hip_decoder *m, const int32_t *tokens, int32_t n_tokens, int32_t pos0) {
    CANDY_REQUIRE(m, "model is nil");
    CANDY_REQUIRE(m->has_embedding(), "embedding table not set");
    CANDY_REQUIRE(tokens && n_tokens > 0, "prompt is empty");
    CANDY_REQUIRE(pos0 >= 0 && (int64_t)pos0 + n_tokens <= m->max_pos,
                  "positions %d..%lld outside the cache (max_pos %d)", pos0, (long long)pos0 + n_tokens - 1, m->max_pos);
    std::vector<int64_t> ids((size_t)n_tokens);
    for (int32_t i = 0; i < n_tokens; ++i) {
        CANDY_REQUIRE(tokens[i] >= 0 && tokens[i] < m->vocab, "token %d outside the vocabulary", tokens[i]);
        ids[(size_t)i] = tokens[i];
    }
    if (int rc = m->check_complete()) return rc;
    if (int rc = check_order(m, pos0)) return rc;
    if (int rc = use_device(m->dev)) return rc;
    if (n_tokens > m->prompt_cap) {
        CANDY_HIP_TRY(hipStreamSynchronize(m->dev->stream));
        for (void *p : m->prompt_owned) (void)candy_hip_free(m->dev, p);
        m->prompt_owned.clear();
        m->prompt_cap = 0;
        if (int rc = prompt_alloc(m, &m->prompt_ids, (size_t)n_tokens)) return rc;
        if (int rc = m->reserve_prompt(n_tokens)) return rc;
        m->prompt_cap = n_tokens;
    }
    if (int rc = candy_hip_h2d(m->dev, m->prompt_ids, ids.data(), ids.size() * sizeof(int64_t))) return rc;
    m->state.next = -1;
    if (int rc = m->enqueue_prompt(n_tokens, pos0)) return rc;
    m->state.next = pos0 + n_tokens;
    return CANDY_HIP_OK;
}

extern "C" {

int candy_hip_decoder_free(candy_hip_decoder *m) {
    if (!m) return CANDY_HIP_OK;
    (void)hipSetDevice(m->dev->ordinal);
    (void)hipStreamSynchronize(m->dev->stream);
    if (m->graph_exec) (void)hipGraphExecDestroy(m->graph_exec);
    if (m->graph) (void)hipGraphDestroy(m->graph);
    for (void *p : m->owned) (void)candy_hip_free(m->dev, p);
    for (void *p : m->prompt_owned) (void)candy_hip_free(m->dev, p);
    if (m->row_logits) (void)candy_hip_free(m->dev, m->row_logits);
    delete m;
    return CANDY_HIP_OK;
}

int candy_hip_decoder_set_graph(candy_hip_decoder *m, int enable) {
    CANDY_REQUIRE(m, "model is nil");
    m->use_graph = enable != 0;
    m->graph_dirty = true;  // also the way to have a changed device option picked up: the step is captured again
    return CANDY_HIP_OK;
}

int candy_hip_decoder_hidden(candy_hip_decoder *m, const float **dev_hidden) {
    CANDY_REQUIRE(m && dev_hidden, "nil argument");
    *dev_hidden = m->h;
    return CANDY_HIP_OK;
}

int candy_hip_decoder_prompt_hidden(candy_hip_decoder *m, const float **dev_hidden, int64_t *row_floats) {
    CANDY_REQUIRE(m && dev_hidden && row_floats, "nil argument");
    *dev_hidden = m->prompt_hidden();
    *row_floats = m->width_pad;
    return CANDY_HIP_OK;
}

int candy_hip_decoder_kv_cache(candy_hip_decoder *m, void **dev_k, void **dev_v, size_t *bytes_each) {
    CANDY_REQUIRE(m, "model is nil");
    if (dev_k) *dev_k = m->cache.k;
    if (dev_v) *dev_v = m->cache.v;
    if (bytes_each) *bytes_each = m->cache.bytes();
    return CANDY_HIP_OK;
}

int candy_hip_decoder_prefill(candy_hip_decoder *m, const int32_t *tokens, int32_t n_tokens, int32_t pos0,
                              const float **dev_logits, int32_t *next_token) {
    if (int rc = decoder_feed(m, tokens, n_tokens, pos0)) return rc;
    candy_hip_device *dev = m->dev;
    if (int rc = candy_hip_d2d(dev, m->h, m->prompt_hidden() + (size_t)(n_tokens - 1) * m->width_pad,
                               (size_t)m->width_pad * sizeof(float)))
        return rc;
    if (int rc = m->enqueue_head()) return rc;
    if (int rc = launch_zero(dev, m->next_key, sizeof(unsigned long long))) return rc;  // no step kernel in front here
    if (int rc = launch_argmax_key(dev, m->logits, m->vocab, m->next_key)) return rc;
    if (dev_logits) *dev_logits = m->logits;
    if (next_token) {
        unsigned long long key = 0;
        if (int rc = candy_hip_d2h(dev, &key, m->next_key, sizeof(key))) return rc;
        *next_token = (int32_t)argmax_key_index(key);
    }
    return CANDY_HIP_OK;
}

int candy_hip_decoder_prefill_rows(candy_hip_decoder *m, const int32_t *tokens, int32_t n_tokens, int32_t pos0,
                                   const int32_t *rows, int32_t n_rows, const float **dev_logits) {
    CANDY_REQUIRE(n_rows >= 0 && (n_rows == 0 || (rows && dev_logits)), "nil argument");
    for (int32_t i = 0; i < n_rows; ++i)
        CANDY_REQUIRE(rows[i] >= 0 && rows[i] < n_tokens, "row %d outside the prompt of %d tokens", rows[i], n_tokens);
    if (int rc = decoder_feed(m, tokens, n_tokens, pos0)) return rc;
    if (n_rows == 0) return CANDY_HIP_OK;
    const size_t want = (size_t)n_rows * m->vocab + 4;
    if (want > m->row_logits_cap) {
        CANDY_HIP_TRY(hipStreamSynchronize(m->dev->stream));
        if (m->row_logits) (void)candy_hip_free(m->dev, m->row_logits);
        m->row_logits = nullptr;
        m->row_logits_cap = 0;
        if (int rc = candy_hip_alloc(m->dev, want * sizeof(float), (void **)&m->row_logits)) return rc;
        m->row_logits_cap = want;
    }
    if (int rc = m->enqueue_head_rows(rows, n_rows, m->row_logits)) return rc;
    *dev_logits = m->row_logits;
    return CANDY_HIP_OK;
}

int candy_hip_decoder_decode_hidden(candy_hip_decoder *m, const float *dev_hidden, int32_t pos, const float **dev_logits,
                                    int32_t *next_token) {
    CANDY_REQUIRE(m && dev_hidden, "nil argument");
    CANDY_REQUIRE(pos >= 0 && pos < m->max_pos, "position %d outside the cache (max_pos %d)", pos, m->max_pos);
    if (int rc = m->check_complete()) return rc;
    if (int rc = check_order(m, pos)) return rc;
    if (int rc = use_device(m->dev)) return rc;
    return decoder_step(m, pos, -1, dev_hidden, dev_logits, next_token);
}

int candy_hip_decoder_decode(candy_hip_decoder *m, int32_t token, int32_t pos, const float **dev_logits,
                             int32_t *next_token) {
    CANDY_REQUIRE(m, "model is nil");
    CANDY_REQUIRE(m->has_embedding(), "embedding table not set");
    CANDY_REQUIRE(token >= 0 && token < m->vocab, "token %d outside the vocabulary", token);
    CANDY_REQUIRE(pos >= 0 && pos < m->max_pos, "position %d outside the cache (max_pos %d)", pos, m->max_pos);
    if (int rc = m->check_complete()) return rc;
    if (int rc = check_order(m, pos)) return rc;
    if (int rc = use_device(m->dev)) return rc;
    return decoder_step(m, pos, token, nullptr, dev_logits, next_token);
}

int candy_hip_decoder_generate(candy_hip_decoder *m, int32_t token, int32_t pos, int32_t n_steps, int32_t *tokens) {
    CANDY_REQUIRE(m && tokens, "nil argument");
    CANDY_REQUIRE(m->has_embedding(), "embedding table not set");
    CANDY_REQUIRE(token >= 0 && token < m->vocab, "token %d outside the vocabulary", token);
    CANDY_REQUIRE(n_steps >= 1, "invalid number of steps %d", n_steps);
    CANDY_REQUIRE(pos >= 0 && (int64_t)pos + n_steps <= m->max_pos, "positions %d .. %lld outside the cache (max_pos %d)",
                  pos, (long long)pos + n_steps - 1, m->max_pos);
    if (int rc = m->check_complete()) return rc;
    if (int rc = check_order(m, pos)) return rc;
    if (int rc = use_device(m->dev)) return rc;
    int32_t *list = nullptr;  // one slot per step; slot i takes the token step i chose
    if (int rc = candy_hip_alloc(m->dev, (size_t)(n_steps + 1) * sizeof(int32_t), (void **)&list)) return rc;
    int rc = decoder_step(m, pos, token, nullptr, nullptr, nullptr);
    for (int i = 1; i < n_steps && !rc; ++i) rc = decoder_step(m, pos + i, -1, nullptr, nullptr, nullptr, list + i - 1);
    if (!rc) {
        // the last step's choice: recorded by the same kernel, into a step that is not run (position and token
        // registers are rewritten by whatever step comes next)
        hipLaunchKernelGGL(k_chain_step, dim3(1), dim3(1), 0, m->dev->stream, m->d_pos, (int)(pos + n_steps - 1), m->tok_id,
                           m->next_key, list + n_steps - 1);
        if (hipGetLastError() != hipSuccess) rc = fail(CANDY_HIP_ERR_HIP, "launch failed");
    }
    if (!rc) rc = candy_hip_d2h(m->dev, tokens, list, (size_t)n_steps * sizeof(int32_t));
    const int rc2 = candy_hip_free(m->dev, list);
    return rc ? rc : rc2;
}

}  // extern "C"
