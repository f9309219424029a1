// What every decoder of the library shares: the KV cache, the captured decode step and its replay, the prompt pass
// around a model's layers, greedy generation.  A model (llama.hip, suvazen.hip, gulisun.hip) derives from candy_hip_decoder and
// supplies the layers; positions, tokens, logits, graphs and the cache are handled here.  (candy has no model code:
// no counterpart in the reference.)
#pragma once

#include <vector>

#include "internal.h"

namespace candy {

// Keys and values of all layers in two allocations, or in one where a row serves as both (latent attention).  Layer l's
// part is [kv heads][max_pos][row width]; the widths may differ from layer to layer.  A row is written when its position is fed and read only by later positions of the same
// sequence, so a sequence that starts over at position 0 needs no clearing.
struct KvCache {
    struct Layer {
        int n_kv_heads = 0, row = 0;  // row: values per position and head, as stored
        size_t offset = 0;            // in values
        int64_t stride = 0;           // values between kv heads
    };
    int max_pos = 0, elem_bytes = 4;
    std::vector<Layer> layers;
    size_t values = 0;                // per array
    bool one_array = false;           // no separate values: v stays null
    void *k = nullptr, *v = nullptr;

    void add_layer(int n_kv_heads, int row) {
        Layer L;
        L.n_kv_heads = n_kv_heads;
        L.row = row;
        L.offset = values;
        L.stride = (int64_t)max_pos * row;
        values += (size_t)n_kv_heads * (size_t)L.stride;
        layers.push_back(L);
    }
    void *k_of(int l) const { return (uint8_t *)k + layers[(size_t)l].offset * (size_t)elem_bytes; }
    void *v_of(int l) const { return (uint8_t *)v + layers[(size_t)l].offset * (size_t)elem_bytes; }
    size_t bytes() const { return values * (size_t)elem_bytes; }
};

// State of the recurrent layers, f32, one part per layer in one allocation.  It belongs to the sequence being fed and
// stands behind position next - 1; layers take position 0 as a fresh start whatever the state holds, so a sequence that
// starts over needs no clearing, but positions can only be fed in order.
struct RecurrentState {
    std::vector<size_t> offset;
    size_t floats = 0;
    float *data = nullptr;
    int next = 0;                     // -1: a call was cut short, only position 0 makes sense

    int add_layer(size_t n) {
        offset.push_back(floats);
        floats += n;
        return (int)offset.size() - 1;
    }
    float *of(int l) const { return data + offset[(size_t)l]; }
};

}  // namespace candy

struct candy_hip_decoder {
    candy_hip_device *dev = nullptr;
    int width = 0, vocab = 0, max_pos = 0;
    int width_pad = 0;                          // floats between rows of the residual stream
    candy::KvCache cache;
    candy::RecurrentState state;                // empty for models without recurrent layers
    float *h = nullptr;                         // residual stream of the token being decoded
    float *logits = nullptr;
    unsigned long long *next_key = nullptr;     // greedy token of the last step as k_argmax_key leaves it; zero before a step
    int64_t *tok_id = nullptr;
    int *d_pos = nullptr;                       // position of the token being decoded (device copy)
    hipGraph_t graph = nullptr;                 // the captured step (layers + head + argmax)
    hipGraphExec_t graph_exec = nullptr;
    bool graph_dirty = true;
    bool use_graph = true;
    unsigned graph_epoch = 0;                   // the device's option epoch the graph was captured under
    std::vector<void *> owned;                  // freed with the model
    std::vector<void *> prompt_owned;           // prompt buffers, replaced when a longer prompt comes
    int prompt_cap = 0;
    int64_t *prompt_ids = nullptr;
    float *row_logits = nullptr;                // logits of the rows a prompt pass was asked for
    size_t row_logits_cap = 0;                  // in floats

    virtual ~candy_hip_decoder() = default;
    virtual int check_complete() const = 0;
    virtual bool has_embedding() const = 0;
    // rows of the embedding table -> f32, width_pad apart
    virtual int embed(const int64_t *dev_ids, int64_t n, float *out) = 0;
    // h (and the position in d_pos) -> every layer -> logits -> next_key; nothing allocates or synchronises, so that the
    // sequence can be captured once and replayed for every token
    virtual int enqueue_step() = 0;
    // puts what a step counts on (tickets) back to its initial state
    virtual int reset_step() { return CANDY_HIP_OK; }
    // buffers for a prompt of n tokens (through prompt_alloc); called with prompt_cap < n
    virtual int reserve_prompt(int n) = 0;
    // prompt_ids at pos0 .. pos0+n-1 -> every layer; the residual stream of all rows stays behind
    virtual int enqueue_prompt(int n, int pos0) = 0;
    virtual const float *prompt_hidden() const = 0;  // [n][width_pad], after enqueue_prompt
    // h -> logits (final norm and head)
    virtual int enqueue_head() = 0;
    // prompt rows -> [n_rows][vocab]; a model without a batched head takes them one by one
    virtual int enqueue_head_rows(const int32_t *rows, int n_rows, float *out);
};

namespace candy {

template <class T>
int decoder_alloc(candy_hip_decoder *m, T **p, size_t count) {
    void *d = nullptr;
    if (int rc = candy_hip_alloc(m->dev, count * sizeof(T), &d)) return rc;
    m->owned.push_back(d);
    *p = (T *)d;
    return CANDY_HIP_OK;
}

template <class T>
int prompt_alloc(candy_hip_decoder *m, T **p, size_t count) {
    void *d = nullptr;
    if (int rc = candy_hip_alloc(m->dev, count * sizeof(T), &d)) return rc;
    m->prompt_owned.push_back(d);
    *p = (T *)d;
    return CANDY_HIP_OK;
}

// Buffers of the shared part and both cache arrays (cleared); sizes and cache layers are set by then.
int decoder_init(candy_hip_decoder *m);

}  // namespace candy
