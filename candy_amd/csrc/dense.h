// bfloat16 weights, norms, attention, recurrence and experts: launch descriptors and small device helpers shared by
// dense.hip, layer_norm.hip, attention_window.hip, attention_latent.hip, recurrent.hip, experts.hip and the models built
// from them.
#pragma once

#include "blocks.h"
#include "internal.h"

struct candy_hip_dense {
    candy_hip_device *dev = nullptr;
    int64_t rows = 0, cols = 0;          // as given
    int64_t rows_pad = 0, ld = 0;        // as stored: multiples of 64, zero outside rows x cols
    void *data = nullptr;
};

namespace candy {

typedef __bf16 bf16;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4v __attribute__((ext_vector_type(4)));

inline int64_t pad64(int64_t n) { return (n + 63) & ~(int64_t)63; }
inline int64_t pad32(int64_t n) { return (n + 31) & ~(int64_t)31; }

__device__ __forceinline__ void widen8(u32x4v v, float (&f)[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        f[2 * i] = __uint_as_float(v[i] << 16);
        f[2 * i + 1] = __uint_as_float(v[i] & 0xFFFF0000u);
    }
}
__device__ __forceinline__ void lds8(const bf16 *p, float (&f)[8]) { widen8(*(const u32x4v *)p, f); }
__device__ __forceinline__ void lds8(const float *p, float (&f)[8]) {
    const f32x4 a = *(const f32x4 *)p, b = *(const f32x4 *)(p + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) { f[i] = a[i]; f[4 + i] = b[i]; }
}

// Sum over groups of LPR neighbouring lanes, in every lane of the group, on the DPP path.
template <int LPR>
__device__ __forceinline__ float lanes_sum(float v) {
    v += dpp_move<0xB1>(v);                       // quad_perm [1,0,3,2]
    v += dpp_move<0x4E>(v);                       // quad_perm [2,3,0,1]
    if (LPR >= 8) v += dpp_move<0x141>(v);        // row_half_mirror
    if (LPR >= 16) v += dpp_move<0x140>(v);       // row_mirror
    if (LPR >= 32) v += __shfl_xor(v, 16, 64);
    return v;
}

// Sum over the workgroup, in every thread.  red: one float per wavefront; safe to call again at once.
__device__ __forceinline__ float block_sum(float v, float *red) {
    v = wave_sum(v);
    const int n_waves = blockDim.x >> 6;
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = red[0];
    for (int w = 1; w < n_waves; ++w) t += red[w];
    __syncthreads();
    return t;
}

// attention kernels: a running maximum nothing has entered yet; a score whose exponential is 0 whatever the maximum
constexpr float LOW = -1e30f, MASKED = -3e38f;
constexpr float LOG2E = 1.44269504088896341f;

// A projection's f32 result as its consumer takes it: `copies` partial results `stride` floats apart (a contraction
// split along K leaves several), rows `ld` floats apart.
struct Partial {
    const float *p = nullptr;
    int copies = 1;
    size_t stride = 0;
    int ld = 0;
};

// Activation rows dealt to experts: w holds `expert_rows` rows per expert one after the other; tile t of the list takes
// rows first .. first + count - 1 of `perm` for one expert, whose tiles are of_expert in number from tile0 on.  perm holds slots (token * top + choice); a slot's
// activations are row slot / x_div, its result is row slot.
struct alignas(16) GroupTile {
    int expert, first;
    int count;
    uint16_t tile0, of_expert;
};
struct GroupedRows {
    const int *perm = nullptr;
    const GroupTile *tiles = nullptr;
    const int *n_tiles = nullptr;   // device memory; at most max_tiles
    int max_tiles = 0, tile_rows = 64;
    int x_div = 1, expert_rows = 0;
};

struct DenseLaunch {
    const candy_hip_dense *w = nullptr;
    const void *x = nullptr;  // activations, rows of w->ld values `ldx` apart (zero or finite past w->cols)
    int64_t ldx = 0;
    bool f32 = false;         // activations (and outputs in the activation format) are f32, otherwise bfloat16
    int m = 0;
    int epi = CANDY_HIP_EPI_NONE;
    float scale = 1.0f, cap = 0.0f;
    void *y = nullptr;        // NONE / SOFTCAP: f32; SQUARED_RELU / ACT: the activation format
    int64_t ldy = 0;
    int64_t n_store = 0;      // columns written per row: w->rows, or w->rows_pad (the padding comes out as zero)
    // NONE only, optional: the contraction may leave partial copies in the handle's split workspace instead of y
    Partial *partial = nullptr;
    // block-diagonal weights: rows b * block_rows .. belong to block b, whose activations start at column b * w->ld
    // (a multiple of 128).  0: one block
    int block_rows = 0;
    const GroupedRows *group = nullptr;  // NONE / SQUARED_RELU, m: rows over all experts
};
int launch_dense(candy_hip_device *dev, const DenseLaunch &L);

// How a contraction of one row deals its weight rows to wavefronts.
struct MvShape {
    int waves, rows;  // wavefronts per workgroup, weight rows per wavefront
};
MvShape mv_shape(const candy_hip_device *dev, int64_t rows);

// The norms between two sublayers, per row: x + mult * norm(y) + step is the new residual row, out the norm of it.
// Layer norms, or RMS norms with `rms` (no mean taken off, no biases).
struct NormArgs {
    const float *x = nullptr;       // residual rows, ldx apart
    int64_t ldx = 0;
    bool rms = false;
    Partial y;                      // y.p null (and no slots): nothing is added
    // optional, added to y: sum over k of slot_weight[row * top + k] * slots[row * top + k] (prompt pass of routed experts)
    const float *slots = nullptr, *slot_weight = nullptr;
    int64_t slot_ld = 0;
    int top = 0;
    float mult = 1.0f;
    const float *post_w = nullptr, *post_b = nullptr;   // norm of y (with y.p)
    const float *step = nullptr;    // optional row added to every x
    float *x_out = nullptr;         // optional
    const float *pre_w = nullptr, *pre_b = nullptr;     // norm of the new x, written to out (pre_w null: x itself)
    void *out = nullptr;            // optional activations, rows ldo apart
    int64_t ldo = 0;
    bool f32 = false;
    float eps = 0.0f;
    int rows = 0, cols = 0;
    const int *row_ids = nullptr;   // optional: row r of the output is made from residual row row_ids[r]
};
int launch_norm_chain(candy_hip_device *dev, const NormArgs &A);  // layer_norm.hip; x_out may be x

// One bfloat16 row: the same norms in the prologue of the contraction that reads them (every workgroup repeats them, so
// x_out must not be x).  CANDY_HIP_ERR_UNSUPPORTED where two launches are the way.
int launch_dense_norm(candy_hip_device *dev, const DenseLaunch &L, const NormArgs &A);
// f32 rows <-> activation rows of `ld` values (zero past cols)
int launch_to_act(candy_hip_device *dev, bool f32, const float *src, void *dst, int64_t rows, int64_t cols, int64_t ld);
int launch_from_act(candy_hip_device *dev, bool f32, const void *src, float *dst, int64_t rows, int64_t cols, int64_t ld);
int launch_dense_gather(candy_hip_device *dev, const candy_hip_dense *w, const int64_t *ids, int64_t n, float *out, int64_t ldo,
                        float scale = 1.0f);

// attention_window.hip
struct WindowAttn {
    candy_hip_attn_spec s{};
    int row = 0;                    // candy_hip_attn_row(head_dim)
    int max_pos = 0;
    bool f32 = false;               // caches and q / out in f32, otherwise bfloat16
    const float *cos_t = nullptr, *sin_t = nullptr;  // [max_pos][rope_dims / 2]
    const float *sink = nullptr;    // optional [n_heads]
    void *k_cache = nullptr, *v_cache = nullptr;
    Partial qk;                     // projected q and k rows
    void *q = nullptr;              // scratch: n * n_heads * row values of the activation format (prompts and f32)
    float *part = nullptr;          // scratch of the decode kernel: window_scratch_floats()
    int n_splits = 1;
    void *out = nullptr;            // n rows, ldo apart, of the activation format; zeroed up to out_cols
    int64_t ldo = 0;
    int out_cols = 0;
};
int check_attn_spec(const candy_hip_attn_spec &s);
void fill_rope_tables(const candy_hip_attn_spec &s, int max_pos, float *cos_t, float *sin_t);  // host memory
int window_splits(const candy_hip_device *dev, const candy_hip_attn_spec &s, int max_pos);
size_t window_scratch_floats(const candy_hip_attn_spec &s, int n_splits);
int launch_window_prompt(candy_hip_device *dev, const WindowAttn &A, int n, int pos0);
int launch_window_decode(candy_hip_device *dev, const WindowAttn &A, const int *pos_ptr);

// attention_latent.hip.  Widths: dim, rotated part and values of a head in multiples of 32, ranks in multiples of 64.
struct LatentAttn {
    candy_hip_latent_spec s{};
    int max_pos = 0;
    bool f32 = false;               // cache, kv and out in f32, otherwise bfloat16
    const float *cos_t = nullptr, *sin_t = nullptr;  // [max_pos][rot_dim / 2]
    const float *sink = nullptr;    // optional [n_heads]
    const float *q_norm = nullptr, *kv_norm = nullptr;
    float eps = 0.0f;
    void *cache = nullptr;          // [max_pos][latent_row]
    bool own = true;                // the cache is this layer's to fill
    Partial down;                   // rows: pad64(q_rank) values in front of the normed query latent, then (own) the new cache row
    Partial q;                      // projected queries
    const candy_hip_dense *ukv = nullptr, *ukt = nullptr;
    void *cq = nullptr;             // out of launch_latent_rows: n rows of pad64(q_rank) activations
    void *kv = nullptr;             // prompts, scratch: keys and values of every head, max_pos rows of ukv->rows_pad activations
    void *qa = nullptr;             // decode, scratch: latent_query_bytes()
    float *part = nullptr;          // decode, scratch: latent_scratch_floats()
    int n_splits = 1;
    void *out = nullptr;            // n rows, ldo apart, of the activation format; zeroed up to out_cols
    int64_t ldo = 0;
    int out_cols = 0;
};
int check_latent_spec(const candy_hip_latent_spec &s);
int latent_splits(const candy_hip_device *dev, const candy_hip_latent_spec &s, int max_pos);
size_t latent_query_bytes(const candy_hip_latent_spec &s);
size_t latent_scratch_floats(const candy_hip_latent_spec &s, int n_splits);
// the projected rows -> normed query latents (with A.cq) and new cache rows (with A.own)
int launch_latent_rows(candy_hip_device *dev, const LatentAttn &A, int n, int pos0, const int *pos_ptr);
int launch_latent_prompt(candy_hip_device *dev, const LatentAttn &A, int n, int pos0);
// one token: the new cache row (with A.own), the queries against Wuk, attention over the cache, Wuv
int launch_latent_decode(candy_hip_device *dev, const LatentAttn &A, const int *pos_ptr);

// recurrent.hip
struct LruLayer {
    candy_hip_lru_spec s{};
    candy_hip_lru_params p{};
    const candy_hip_dense *gates = nullptr;
    bool f32 = false;
    float *state = nullptr;         // lru_state_floats
    Partial z;                      // rows: pad64(width) values for y, then for x
    void *u = nullptr;              // prompts, scratch: n rows of blocks * pad64(width / blocks) activations
    float *g = nullptr;             // prompts, scratch: n rows of gates->rows_pad
    float *scan = nullptr;          // prompts, scratch: lru_scan_floats()
    void *out = nullptr;            // n rows, ldo apart, zeroed up to out_cols
    int64_t ldo = 0;
    int out_cols = 0;
};
int check_lru_spec(const candy_hip_lru_spec &s);
size_t lru_state_floats(const candy_hip_lru_spec &s);
size_t lru_scan_floats(const candy_hip_lru_spec &s);
int lru_gate_rows(const candy_hip_lru_spec &s);
int launch_lru_prompt(candy_hip_device *dev, const LruLayer &A, int n, int pos0);
int launch_lru_step(candy_hip_device *dev, const LruLayer &A, const int *pos_ptr);

// experts.hip
struct ExpertLayer {
    candy_hip_expert_spec s{};
    candy_hip_expert_weights w{};
    int d = 0;
    bool f32 = false;
    const float *x = nullptr;       // n rows, ldx apart: what the router reads (and, one row, the experts)
    int64_t ldx = 0;
    const void *x_act = nullptr;    // prompts: the rows in the activation format, ld_act apart
    int64_t ld_act = 0;
    const float *logits = nullptr;  // one row: the router's
    int *ids = nullptr;             // [n][top]
    float *weights = nullptr;       // [n][top]
    void *act = nullptr;            // scratch: n * top rows of pad64(d_ff) activations; one row: expert_row_values()
    void *shared_act = nullptr;     // prompts, scratch: n rows of pad64(shared_ff)
    int *list = nullptr;            // prompts, scratch: expert_list_ints()
    float *slots = nullptr;         // prompts, out: n * top rows of pad64(d)
    float *y = nullptr;             // one row: the result; prompts: the shared expert's (left as `shared`)
    int64_t ldy = 0;
    Partial *shared = nullptr;
};
int check_expert_spec(const candy_hip_expert_spec &s, int d);
int check_expert_weights(const candy_hip_device *dev, const candy_hip_expert_spec &s, const candy_hip_expert_weights &w, int64_t d);
int expert_row_values(const candy_hip_expert_spec &s);
size_t expert_list_ints(const candy_hip_expert_spec &s, int n);
// the choice, then every chosen expert's result per slot and the shared one's per row (summed by launch_norm_chain)
int launch_experts_prompt(candy_hip_device *dev, const ExpertLayer &A, int n);
int launch_experts_row(candy_hip_device *dev, const ExpertLayer &A);  // A.logits -> A.y

// Scores of one head are squashed by cap * tanh(s / cap); the hardware exponential carries it (absolute error a few
// ulp of cap).
__device__ __forceinline__ float tanh_fast(float z) {
    const float e = __builtin_amdgcn_exp2f(z * 2.88539008177792681f);  // exp(2z); inf and 0 are fine below
    return 1.0f - 2.0f * __builtin_amdgcn_rcpf(e + 1.0f);
}

}  // namespace candy
