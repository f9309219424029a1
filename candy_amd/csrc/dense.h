// bfloat16 weights, layer norms and windowed attention: launch descriptors shared by dense.hip, layer_norm.hip,
// attention_window.hip and the models built from them.
#pragma once

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

// A projection's f32 result as its consumer takes it: `copies` partial results `stride` floats apart (a contraction
// split along K leaves several), rows `ld` floats apart.
struct Partial {
    const float *p = nullptr;
    int copies = 1;
    size_t stride = 0;
    int ld = 0;
};

struct DenseLaunch {
    const candy_hip_dense *w = nullptr;
    const void *x = nullptr;  // activations, rows of w->ld values `ldx` apart (zero or finite past w->cols)
    int64_t ldx = 0;
    bool f32 = false;         // activations (and the squared ReLU's output) are f32, otherwise bfloat16
    int m = 0;
    int epi = CANDY_HIP_EPI_NONE;
    float scale = 1.0f, cap = 0.0f;
    void *y = nullptr;        // NONE / SOFTCAP: f32; SQUARED_RELU: the activation format
    int64_t ldy = 0;
    int64_t n_store = 0;      // columns written per row: w->rows, or w->rows_pad (the padding comes out as zero)
    // NONE only, optional: the contraction may leave partial copies in the handle's split workspace instead of y
    Partial *partial = nullptr;
};
int launch_dense(candy_hip_device *dev, const DenseLaunch &L);

// The norms between two sublayers, per row: x + mult * norm(y) + step is the new residual row, out the norm of it.
struct NormArgs {
    const float *x = nullptr;       // residual rows, ldx apart
    int64_t ldx = 0;
    Partial y;                      // y.p null: nothing is added
    float mult = 1.0f;
    const float *post_w = nullptr, *post_b = nullptr;   // norm of y (with y.p)
    const float *step = nullptr;    // optional row added to every x
    float *x_out = nullptr;         // optional
    const float *pre_w = nullptr, *pre_b = nullptr;     // norm of the new x, written to out
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
int launch_dense_gather(candy_hip_device *dev, const candy_hip_dense *w, const int64_t *ids, int64_t n, float *out, int64_t ldo);

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

// Scores of one head are squashed by cap * tanh(s / cap); the hardware exponential carries it (absolute error a few
// ulp of cap).
__device__ __forceinline__ float tanh_fast(float z) {
    const float e = __builtin_amdgcn_exp2f(z * 2.88539008177792681f);  // exp(2z); inf and 0 are fine below
    return 1.0f - 2.0f * __builtin_amdgcn_rcpf(e + 1.0f);
}

}  // namespace candy
