// Layer normalization or RMS normalization, alone and chained: a sublayer's result enters the residual sum through a norm
// of its own and the next sublayer reads a norm of the sum, or the sum itself,
//     x <- x + mult * N(y) (+ step),   out = N(x) or x,
// in one pass over the row; y may be spread over partial copies and over the results of routed experts.  Everything in f32; `out` is rounded to the activation format on the store.
// One workgroup per row, the row in registers; mean and variance in two passes over them.
// (The reference path this library stands behind normalizes in front of its sublayers only, reduce.go:3071-3092.)
#include <algorithm>

#include "dense.h"

namespace candy {

struct NormKernelArgs {
    const float *x;
    const float *y;
    const float *post_w, *post_b, *step, *pre_w, *pre_b;
    float *x_out;
    void *out;
    const int *row_ids;
    int64_t ldx, ldy, ldo;
    size_t y_stride;
    const float *slots, *slot_weight;
    int64_t slot_ld;
    int y_copies, cols, top, rms;
    float mult, eps;
};

// V: float4 per thread; columns past `cols` (inside the padding) hold zeros and stay zero
template <class AT, int V>
__global__ __launch_bounds__(256) void k_norm_chain(const NormKernelArgs a) {
    __shared__ float red[4];
    const int tid = threadIdx.x;
    const size_t row = blockIdx.x;
    const size_t src = a.row_ids ? (size_t)a.row_ids[row] : row;
    const int cols = a.cols, padded = (cols + 63) & ~63;
    const float inv_n = 1.0f / (float)cols;
    f32x4 x[V], y[V];
    auto col = [&](int i) { return (tid + 256 * i) * 4; };
    auto load_row = [&](const float *p, f32x4 (&d)[V]) {
#pragma unroll
        for (int i = 0; i < V; ++i) d[i] = col(i) < padded ? *(const f32x4 *)(p + col(i)) : f32x4{0.f, 0.f, 0.f, 0.f};
    };
    // in place: d <- (d - mean) * rstd * w + b inside `cols`, 0 outside (RMS: mean and b are 0)
    auto normalize = [&](f32x4 (&d)[V], const float *w, const float *b) {
        float mean = 0.0f;
        if (!a.rms) {
            float s = 0.0f;
#pragma unroll
            for (int i = 0; i < V; ++i) s += (d[i][0] + d[i][1]) + (d[i][2] + d[i][3]);
            mean = block_sum(s, red) * inv_n;
        }
        float q = 0.0f;
#pragma unroll
        for (int i = 0; i < V; ++i)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                d[i][j] = col(i) + j < cols ? d[i][j] - mean : 0.0f;
                q += d[i][j] * d[i][j];
            }
        const float rstd = 1.0f / sqrtf(block_sum(q, red) * inv_n + a.eps);
#pragma unroll
        for (int i = 0; i < V; ++i) {
            if (col(i) >= padded) continue;
            const f32x4 wv = *(const f32x4 *)(w + col(i));  // zero in the padding, like b
            const f32x4 bv = b ? *(const f32x4 *)(b + col(i)) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < 4; ++j) d[i][j] = d[i][j] * rstd * wv[j] + bv[j];
        }
    };
    load_row(a.x + src * a.ldx, x);
    if (a.y || a.slots) {
#pragma unroll
        for (int i = 0; i < V; ++i) y[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int c = 0; a.y && c < a.y_copies; ++c) {
            f32x4 t[V];
            load_row(a.y + src * a.ldy + (size_t)c * a.y_stride, t);
#pragma unroll
            for (int i = 0; i < V; ++i) y[i] += t[i];
        }
        for (int k = 0; a.slots && k < a.top; ++k) {
            const size_t slot = src * a.top + k;
            const float g = a.slot_weight[slot];
            f32x4 t[V];
            load_row(a.slots + slot * a.slot_ld, t);
#pragma unroll
            for (int i = 0; i < V; ++i) y[i] += g * t[i];
        }
        normalize(y, a.post_w, a.post_b);
#pragma unroll
        for (int i = 0; i < V; ++i) x[i] += a.mult * y[i];
    }
    if (a.step) {
        load_row(a.step, y);
#pragma unroll
        for (int i = 0; i < V; ++i) x[i] += y[i];
    }
    if (a.x_out) {
#pragma unroll
        for (int i = 0; i < V; ++i)
            if (col(i) < padded) *(f32x4 *)(a.x_out + row * a.ldx + col(i)) = x[i];
    }
    if (a.out) {
        if (a.pre_w) normalize(x, a.pre_w, a.pre_b);
        AT *o = (AT *)a.out + row * a.ldo;
        typedef AT at4 __attribute__((ext_vector_type(4)));
#pragma unroll
        for (int i = 0; i < V; ++i)
            if (col(i) < padded) *(at4 *)(o + col(i)) = __builtin_convertvector(x[i], at4);
    }
}

int launch_norm_chain(candy_hip_device *dev, const NormArgs &A) {
    CANDY_REQUIRE(A.rows > 0 && A.cols > 0 && A.cols <= 16384, "layer norm takes rows of 1 .. 16384 values, got %d", A.cols);
    NormKernelArgs k{A.x, A.y.p, A.post_w, A.post_b, A.step, A.pre_w, A.pre_b, A.x_out, A.out, A.row_ids,
                     A.ldx, A.y.ld, A.ldo, A.y.stride, A.slots, A.slot_weight, A.slot_ld, A.y.copies, A.cols, A.top, A.rms, A.mult,
                     A.eps};
    const int v = (int)((pad64(A.cols) + 1023) / 1024);
    const dim3 g((unsigned)A.rows), b(256);
#define CANDY_NORM(AT)                                                                         \
    do {                                                                                       \
        if (v <= 1) hipLaunchKernelGGL((k_norm_chain<AT, 1>), g, b, 0, dev->stream, k);        \
        else if (v <= 2) hipLaunchKernelGGL((k_norm_chain<AT, 2>), g, b, 0, dev->stream, k);   \
        else if (v <= 4) hipLaunchKernelGGL((k_norm_chain<AT, 4>), g, b, 0, dev->stream, k);   \
        else if (v <= 8) hipLaunchKernelGGL((k_norm_chain<AT, 8>), g, b, 0, dev->stream, k);   \
        else hipLaunchKernelGGL((k_norm_chain<AT, 16>), g, b, 0, dev->stream, k);              \
    } while (0)
    if (A.f32) CANDY_NORM(float);
    else CANDY_NORM(bf16);
#undef CANDY_NORM
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

// [rows][cols] dense <-> rows `ld` apart with a zeroed tail
__global__ __launch_bounds__(256) void k_repitch(const float *src, int64_t lds, float *dst, int64_t ldd, int64_t rows,
                                                 int64_t cols) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= rows * ldd) return;
    const int64_t r = i / ldd, c = i % ldd;
    dst[i] = c < cols ? src[r * lds + c] : 0.0f;
}

static int repitch(candy_hip_device *dev, const float *src, int64_t lds, float *dst, int64_t ldd, int64_t rows, int64_t cols) {
    const int64_t grid = (rows * ldd + 255) / 256;
    CANDY_REQUIRE(grid <= 0x7FFFFFFF, "matrix too large");
    hipLaunchKernelGGL(k_repitch, dim3((unsigned)grid), dim3(256), 0, dev->stream, src, lds, dst, ldd, rows, cols);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

}  // namespace candy

using namespace candy;

extern "C" {

// The kernels work on rows padded to multiples of 64; these two entry points take plain ones and go through the
// handle's workspace.
static int norm_op(candy_hip_device *dev, const float *x, const float *y, const float *w, const float *b, float eps,
                   float mult, const float *step, int64_t rows, int64_t cols, float *out, bool rms = false) {
    CANDY_REQUIRE(dev, "device handle is nil");
    CANDY_REQUIRE(rows >= 0 && cols > 0 && cols <= 16384, "layer norm takes rows of 1 .. 16384 values, got %lld", (long long)cols);
    if (rows == 0) return CANDY_HIP_OK;
    CANDY_REQUIRE(rows <= 0x7FFFFFFF / 16384, "too many rows");
    CANDY_REQUIRE(x && w && (b || rms) && out, "nil pointer");
    if (int rc = use_device(dev)) return rc;
    const int64_t ld = pad64(cols);
    void *ws = nullptr;
    if (int rc = workspace(dev, (size_t)(2 * rows + 3) * ld * sizeof(float), &ws)) return rc;
    float *px = (float *)ws, *py = px + rows * ld, *pw = py + rows * ld, *pb = pw + ld, *ps = pw + 2 * ld;
    if (int rc = repitch(dev, x, cols, px, ld, rows, cols)) return rc;
    if (int rc = repitch(dev, w, cols, pw, ld, 1, cols)) return rc;
    if (b)
        if (int rc = repitch(dev, b, cols, pb, ld, 1, cols)) return rc;
    if (!b) pb = nullptr;
    NormArgs A;
    A.x = px; A.ldx = ld; A.eps = eps; A.rms = rms; A.rows = (int)rows; A.cols = (int)cols; A.f32 = true;
    if (y) {
        if (int rc = repitch(dev, y, cols, py, ld, rows, cols)) return rc;
        A.y.p = py; A.y.ld = (int)ld; A.post_w = pw; A.post_b = pb; A.mult = mult; A.x_out = px;
        if (step) {
            if (int rc = repitch(dev, step, cols, ps, ld, 1, cols)) return rc;
            A.step = ps;
        }
    } else {
        A.pre_w = pw; A.pre_b = pb; A.out = px; A.ldo = ld;
    }
    if (int rc = launch_norm_chain(dev, A)) return rc;
    return repitch(dev, px, ld, out, cols, rows, cols);
}

int candy_hip_layer_norm(candy_hip_device *dev, const float *x, const float *w, const float *b, float eps, int64_t rows,
                         int64_t cols, float *out) {
    return norm_op(dev, x, nullptr, w, b, eps, 1.0f, nullptr, rows, cols, out);
}

int candy_hip_add_layer_norm(candy_hip_device *dev, float *x, const float *y, const float *w, const float *b, float eps,
                             float mult, const float *step, int64_t rows, int64_t cols) {
    CANDY_REQUIRE(rows == 0 || y, "nil pointer");
    return norm_op(dev, x, y, w, b, eps, mult, step, rows, cols, x);
}

int candy_hip_add_rms_norm(candy_hip_device *dev, float *x, const float *y, const float *w, float eps, float mult, int64_t rows,
                           int64_t cols) {
    CANDY_REQUIRE(rows == 0 || y, "nil pointer");
    return norm_op(dev, x, y, w, nullptr, eps, mult, nullptr, rows, cols, x, true);
}

}  // extern "C"
