// Real-gated linear recurrent unit behind its projections (equations and layouts: include/candy_hip.h): a causal
// convolution per channel, two block-diagonal gates, a diagonal linear recurrence, and a gelu branch it is multiplied with.
//   prompts: k_lru_conv    u, rounded to the activation format
//            the gates' products (block-diagonal contraction, dense.hip)
//            k_lru_chunks  per chunk of tokens and channel: S behind it = A * S in front of it + B
//            k_lru_apply   S in front of a chunk from the chunks before it, then token by token; the last one leaves the state
//   decode:  k_lru_step    all of it for one token, 16 channels per workgroup
// The state of a sequence is S and the last `taps` inputs of the convolution, in f32: the input of position p sits in
// slot p mod taps, so that a step writes the one slot that none of its workgroups reads.  Position 0 ignores whatever
// the state holds.  (No counterpart in the reference, which has no recurrent layer.)
#include <algorithm>

#include "dense.h"

namespace candy {

struct LruArgs {
    candy_hip_lru_params p;
    int w, wp, blocks, size, size_p, taps;   // size: channels per block
    int out_cols;
    int64_t ldo;
};

__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-z * LOG2E)); }

// 0.5 z (1 + tanh(t)) = z / (1 + exp(-2t)), t = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh_f(float z) {
    return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-2.0f * LOG2E * 0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

__device__ __forceinline__ float decay_rate(float lam) { return -8.0f * (fmaxf(lam, 0.0f) + log1pf(expf(-fabsf(lam)))); }

// gate products (bias included), the unit's input and decay_rate -> S = a S + b
__device__ __forceinline__ void lru_coefficients(float zr, float zi, float u, float rate, float &a, float &b) {
    const float la = rate * sigmoid_f(zr), t = 2.0f * la;
    a = __builtin_amdgcn_exp2f(la * LOG2E);
    // 1 - exp(t): the series where the difference would cancel
    const float series = -t * (1.0f + t * (1.0f / 2) * (1.0f + t * (1.0f / 3) * (1.0f + t * (1.0f / 4) * (1.0f + t * (1.0f / 5) * (1.0f + t * (1.0f / 6))))));
    b = __builtin_amdgcn_sqrtf(t > -0.25f ? series : 1.0f - a * a) * sigmoid_f(zi) * u;
}

__device__ __forceinline__ float z_at(const Partial &z, size_t row, int i) {
    const float *s = z.p + row * (size_t)z.ld + i;
    float t = s[0];
    for (int c = 1; c < z.copies; ++c) t += s[(size_t)c * z.stride];
    return t;
}

// column of a channel's r product among the gates'; its i product stands 64 columns further
__device__ __forceinline__ int gate_column(const LruArgs &a, int block, int off) {
    return block * 2 * a.size_p + (off >> 6) * 128 + (off & 63);
}

// ------------------------------------------------------------------ prompts
constexpr int CONV_T = 8, CONV_TAPS = 4;

// The input of the convolution for token t of the portion (t < 0: earlier ones), bias included.
__device__ __forceinline__ float conv_input(const LruArgs &a, const Partial &z, const float *history, int c, float bx, int t, int pos0) {
    if (t >= 0) return z_at(z, (size_t)t, a.wp + c) + bx;
    return pos0 + t >= 0 ? history[(size_t)((pos0 + t) % a.taps) * a.wp + c] : 0.0f;
}

// grid (blocks * size_p / 256, ceil(n / 8)): one thread per padded channel and eight tokens.  FEW: at most 4 taps, the
// inputs are requested together.
template <class AT, bool FEW>
__global__ __launch_bounds__(256) void k_lru_conv(const LruArgs a, const Partial z, const float *__restrict__ history, AT *__restrict__ u,
                                                  int n, int pos0) {
    const int cp = blockIdx.x * 256 + threadIdx.x, cols = a.blocks * a.size_p;
    if (cp >= cols) return;
    const int off = cp % a.size_p, c = cp / a.size_p * a.size + off, t0 = blockIdx.y * CONV_T;
    float acc[CONV_T];
#pragma unroll
    for (int k = 0; k < CONV_T; ++k) acc[k] = 0.0f;
    if (off < a.size) {
        const float bx = a.p.bx[c], cb = a.p.conv_b[c];
#pragma unroll
        for (int k = 0; k < CONV_T; ++k) acc[k] = cb;
        if (FEW) {
            float v[CONV_T + CONV_TAPS - 1], w[CONV_TAPS];
#pragma unroll
            for (int j = 0; j < CONV_TAPS; ++j) w[j] = j < a.taps ? a.p.conv[(size_t)(a.taps - 1 - j) * a.wp + c] : 0.0f;  // j tokens back
#pragma unroll
            for (int i = 0; i < CONV_T + CONV_TAPS - 1; ++i) {
                const int t = min(t0 + i - (CONV_TAPS - 1), n - 1);
                v[i] = CONV_TAPS - 1 - i < a.taps ? conv_input(a, z, history, c, bx, t, pos0) : 0.0f;  // what no tap reaches may not exist
            }
#pragma unroll
            for (int k = 0; k < CONV_T; ++k)
#pragma unroll
                for (int j = CONV_TAPS - 1; j >= 0; --j) acc[k] = fmaf(w[j], v[k + CONV_TAPS - 1 - j], acc[k]);
        } else {
            for (int t = t0 - a.taps + 1; t < t0 + CONV_T && t < n; ++t) {
                const float v = conv_input(a, z, history, c, bx, t, pos0);
#pragma unroll
                for (int k = 0; k < CONV_T; ++k) {
                    const int tap = t - (t0 + k) + a.taps - 1;
                    if (tap >= 0 && tap < a.taps) acc[k] = fmaf(a.p.conv[(size_t)tap * a.wp + c], v, acc[k]);
                }
            }
        }
    }
#pragma unroll
    for (int k = 0; k < CONV_T; ++k)
        if (t0 + k < n) u[(size_t)(t0 + k) * cols + cp] = (AT)acc[k];
}

constexpr int SCAN_U = 8;   // tokens whose values are requested together

// f(t, a, b, y) over tokens t0 .. t1 - 1 of channel c; Y: y is the projection for the other branch
template <bool Y, class AT, class F>
__device__ __forceinline__ void lru_tokens(const LruArgs &a, const Partial &z, const float *__restrict__ g, const AT *__restrict__ u, int c,
                                           int t0, int t1, F f) {
    const int block = c / a.size, off = c - block * a.size, gld = 2 * a.blocks * a.size_p, uld = a.blocks * a.size_p;
    const float *gr = g + gate_column(a, block, off);
    const AT *uc = u + block * a.size_p + off;
    const float rate = decay_rate(a.p.lam[c]), br = a.p.ra_b[c], bi = a.p.ri_b[c];
    for (int t = t0; t < t1; t += SCAN_U) {
        float r[SCAN_U], i[SCAN_U], x[SCAN_U], y[SCAN_U];
#pragma unroll
        for (int k = 0; k < SCAN_U; ++k) {
            const size_t tt = (size_t)min(t + k, t1 - 1);
            r[k] = gr[tt * gld];
            i[k] = gr[tt * gld + 64];
            x[k] = (float)uc[tt * uld];
            y[k] = Y ? z.p[tt * z.ld + c] : 0.0f;
        }
        for (int q = 1; Y && q < z.copies; ++q) {
#pragma unroll
            for (int k = 0; k < SCAN_U; ++k) y[k] += z.p[(size_t)q * z.stride + (size_t)min(t + k, t1 - 1) * z.ld + c];
        }
#pragma unroll
        for (int k = 0; k < SCAN_U; ++k)
            if (t + k < t1) {
                float aa, bb;
                lru_coefficients(r[k] + br, i[k] + bi, x[k], rate, aa, bb);
                f(t + k, aa, bb, y[k]);
            }
    }
}

// scan: [wp] S in front of the portion, then per chunk [wp] A, [wp] B.  grid (wp / 256, chunks)
template <class AT>
__global__ __launch_bounds__(256) void k_lru_chunks(const LruArgs a, const float *__restrict__ g, const AT *__restrict__ u,
                                                    const float *__restrict__ state, float *__restrict__ scan, int n, int chunk, int fresh) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= a.w) return;
    if (blockIdx.y == 0) scan[c] = fresh ? 0.0f : state[c];
    float A = 1.0f, B = 0.0f;
    const int t0 = blockIdx.y * chunk;
    lru_tokens<false>(a, Partial{}, g, u, c, t0, min(t0 + chunk, n), [&](int, float aa, float bb, float) {
        A *= aa;
        B = fmaf(aa, B, bb);
    });
    float *s = scan + (size_t)(1 + 2 * blockIdx.y) * a.wp + c;
    s[0] = A;
    s[a.wp] = B;
}

template <class AT>
__global__ __launch_bounds__(256) void k_lru_apply(const LruArgs a, const Partial z, const float *__restrict__ g, const AT *__restrict__ u,
                                                   const float *__restrict__ scan, float *__restrict__ state, AT *__restrict__ out, int n,
                                                   int pos0, int chunk) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    const int t0 = blockIdx.y * chunk, t1 = min(t0 + chunk, n);
    if (c >= a.w) {
        for (int t = t0; c < a.out_cols && t < t1; ++t) out[(size_t)t * a.ldo + c] = (AT)0.0f;
        return;
    }
    float S = scan[c];
    const float *s = scan + a.wp + c;
#pragma unroll 8
    for (int k = 0; k < (int)blockIdx.y; ++k, s += 2 * (size_t)a.wp) S = fmaf(s[0], S, s[a.wp]);
    const float by = a.p.by[c];
    lru_tokens<true>(a, z, g, u, c, t0, t1, [&](int t, float aa, float bb, float y) {
        S = fmaf(aa, S, bb);
        out[(size_t)t * a.ldo + c] = (AT)(S * gelu_tanh_f(y + by));
    });
    if (t1 < n) return;
    state[c] = S;
    const float bx = a.p.bx[c];
    for (int t = max(0, n - a.taps); t < n; ++t)
        state[(size_t)(1 + (pos0 + t) % a.taps) * a.wp + c] = z_at(z, (size_t)t, a.wp + c) + bx;
}

// ------------------------------------------------------------------ decode
// grid (blocks, ceil(size / 16)): u of the block in LDS, 16 channels' rows of both gates, a 16-lane group per row
template <class AT>
__global__ __launch_bounds__(256) void k_lru_step(const LruArgs a, const float *__restrict__ z, const bf16 *__restrict__ W,
                                                  float *__restrict__ state, AT *__restrict__ out, const int *__restrict__ pos_ptr) {
    extern __shared__ __align__(16) float us[];   // [size_p]
    __shared__ float gate[32];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15;
    const int b = blockIdx.x, off0 = blockIdx.y * 16, ld = a.size_p;
    // weight rows of this lane's group: number rho = 16 * gate + channel
    const bf16 *w[2];
    u32x4v first[2][2];
#pragma unroll
    for (int it = 0; it < 2; ++it) {
        const int rho = wave * 8 + it * 4 + (lane >> 4);
        w[it] = W + (size_t)(gate_column(a, b, off0 + (rho & 15)) + (rho >> 4) * 64) * ld;
#pragma unroll
        for (int s = 0; s < 2; ++s) first[it][s] = *(const u32x4v *)(w[it] + min(s * 128 + l16 * 8, ld - 8));
    }
    const int pos = *pos_ptr;
    const float *history = state + a.wp;
    for (int i = tid; i < a.size_p; i += 256) {
        float v = 0.0f;
        if (i < a.size) {
            const int c = b * a.size + i;
            v = fmaf(a.p.conv[(size_t)(a.taps - 1) * a.wp + c], z[a.wp + c] + a.p.bx[c], a.p.conv_b[c]);
            for (int j = 1; j < a.taps && j <= pos; ++j)
                v = fmaf(a.p.conv[(size_t)(a.taps - 1 - j) * a.wp + c], history[(size_t)((pos - j) % a.taps) * a.wp + c], v);
        }
        us[i] = v;
    }
    __syncthreads();
    float acc[2] = {0.f, 0.f};
    for (int k0 = 0; k0 < ld; k0 += 128) {
        const int k = k0 + l16 * 8;
        if (k >= ld) break;
        float x[8];
        lds8(us + k, x);
#pragma unroll
        for (int it = 0; it < 2; ++it) {
            float f[8];
            widen8(k0 == 0 ? first[it][0] : k0 == 128 ? first[it][1] : *(const u32x4v *)(w[it] + k), f);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[it] = fmaf(f[e], x[e], acc[it]);
        }
    }
#pragma unroll
    for (int it = 0; it < 2; ++it) {
        const float v = lanes_sum<16>(acc[it]);
        if (l16 == 0) gate[wave * 8 + it * 4 + (lane >> 4)] = v;
    }
    __syncthreads();
    if (tid < 16 && off0 + tid < a.size) {
        const int c = b * a.size + off0 + tid;
        float aa, bb;
        lru_coefficients(gate[tid] + a.p.ra_b[c], gate[16 + tid] + a.p.ri_b[c], us[off0 + tid], decay_rate(a.p.lam[c]), aa, bb);
        const float S = pos > 0 ? fmaf(aa, state[c], bb) : bb;
        state[c] = S;
        state[(size_t)(1 + pos % a.taps) * a.wp + c] = z[a.wp + c] + a.p.bx[c];
        out[c] = (AT)(S * gelu_tanh_f(z[c] + a.p.by[c]));
    }
    if (b == 0 && blockIdx.y == 0)
        for (int i = a.w + tid; i < a.out_cols; i += 256) out[i] = (AT)0.0f;
}

// ------------------------------------------------------------------ host side
int check_lru_spec(const candy_hip_lru_spec &s) {
    CANDY_REQUIRE(s.width > 0 && s.width <= 65536 && s.blocks > 0 && s.width % s.blocks == 0 && s.width / s.blocks <= 8192,
                  "recurrent width %d in %d blocks unsupported", s.width, s.blocks);
    CANDY_REQUIRE(s.taps > 0 && s.taps <= 64, "%d taps unsupported (1 .. 64)", s.taps);
    return CANDY_HIP_OK;
}

static LruArgs lru_args(const LruLayer &A) {
    LruArgs a;
    a.p = A.p;
    a.w = A.s.width; a.wp = (int)pad64(A.s.width); a.blocks = A.s.blocks; a.size = A.s.width / A.s.blocks; a.size_p = (int)pad64(a.size);
    a.taps = A.s.taps; a.out_cols = A.out_cols; a.ldo = A.ldo;
    return a;
}

size_t lru_state_floats(const candy_hip_lru_spec &s) { return (size_t)(1 + s.taps) * pad64(s.width); }
constexpr int MAX_CHUNKS = 64;
size_t lru_scan_floats(const candy_hip_lru_spec &s) { return (size_t)(1 + 2 * MAX_CHUNKS) * pad64(s.width); }
int lru_gate_rows(const candy_hip_lru_spec &s) { return (int)(2 * s.blocks * pad64(s.width / s.blocks)); }

template <class AT>
static int lru_prompt(candy_hip_device *dev, const LruLayer &A, int n, int pos0) {
    const LruArgs a = lru_args(A);
    const int cols = a.blocks * a.size_p;
    CANDY_REQUIRE(A.gates->rows == 2 * cols && A.gates->ld == a.size_p && a.out_cols <= a.wp && (n + CONV_T - 1) / CONV_T <= 65535,
                  "internal: recurrent launch");
    const dim3 gc((unsigned)((cols + 255) / 256), (unsigned)((n + CONV_T - 1) / CONV_T));
    if (a.taps <= CONV_TAPS)
        hipLaunchKernelGGL((k_lru_conv<AT, true>), gc, dim3(256), 0, dev->stream, a, A.z, A.state + a.wp, (AT *)A.u, n, pos0);
    else
        hipLaunchKernelGGL((k_lru_conv<AT, false>), gc, dim3(256), 0, dev->stream, a, A.z, A.state + a.wp, (AT *)A.u, n, pos0);
    CANDY_LAUNCH_CHECK();
    DenseLaunch D;
    D.w = A.gates; D.x = A.u; D.ldx = cols; D.f32 = A.f32; D.m = n; D.block_rows = 2 * a.size_p;
    D.y = A.g; D.ldy = D.n_store = A.gates->rows_pad;
    if (int rc = launch_dense(dev, D)) return rc;
    const int chunk = std::max(16, (n + MAX_CHUNKS - 1) / MAX_CHUNKS), chunks = (n + chunk - 1) / chunk;
    const dim3 g((unsigned)((a.wp + 255) / 256), (unsigned)chunks);
    hipLaunchKernelGGL((k_lru_chunks<AT>), g, dim3(256), 0, dev->stream, a, A.g, (const AT *)A.u, A.state, A.scan, n, chunk, (int)(pos0 == 0));
    CANDY_LAUNCH_CHECK();
    hipLaunchKernelGGL((k_lru_apply<AT>), g, dim3(256), 0, dev->stream, a, A.z, A.g, (const AT *)A.u, A.scan, A.state, (AT *)A.out, n, pos0,
                       chunk);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}
int launch_lru_prompt(candy_hip_device *dev, const LruLayer &A, int n, int pos0) {
    return A.f32 ? lru_prompt<float>(dev, A, n, pos0) : lru_prompt<bf16>(dev, A, n, pos0);
}

template <class AT>
static int lru_step(candy_hip_device *dev, const LruLayer &A, const int *pos_ptr) {
    const LruArgs a = lru_args(A);
    CANDY_REQUIRE(A.z.copies == 1 && A.gates->rows == 2 * a.blocks * a.size_p && A.gates->ld == a.size_p, "internal: recurrent launch");
    hipLaunchKernelGGL((k_lru_step<AT>), dim3((unsigned)a.blocks, (unsigned)((a.size + 15) / 16)), dim3(256), (size_t)a.size_p * 4, dev->stream,
                       a, A.z.p, (const bf16 *)A.gates->data, A.state, (AT *)A.out, pos_ptr);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}
int launch_lru_step(candy_hip_device *dev, const LruLayer &A, const int *pos_ptr) {
    return A.f32 ? lru_step<float>(dev, A, pos_ptr) : lru_step<bf16>(dev, A, pos_ptr);
}

}  // namespace candy

using namespace candy;

extern "C" {

int64_t candy_hip_lru_state_floats(const candy_hip_lru_spec *spec) {
    return spec && check_lru_spec(*spec) == CANDY_HIP_OK ? (int64_t)lru_state_floats(*spec) : 0;
}
int64_t candy_hip_lru_gate_rows(const candy_hip_lru_spec *spec) {
    return spec && check_lru_spec(*spec) == CANDY_HIP_OK ? lru_gate_rows(*spec) : 0;
}

int candy_hip_lru(candy_hip_device *dev, const candy_hip_lru_spec *spec, int act, const float *z, const candy_hip_lru_params *params,
                  const candy_hip_dense *gates, float *state, int64_t n, int32_t pos0, int decode, float *out) {
    CANDY_REQUIRE(dev && spec && params, "nil argument");
    if (int rc = check_lru_spec(*spec)) return rc;
    CANDY_REQUIRE(act == CANDY_HIP_ACT_BF16 || act == CANDY_HIP_ACT_F32, "unknown activation format %d", act);
    CANDY_REQUIRE(n >= 1 && n <= 1 << 17 && pos0 >= 0 && pos0 <= 1 << 30, "invalid positions");
    CANDY_REQUIRE(!decode || n == 1, "the decode kernel takes one token");
    CANDY_REQUIRE(z && gates && state && out && params->by && params->bx && params->conv && params->conv_b && params->ra_b && params->ri_b &&
                      params->lam, "nil pointer");
    CANDY_REQUIRE(gates->dev == dev && gates->rows == lru_gate_rows(*spec) && gates->cols == spec->width / spec->blocks,
                  "gate matrix does not fit the spec");
    if (int rc = use_device(dev)) return rc;
    const bool f32 = act == CANDY_HIP_ACT_F32;
    const size_t es = f32 ? 4 : 2, N = (size_t)n;
    LruLayer A;
    A.s = *spec; A.p = *params; A.gates = gates; A.f32 = f32; A.state = state;
    const int wp = (int)pad64(spec->width);
    auto al = [](size_t b) { return (b + 255) & ~(size_t)255; };
    const size_t u_b = al(N * (gates->rows / 2) * es), g_b = al(N * gates->rows_pad * 4), s_b = al(lru_scan_floats(*spec) * 4), o_b = al(N * wp * es);
    void *ws = nullptr;
    if (int rc = workspace(dev, u_b + g_b + s_b + o_b, &ws)) return rc;
    uint8_t *w = (uint8_t *)ws;
    A.u = w; A.g = (float *)(w + u_b); A.scan = (float *)(w + u_b + g_b); A.out = w + u_b + g_b + s_b;
    A.z.p = z; A.z.ld = 2 * wp;
    A.ldo = A.out_cols = wp;
    if (decode) {
        int *pos = (int *)A.scan;
        if (int rc = candy_hip_h2d(dev, pos, &pos0, sizeof(int))) return rc;
        if (int rc = launch_lru_step(dev, A, pos)) return rc;
    } else {
        if (int rc = launch_lru_prompt(dev, A, (int)n, pos0)) return rc;
    }
    return launch_from_act(dev, f32, A.out, out, n, spec->width, wp);
}

}  // extern "C"
