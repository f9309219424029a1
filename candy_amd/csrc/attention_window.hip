// Attention with a sliding window, capped scores and a sink, over a KV cache whose values are the keys before
// rotation.  Position i sees positions max(0, i - window + 1) .. i; a score is cap * tanh(scale * q.k / cap); the
// softmax denominator of head h also holds exp(sink_h), which has no key and no value.  Rotary positions turn the
// first rope_dims dimensions of a head (pairs i, i + rope_dims / 2), the rest passes.
//   k_rope_cache            projected q and k rows -> rotated q, and the new rows of both caches
//   k_window_attn_row       one wavefront per (query, head), vector ALU: f32 activations, prompt and decode
//   k_window_attn_prompt    bfloat16 prompts on the matrix cores, 64 queries of one head per workgroup
//   k_window_attn_decode    bfloat16 decode: rotation, cache append and attention of the new token, split over the window
//   k_window_attn_merge     its splits and the sink -> the head's output
// Scores, weights and sums are f32; in the bfloat16 prompt kernel the weights meet V as the sum of two bfloat16 parts
// (16 bits of each weight).  (No counterpart in the reference, which composes attention from MatMul / FastSoftmax /
// MatMul, backend.go:78,147, without window, cap or sink.)
#include <algorithm>
#include <cmath>
#include <vector>

#include "dense.h"

namespace candy {

int attn_row(int head_dim) {
    for (int r : {32, 64, 96, 128, 192, 256})
        if (head_dim >= 1 && head_dim <= r) return r;
    return 0;
}

struct RopeArgs {
    const float *qk;
    size_t qk_stride;
    int qk_copies, qk_ld;
    const float *cos_t, *sin_t;
    int H, G, dim, row, half;   // half: rope_dims / 2
    int64_t kv_stride;          // values between kv heads of the cache
};

// element i of projected head `slot` (query heads first) of one token's row, copies summed
__device__ __forceinline__ float qk_at(const RopeArgs &a, const float *token, int slot, int i) {
    const float *p = token + (size_t)slot * a.dim + i;
    float t = p[0];
    for (int c = 1; c < a.qk_copies; ++c) t += p[(size_t)c * a.qk_stride];
    return t;
}
__device__ __forceinline__ float rotated(const RopeArgs &a, const float *token, int slot, int i, int pos, float plain) {
    if (i >= 2 * a.half) return plain;
    const int j = i < a.half ? i : i - a.half;
    const float c = a.cos_t[(size_t)pos * a.half + j], s = a.sin_t[(size_t)pos * a.half + j];
    const float other = qk_at(a, token, slot, i < a.half ? i + a.half : j);
    return i < a.half ? plain * c - other * s : plain * c + other * s;
}

// one thread per (token, head, element of the stored row)
template <class AT>
__global__ __launch_bounds__(256) void k_rope_cache(const RopeArgs a, AT *__restrict__ q, AT *__restrict__ kc, AT *__restrict__ vc,
                                                    int n, int pos0, const int *pos_ptr) {
    const int slots = a.H + a.G;
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= (int64_t)n * slots * a.row) return;
    const int i = (int)(idx % a.row);
    const int slot = (int)(idx / a.row % slots);
    const int t = (int)(idx / ((int64_t)a.row * slots));
    const int pos = (pos_ptr ? *pos_ptr : pos0) + t;
    const float *token = a.qk + (size_t)t * a.qk_ld;
    float plain = 0.0f, turned = 0.0f;
    if (i < a.dim) {
        plain = qk_at(a, token, slot, i);
        turned = rotated(a, token, slot, i, pos, plain);
    }
    if (slot < a.H) {
        q[((size_t)t * a.H + slot) * a.row + i] = (AT)turned;
    } else {
        const size_t off = (size_t)(slot - a.H) * a.kv_stride + (size_t)pos * a.row + i;
        kc[off] = (AT)turned;
        vc[off] = (AT)plain;
    }
}

// The same for heads whose halves are multiples of four values: one thread per four pairs, or four values that pass.
template <class AT>
__global__ __launch_bounds__(256) void k_rope_cache4(const RopeArgs a, AT *__restrict__ q, AT *__restrict__ kc, AT *__restrict__ vc,
                                                     int n, int pos0) {
    typedef AT at4 __attribute__((ext_vector_type(4)));
    const int slots = a.H + a.G, pairs = a.half >> 2, items = pairs + ((a.row - 2 * a.half) >> 2);
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= (int64_t)n * slots * items) return;
    const int item = (int)(idx % items);
    const int slot = (int)(idx / items % slots);
    const int t = (int)(idx / ((int64_t)items * slots));
    const int pos = pos0 + t;
    const float *head = a.qk + (size_t)t * a.qk_ld + (size_t)slot * a.dim;
    auto load = [&](int i) {
        f32x4 v = *(const f32x4 *)(head + i);
        for (int c = 1; c < a.qk_copies; ++c) v += *(const f32x4 *)(head + (size_t)c * a.qk_stride + i);
        return v;
    };
    const bool is_q = slot < a.H;
    const size_t cache = (size_t)(slot - a.H) * a.kv_stride + (size_t)pos * a.row;
    AT *dst = is_q ? q + ((size_t)t * a.H + slot) * a.row : kc + cache;
    if (item < pairs) {
        const int i = item * 4;
        const f32x4 u = load(i), v = load(i + a.half);
        const f32x4 c = *(const f32x4 *)(a.cos_t + (size_t)pos * a.half + i), s = *(const f32x4 *)(a.sin_t + (size_t)pos * a.half + i);
        *(at4 *)(dst + i) = __builtin_convertvector(u * c - v * s, at4);
        *(at4 *)(dst + i + a.half) = __builtin_convertvector(v * c + u * s, at4);
        if (!is_q) {
            *(at4 *)(vc + cache + i) = __builtin_convertvector(u, at4);
            *(at4 *)(vc + cache + i + a.half) = __builtin_convertvector(v, at4);
        }
    } else {
        const int i = 2 * a.half + (item - pairs) * 4;
        const f32x4 u = i < a.dim ? load(i) : f32x4{0.f, 0.f, 0.f, 0.f};
        const at4 o = __builtin_convertvector(u, at4);
        *(at4 *)(dst + i) = o;
        if (!is_q) *(at4 *)(vc + cache + i) = o;
    }
}

struct WindowArgs {
    const float *sink;
    int H, G, dim, row, window, out_cols;
    int64_t kv_stride, ldo;
    float scale, cap;
};

// ------------------------------------------------------------------ one wavefront per (query, head)
__global__ __launch_bounds__(256) void k_window_attn_row(const WindowArgs a, const float *__restrict__ q, const float *__restrict__ kc,
                                                         const float *__restrict__ vc, float *__restrict__ out, int n, int pos0,
                                                         const int *pos_ptr) {
    __shared__ __align__(16) float sq[4][256];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int t = blockIdx.x * 4 + wave, h = blockIdx.y;
    if (t < n)
        for (int i = lane; i < a.row; i += 64) sq[wave][i] = q[((size_t)t * a.H + h) * a.row + i];
    __syncthreads();
    if (t >= n) return;
    const int pos = (pos_ptr ? *pos_ptr : pos0) + t;
    const int lo = max(0, pos - a.window + 1);
    const int g = h / (a.H / a.G);
    const float *kh = kc + (size_t)g * a.kv_stride, *vh = vc + (size_t)g * a.kv_stride;
    float m = a.sink ? a.sink[h] : LOW, l = a.sink ? 1.0f : 0.0f;
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int p0 = lo; p0 <= pos; p0 += 64) {
        const int p = p0 + lane;
        float s = MASKED;
        if (p <= pos) {
            const float *kr = kh + (size_t)p * a.row;
            f32x4 d4{0.f, 0.f, 0.f, 0.f};
            for (int i = 0; i < a.row; i += 4) d4 += *(const f32x4 *)&sq[wave][i] * *(const f32x4 *)(kr + i);
            s = ((d4[0] + d4[1]) + (d4[2] + d4[3])) * a.scale;
            if (a.cap > 0.0f) s = a.cap * tanhf(s / a.cap);
        }
        const float m_new = fmaxf(m, wave_max(s));
        const float corr = expf(m - m_new);
        const float w = p <= pos ? expf(s - m_new) : 0.0f;
        l = l * corr + wave_sum(w);
        m = m_new;
#pragma unroll
        for (int c = 0; c < 4; ++c) o[c] *= corr;
        const int cnt = min(64, pos - p0 + 1);
        for (int j = 0; j < cnt; ++j) {
            const float wj = __shfl(w, j, 64);
            const float *vr = vh + (size_t)(p0 + j) * a.row;
#pragma unroll
            for (int c = 0; c < 4; ++c)
                if (lane + 64 * c < a.row) o[c] = fmaf(wj, vr[lane + 64 * c], o[c]);
        }
    }
    float *dst = out + (size_t)t * a.ldo;
#pragma unroll
    for (int c = 0; c < 4; ++c)
        if (lane + 64 * c < a.dim) dst[(size_t)h * a.dim + lane + 64 * c] = o[c] / l;
    if (h == a.H - 1)
        for (int i = a.H * a.dim + lane; i < a.out_cols; i += 64) dst[i] = 0.0f;
}

// ------------------------------------------------------------------ prompts, bfloat16, matrix cores
// grid (heads, ceil(n / 64)), 4 wavefronts of 16 queries, keys in tiles of 64 through LDS.  The scores are computed
// transposed (keys x queries), so that a lane holds scores of one query only (16 of a tile's 64; the four lanes 16
// apart share the query) and hands them to the second product from registers: its K index 8 g + e stands for key
// 4 g + e of one 16-key tile (e < 4) or of the next (e >= 4), and V is stored transposed in LDS in that key order.
template <int DP>
__global__ __launch_bounds__(256, 2) void k_window_attn_prompt(const WindowArgs a, const bf16 *__restrict__ q, const bf16 *__restrict__ kc,
                                                               const bf16 *__restrict__ vc, bf16 *__restrict__ out, int n, int pos0) {
    constexpr int QT = 64, KT = 64, KP = DP + 8, VP = KT + 8, C8 = DP / 8;
    constexpr int K_IT = (KT * C8 + 255) / 256, V_IT = (KT / 2 * C8 + 255) / 256;
    __shared__ __align__(16) bf16 s_k[KT * KP];
    __shared__ __align__(16) bf16 s_v[DP * VP];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int r16 = lane & 15, g = lane >> 4;
    const int h = blockIdx.x, i0 = blockIdx.y * QT;
    const int kvh = h / (a.H / a.G);
    const bf16 *kh = kc + (size_t)kvh * a.kv_stride, *vh = vc + (size_t)kvh * a.kv_stride;
    const int last = pos0 + min(i0 + QT, n) - 1;                 // last position the workgroup's queries see
    const int first = max(0, pos0 + i0 - a.window + 1);           // first
    const int qi = i0 + 16 * wave + r16;                          // this lane's query
    const int qpos = pos0 + qi;
    const int wq0 = pos0 + i0 + 16 * wave, wq1 = wq0 + 15;        // the wavefront's queries
    bf16x8 qf[DP / 32];
#pragma unroll
    for (int ks = 0; ks < DP / 32; ++ks)
        qf[ks] = *(const bf16x8 *)(q + ((size_t)min(qi, n - 1) * a.H + h) * DP + ks * 32 + g * 8);
    float m = a.sink ? a.sink[h] * LOG2E : LOW, l = a.sink ? (g == 0 ? 1.0f : 0.0f) : 0.0f;  // l: summed over g at the end
    f32x4 o[DP / 16];
#pragma unroll
    for (int d = 0; d < DP / 16; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};

    u32x4v kreg[K_IT], vreg[V_IT][2];
    auto request = [&](int p0) __attribute__((always_inline)) {
#pragma unroll
        for (int it = 0; it < K_IT; ++it) {
            const int e = tid + it * 256, key = e / C8, c = e % C8;
            if (K_IT * 256 == KT * C8 || e < KT * C8) kreg[it] = *(const u32x4v *)(kh + (size_t)min(p0 + key, last) * DP + c * 8);
        }
#pragma unroll
        for (int it = 0; it < V_IT; ++it) {
            const int e = tid + it * 256, kp = e & 31, c = e >> 5;
            if (V_IT * 256 == KT / 2 * C8 || e < KT / 2 * C8) {
                vreg[it][0] = *(const u32x4v *)(vh + (size_t)min(p0 + 2 * kp, last) * DP + c * 8);
                vreg[it][1] = *(const u32x4v *)(vh + (size_t)min(p0 + 2 * kp + 1, last) * DP + c * 8);
            }
        }
    };
    const float c_in = a.cap > 0.0f ? a.scale / a.cap : a.scale * LOG2E, c_out = a.cap * LOG2E;
    const int p_first = first & ~(KT - 1);
    request(p_first);
    for (int p0 = p_first; p0 <= last; p0 += KT) {
        __syncthreads();  // the previous tile is consumed
#pragma unroll
        for (int it = 0; it < K_IT; ++it) {
            const int e = tid + it * 256, key = e / C8, c = e % C8;
            if (K_IT * 256 == KT * C8 || e < KT * C8) *(u32x4v *)&s_k[key * KP + c * 8] = kreg[it];
        }
#pragma unroll
        for (int it = 0; it < V_IT; ++it) {
            const int e = tid + it * 256, kp = e & 31, c = e >> 5;
            if (V_IT * 256 == KT / 2 * C8 || e < KT / 2 * C8) {
                // keys 2kp, 2kp+1 of their 32-key block: key 16 hh + 4 gg + ee sits at 8 gg + 4 hh + ee
                const int k32 = 2 * kp & 31;
                const int at = (2 * kp & 32) + ((k32 >> 2) & 3) * 8 + (k32 >> 4) * 4 + (k32 & 3);
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const uint32_t w0 = vreg[it][0][j >> 1], w1 = vreg[it][1][j >> 1];
                    const uint32_t lo = j & 1 ? w0 >> 16 : w0 & 0xFFFFu, hi = j & 1 ? w1 & 0xFFFF0000u : w1 << 16;
                    *(uint32_t *)&s_v[(c * 8 + j) * VP + at] = lo | hi;
                }
            }
        }
        if (p0 + KT <= last) request(p0 + KT);
        __syncthreads();
        if (p0 > wq1 || p0 + KT - 1 <= wq0 - a.window) continue;  // nothing of the tile is visible to these 16 queries
        f32x4 s[4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
            s[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DP / 32; ++ks)
                s[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8 *)&s_k[(kt * 16 + r16) * KP + ks * 32 + g * 8], qf[ks],
                                                                s[kt], 0, 0, 0);
        }
        const bool whole = p0 + KT - 1 <= wq0 && p0 > wq1 - a.window;  // every key visible to every query
        float mx = MASKED;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                float z = s[kt][j] * c_in;
                if (a.cap > 0.0f) z = c_out * tanh_fast(z);
                if (!whole) {
                    const int p = p0 + kt * 16 + 4 * g + j;
                    z = p <= qpos && p > qpos - a.window ? z : MASKED;
                }
                s[kt][j] = z;
                mx = fmaxf(mx, z);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m, mx);
        const float corr = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        float sum = 0.0f;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                s[kt][j] = __builtin_amdgcn_exp2f(s[kt][j] - m_new);
                sum += s[kt][j];
            }
        l = l * corr + sum;
        if (__any(corr != 1.0f)) {
#pragma unroll
            for (int d = 0; d < DP / 16; ++d) o[d] *= corr;
        }
#pragma unroll
        for (int kb = 0; kb < 2; ++kb) {
            bf16x8 hi, lo;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const float w = s[2 * kb + (e >> 2)][e & 3];
                hi[e] = (bf16)w;
                lo[e] = (bf16)(w - (float)hi[e]);
            }
#pragma unroll
            for (int d = 0; d < DP / 16; ++d) {
                const bf16x8 vt = *(const bf16x8 *)&s_v[(d * 16 + r16) * VP + kb * 32 + g * 8];
                o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, lo, o[d], 0, 0, 0);
                o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, hi, o[d], 0, 0, 0);
            }
        }
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (qi >= n) return;
    const float inv = 1.0f / l;
    bf16 *dst = out + (size_t)qi * a.ldo + (size_t)h * a.dim;
#pragma unroll
    for (int d = 0; d < DP / 16; ++d) {
        const int c = d * 16 + 4 * g;
        const f32x4 v = o[d] * inv;
        if ((a.dim & 3) == 0) {
            if (c < a.dim) *(bf16x4 *)(dst + c) = __builtin_convertvector(v, bf16x4);
        } else {
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (c + j < a.dim) dst[c + j] = (bf16)v[j];
        }
    }
    if (h == a.H - 1)
        for (int i = a.H * a.dim + g; i < a.out_cols; i += 4) out[(size_t)qi * a.ldo + i] = (bf16)0.0f;
}

// ------------------------------------------------------------------ decode, bfloat16
// grid (kv heads, splits, chunks of GROUP query heads of the kv head), 4 wavefronts.  LPR lanes hold one cache row (8
// values each); a wavefront takes 64 / LPR rows per load, UNR loads per batch; batches of the window are dealt to the
// splits round robin.  The new token's rows do not go through memory: split 0 rotates and appends them, and its first
// wavefront attends to them from LDS.
constexpr int DEC_UNR = 4;

template <int LPR> constexpr int dec_batch() { return 4 * (64 / LPR) * DEC_UNR; }

template <int LPR, int GROUP>
__global__ __launch_bounds__(256) void k_window_attn_decode(const WindowArgs a, const RopeArgs ra, bf16 *kc, bf16 *vc,
                                                            const int *__restrict__ pos_ptr, float *__restrict__ part, int n_splits) {
    constexpr int RPW = 64 / LPR, BATCH = dec_batch<LPR>(), W = LPR * 8, SLOTS = 4 * RPW;
    __shared__ __align__(16) float sq[GROUP + 2][W];   // rotated queries, then the new token's key and value
    __shared__ float sm[SLOTS][GROUP], sl[SLOTS][GROUP], tot[GROUP][2];
    __shared__ __align__(16) float so[SLOTS][GROUP][W];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int kvh = blockIdx.x, split = blockIdx.y, ratio = a.H / a.G, h0 = blockIdx.z * GROUP;
    const int rl = lane / LPR, cl = lane % LPR;       // row of a load, chunk of the row
    const bool chunk = cl * 8 < a.row;                // rows narrower than LPR chunks leave lanes idle
    const int coff = chunk ? cl * 8 : 0;
    bf16 *kh = kc + (size_t)kvh * a.kv_stride, *vh = vc + (size_t)kvh * a.kv_stride;
    const bool fresh = split == 0;
    // Requested in the order they become possible: the projected rows at once, what depends on the position behind it,
    // the cache rows last, so that the rotation below does not wait for them.
    constexpr int PER = ((GROUP + 2) * W + 255) / 256;
    const int rows = GROUP + (fresh ? 2 : 0);
    float plain[PER], other[PER];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
        const int i = tid + 256 * j, r = i / W, c = i % W;
        const bool used = r < rows && c < a.dim;
        const float *head = ra.qk + (size_t)(r < GROUP ? kvh * ratio + min(h0 + r, ratio - 1) : a.H + kvh) * a.dim;
        plain[j] = used ? head[c] : 0.0f;
        other[j] = used && c < 2 * ra.half ? head[c < ra.half ? c + ra.half : c - ra.half] : 0.0f;
    }
    const int pos = *pos_ptr;
    const int lo = max(0, pos - a.window + 1);        // positions lo .. pos-1 are in the cache
    const int cached = pos - lo;
    float cs[PER], sn[PER];
#pragma unroll
    for (int j = 0; j < PER; ++j) {
        const int i = tid + 256 * j, r = i / W, c = i % W;
        const bool used = r <= GROUP && r < rows && c < 2 * ra.half;
        const size_t at = (size_t)pos * ra.half + (c < ra.half ? c : c - ra.half);
        cs[j] = used ? ra.cos_t[at] : 1.0f;
        sn[j] = used ? ra.sin_t[at] : 0.0f;
    }
    u32x4v kv[DEC_UNR], vv[DEC_UNR];
    auto fetch = [&](int b) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < DEC_UNR; ++u) {
            const int p = b * BATCH + (wave * DEC_UNR + u) * RPW + rl;
            const size_t off = (size_t)(lo + max(min(p, cached - 1), 0)) * a.row + coff;
            kv[u] = __builtin_nontemporal_load((const u32x4v *)(kh + off));
            vv[u] = __builtin_nontemporal_load((const u32x4v *)(vh + off));
        }
    };
    fetch(split);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int j = 0; j < PER; ++j) {
        const int i = tid + 256 * j, r = i / W, c = i % W;
        if (r >= rows) continue;
        float v = c < ra.half ? plain[j] * cs[j] - other[j] * sn[j] : plain[j] * cs[j] + other[j] * sn[j];
        if (r >= GROUP) {
            const bf16 b = (bf16)v;  // attend to the rows as the cache holds them
            v = (float)b;
            if (blockIdx.z == 0 && c < a.row) (r == GROUP ? kh : vh)[(size_t)pos * a.row + c] = b;
        }
        sq[r][c] = v;
    }
    __syncthreads();
    const float c_in = a.cap > 0.0f ? a.scale / a.cap : a.scale * LOG2E, c_out = a.cap * LOG2E;
    float qf[GROUP][8], m[GROUP], l[GROUP], o[GROUP][8];
#pragma unroll
    for (int q = 0; q < GROUP; ++q) {
        m[q] = LOW;
        l[q] = 0.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            qf[q][e] = chunk ? sq[q][cl * 8 + e] * c_in : 0.0f;
            o[q][e] = 0.0f;
        }
    }
    auto score = [&](const float (&k)[8], int q) __attribute__((always_inline)) {
        float d = 0.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) d = fmaf(qf[q][e], k[e], d);
        d = lanes_sum<LPR>(d);
        return a.cap > 0.0f ? c_out * tanh_fast(d) : d;
    };
    for (int b = split; b * BATCH < cached; b += n_splits) {
        float kf[DEC_UNR][8], vf[DEC_UNR][8];
        bool valid[DEC_UNR];
#pragma unroll
        for (int u = 0; u < DEC_UNR; ++u) {
            const u32x4v kw = kv[u], vw = vv[u];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                kf[u][2 * i] = __uint_as_float(kw[i] << 16);
                kf[u][2 * i + 1] = __uint_as_float(kw[i] & 0xFFFF0000u);
                vf[u][2 * i] = __uint_as_float(vw[i] << 16);
                vf[u][2 * i + 1] = __uint_as_float(vw[i] & 0xFFFF0000u);
            }
            valid[u] = b * BATCH + (wave * DEC_UNR + u) * RPW + rl < cached;
        }
        if ((b + n_splits) * BATCH < cached) fetch(b + n_splits);
#pragma unroll
        for (int q = 0; q < GROUP; ++q) {
            float s[DEC_UNR], m_new = m[q];
#pragma unroll
            for (int u = 0; u < DEC_UNR; ++u) {
                s[u] = score(kf[u], q);
                if (!valid[u]) s[u] = MASKED;
                m_new = fmaxf(m_new, s[u]);
            }
            const float corr = __builtin_amdgcn_exp2f(m[q] - m_new);
            m[q] = m_new;
            l[q] *= corr;
#pragma unroll
            for (int e = 0; e < 8; ++e) o[q][e] *= corr;
#pragma unroll
            for (int u = 0; u < DEC_UNR; ++u) {
                const float w = __builtin_amdgcn_exp2f(s[u] - m_new);
                l[q] += w;
#pragma unroll
                for (int e = 0; e < 8; ++e) o[q][e] = fmaf(w, vf[u][e], o[q][e]);
            }
        }
    }
    if (fresh && wave == 0) {  // the new token, by the lanes of the first row
        float kn[8], vn[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            kn[e] = sq[GROUP][cl * 8 + e];
            vn[e] = sq[GROUP + 1][cl * 8 + e];
        }
#pragma unroll
        for (int q = 0; q < GROUP; ++q) {
            float s = score(kn, q);
            if (rl != 0) s = MASKED;
            const float m_new = fmaxf(m[q], s);
            const float corr = __builtin_amdgcn_exp2f(m[q] - m_new), w = __builtin_amdgcn_exp2f(s - m_new);
            m[q] = m_new;
            l[q] = l[q] * corr + w;
#pragma unroll
            for (int e = 0; e < 8; ++e) o[q][e] = fmaf(w, vn[e], o[q][e] * corr);
        }
    }
    const int slot = wave * RPW + rl;
#pragma unroll
    for (int q = 0; q < GROUP; ++q) {
        if (cl == 0) {
            sm[slot][q] = m[q];
            sl[slot][q] = l[q];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) so[slot][q][cl * 8 + e] = o[q][e];
    }
    __syncthreads();
    // a wavefront's lanes hold one slot each: the factor of every slot, once
    for (int q = wave; q < GROUP; q += 4) {
        const float ms = lane < SLOTS ? sm[lane][q] : LOW;
        const float mm = wave_max(ms), f = __builtin_amdgcn_exp2f(ms - mm);
        const float ll = wave_sum(lane < SLOTS ? sl[lane][q] * f : 0.0f);
        if (lane < SLOTS) sm[lane][q] = f;
        if (lane == 0) {
            tot[q][0] = mm;
            tot[q][1] = ll;
        }
    }
    __syncthreads();
    for (int i = tid; i < GROUP * W; i += 256) {
        const int q = i / W, c = i % W;
        if (h0 + q >= ratio || c >= a.row) continue;
        float oo = 0.0f;
#pragma unroll
        for (int s = 0; s < SLOTS; ++s) oo += so[s][q][c] * sm[s][q];
        // per (head, split): row values, then the maximum and the sum
        float *p = part + ((size_t)(kvh * ratio + h0 + q) * n_splits + split) * (a.row + 4);
        p[c] = oo;
        if (c == 0) {
            p[a.row] = tot[q][0];
            p[a.row + 1] = tot[q][1];
        }
    }
}

// one workgroup per head; at most 64 splits, a lane each for the maxima
__global__ __launch_bounds__(256) void k_window_attn_merge(const WindowArgs a, const float *__restrict__ part, int n_splits,
                                                           bf16 *__restrict__ out) {
    constexpr int MAX_SPLITS = 64;
    __shared__ __align__(16) f32x4 red[256];
    const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63;
    // the head's partial outputs as 16-byte loads: thread (sg, c4) takes columns 4 c4 .. of splits sg, sg + SG, ...
    const int pitch = a.row + 4, C4 = a.row >> 2, SG = 256 / C4, c4 = tid % C4, sg = tid / C4;
    const float *p = part + (size_t)h * n_splits * pitch;
    float ms = LOW, ls = 0.0f;
    if (lane < n_splits) {
        ms = p[(size_t)lane * pitch + a.row];
        ls = p[(size_t)lane * pitch + a.row + 1];
    }
    const float sink = a.sink ? a.sink[h] * LOG2E : MASKED;
    constexpr int AHEAD = 8;
    f32x4 v[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) v[j] = *(const f32x4 *)(p + (size_t)min(sg + SG * j, n_splits - 1) * pitch + 4 * c4);
    __builtin_amdgcn_sched_barrier(0);  // every load above is requested before anything below waits
    const float m = fmaxf(wave_max(ms), sink);
    const float w = lane < n_splits ? __builtin_amdgcn_exp2f(ms - m) : 0.0f;
    const float l = wave_sum(ls * w) + (a.sink ? __builtin_amdgcn_exp2f(sink - m) : 0.0f);
    const float f = w / l;
    f32x4 o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) {
        const int s = sg + SG * j;
        const float fs = __shfl(f, min(s, 63), 64);
        o += v[j] * (s < n_splits ? fs : 0.0f);
    }
    for (int j = AHEAD; SG * j < MAX_SPLITS; ++j) {
        const int s = sg + SG * j;
        const float fs = __shfl(f, min(s, 63), 64);
        if (s < n_splits) o += *(const f32x4 *)(p + (size_t)s * pitch + 4 * c4) * fs;
    }
    red[tid] = o;
    __syncthreads();
    for (int c = tid; c < a.dim; c += 256) {
        float t = 0.0f;
        for (int g = 0; g < SG; ++g) t += red[g * C4 + (c >> 2)][c & 3];
        out[(size_t)h * a.dim + c] = (bf16)t;
    }
    if (h == a.H - 1)
        for (int i = a.H * a.dim + tid; i < a.out_cols; i += 256) out[i] = (bf16)0.0f;
}

// ------------------------------------------------------------------ host side
int check_attn_spec(const candy_hip_attn_spec &s) {
    CANDY_REQUIRE(s.n_heads > 0 && s.n_kv_heads > 0 && s.n_heads % s.n_kv_heads == 0 && s.n_heads <= 65535,
                  "invalid head counts %d / %d", s.n_heads, s.n_kv_heads);
    CANDY_REQUIRE(attn_row(s.head_dim) != 0, "head_dim %d unsupported (1 .. 256)", s.head_dim);
    CANDY_REQUIRE(s.window >= 0, "negative window");
    CANDY_REQUIRE(s.rope_dims >= 0 && s.rope_dims % 2 == 0 && s.rope_dims <= s.head_dim, "rope_dims %d must be even and within head_dim %d",
                  s.rope_dims, s.head_dim);
    CANDY_REQUIRE(s.rope_dims == 0 || s.rope_base > 0, "rope_base must be positive");
    CANDY_REQUIRE(s.rope_original >= 0 && (s.rope_original == 0 || (s.rope_factor > 0 && s.rope_low > 0 && s.rope_high > s.rope_low)),
                  "invalid rotary frequency scaling");
    CANDY_REQUIRE(s.softcap >= 0, "negative score cap");
    return CANDY_HIP_OK;
}

void fill_rope_tables(const candy_hip_attn_spec &s, int max_pos, float *cos_t, float *sin_t) {
    const int half = s.rope_dims / 2;
    const double two_pi = 6.283185307179586476925286766559;
    std::vector<double> f((size_t)half);
    for (int i = 0; i < half; ++i) {
        double v = std::pow(s.rope_base, -2.0 * i / s.rope_dims);
        if (s.rope_original > 0) {
            const double turns = s.rope_original * v / two_pi;  // original context / wavelength
            if (turns < s.rope_low) v /= s.rope_factor;
            else if (turns <= s.rope_high) {
                const double mix = (turns - s.rope_low) / (s.rope_high - s.rope_low);
                v = (1.0 - mix) * v / s.rope_factor + mix * v;
            }
        }
        f[(size_t)i] = v;
    }
    for (int p = 0; p < max_pos; ++p)
        for (int i = 0; i < half; ++i) {
            cos_t[(size_t)p * half + i] = (float)std::cos(p * f[(size_t)i]);
            sin_t[(size_t)p * half + i] = (float)std::sin(p * f[(size_t)i]);
        }
}

static int lanes_per_row(int row) { return row <= 32 ? 4 : row <= 64 ? 8 : row <= 128 ? 16 : 32; }
static int group_of(const candy_hip_attn_spec &s) {
    const int ratio = s.n_heads / s.n_kv_heads;
    return ratio >= 3 ? 4 : ratio;
}

int window_splits(const candy_hip_device *dev, const candy_hip_attn_spec &s, int max_pos) {
    const int range = s.window > 0 ? std::min(s.window, max_pos) : max_pos;
    const int lpr = lanes_per_row(attn_row(s.head_dim)), batch = 4 * (64 / lpr) * DEC_UNR;
    const int chunks = (s.n_heads / s.n_kv_heads + group_of(s) - 1) / group_of(s);
    const int64_t fill = (4 * (int64_t)dev->num_cus + s.n_kv_heads * chunks - 1) / (s.n_kv_heads * chunks);
    const int64_t n = std::min<int64_t>(std::min<int64_t>(fill, (range + batch - 1) / batch), 64);
    return n < 1 ? 1 : (int)n;
}

size_t window_scratch_floats(const candy_hip_attn_spec &s, int n_splits) {
    return (size_t)s.n_heads * n_splits * (attn_row(s.head_dim) + 4);
}

static WindowArgs window_args(const WindowAttn &A) {
    WindowArgs a;
    a.sink = A.sink;
    a.H = A.s.n_heads; a.G = A.s.n_kv_heads; a.dim = A.s.head_dim; a.row = A.row;
    a.window = A.s.window > 0 ? A.s.window : 0x3FFFFFFF;
    a.out_cols = A.out_cols;
    a.kv_stride = (int64_t)A.max_pos * A.row;
    a.ldo = A.ldo;
    a.scale = A.s.scale; a.cap = A.s.softcap;
    return a;
}

static RopeArgs rope_args(const WindowAttn &A) {
    RopeArgs a;
    a.qk = A.qk.p; a.qk_stride = A.qk.stride; a.qk_copies = A.qk.copies; a.qk_ld = A.qk.ld;
    a.cos_t = A.cos_t; a.sin_t = A.sin_t;
    a.H = A.s.n_heads; a.G = A.s.n_kv_heads; a.dim = A.s.head_dim; a.row = A.row; a.half = A.s.rope_dims / 2;
    a.kv_stride = (int64_t)A.max_pos * A.row;
    return a;
}

static int launch_rope(candy_hip_device *dev, const WindowAttn &A, int n, int pos0, const int *pos_ptr) {
    const RopeArgs ra = rope_args(A);
    if (!pos_ptr && A.s.head_dim % 4 == 0 && ra.half % 4 == 0 && ra.qk_ld % 4 == 0 && ((uintptr_t)ra.qk & 15) == 0 && ra.qk_stride % 4 == 0) {
        const int64_t items = (ra.half >> 2) + ((A.row - 2 * ra.half) >> 2);
        const int64_t grid = ((int64_t)n * (ra.H + ra.G) * items + 255) / 256;
        CANDY_REQUIRE(grid <= 0x7FFFFFFF, "prompt too long for one pass");
        if (A.f32)
            hipLaunchKernelGGL((k_rope_cache4<float>), dim3((unsigned)grid), dim3(256), 0, dev->stream, ra, (float *)A.q,
                               (float *)A.k_cache, (float *)A.v_cache, n, pos0);
        else
            hipLaunchKernelGGL((k_rope_cache4<bf16>), dim3((unsigned)grid), dim3(256), 0, dev->stream, ra, (bf16 *)A.q,
                               (bf16 *)A.k_cache, (bf16 *)A.v_cache, n, pos0);
        CANDY_LAUNCH_CHECK();
        return CANDY_HIP_OK;
    }
    const int64_t grid = ((int64_t)n * (A.s.n_heads + A.s.n_kv_heads) * A.row + 255) / 256;
    CANDY_REQUIRE(grid <= 0x7FFFFFFF, "prompt too long for one pass");
    if (A.f32)
        hipLaunchKernelGGL((k_rope_cache<float>), dim3((unsigned)grid), dim3(256), 0, dev->stream, ra, (float *)A.q,
                           (float *)A.k_cache, (float *)A.v_cache, n, pos0, pos_ptr);
    else
        hipLaunchKernelGGL((k_rope_cache<bf16>), dim3((unsigned)grid), dim3(256), 0, dev->stream, ra, (bf16 *)A.q,
                           (bf16 *)A.k_cache, (bf16 *)A.v_cache, n, pos0, pos_ptr);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

static int launch_rows(candy_hip_device *dev, const WindowAttn &A, int n, int pos0, const int *pos_ptr) {
    hipLaunchKernelGGL(k_window_attn_row, dim3((unsigned)((n + 3) / 4), (unsigned)A.s.n_heads), dim3(256), 0, dev->stream,
                       window_args(A), (const float *)A.q, (const float *)A.k_cache, (const float *)A.v_cache, (float *)A.out, n,
                       pos0, pos_ptr);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

int launch_window_prompt(candy_hip_device *dev, const WindowAttn &A, int n, int pos0) {
    if (int rc = launch_rope(dev, A, n, pos0, nullptr)) return rc;
    if (A.f32) return launch_rows(dev, A, n, pos0, nullptr);
    CANDY_REQUIRE((n + 63) / 64 <= 65535, "prompt too long for one pass");
    const dim3 g((unsigned)A.s.n_heads, (unsigned)((n + 63) / 64)), b(256);
    const WindowArgs a = window_args(A);
#define CANDY_WP(DP)                                                                                                              \
    case DP:                                                                                                                      \
        hipLaunchKernelGGL((k_window_attn_prompt<DP>), g, b, 0, dev->stream, a, (const bf16 *)A.q, (const bf16 *)A.k_cache,        \
                           (const bf16 *)A.v_cache, (bf16 *)A.out, n, pos0);                                                      \
        break
    switch (A.row) {
        CANDY_WP(32); CANDY_WP(64); CANDY_WP(96); CANDY_WP(128); CANDY_WP(192); CANDY_WP(256);
    default: return fail(CANDY_HIP_ERR_UNSUPPORTED, "no attention kernel for rows of %d values", A.row);
    }
#undef CANDY_WP
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

template <int LPR>
static void launch_dec(candy_hip_device *dev, const WindowAttn &A, int group, const int *pos_ptr) {
    const int ratio = A.s.n_heads / A.s.n_kv_heads;
    const dim3 g((unsigned)A.s.n_kv_heads, (unsigned)A.n_splits, (unsigned)((ratio + group - 1) / group)), b(256);
    const WindowArgs a = window_args(A);
    const RopeArgs ra = rope_args(A);
    bf16 *k = (bf16 *)A.k_cache, *v = (bf16 *)A.v_cache;
    switch (group) {
    case 1: hipLaunchKernelGGL((k_window_attn_decode<LPR, 1>), g, b, 0, dev->stream, a, ra, k, v, pos_ptr, A.part, A.n_splits); break;
    case 2: hipLaunchKernelGGL((k_window_attn_decode<LPR, 2>), g, b, 0, dev->stream, a, ra, k, v, pos_ptr, A.part, A.n_splits); break;
    default: hipLaunchKernelGGL((k_window_attn_decode<LPR, 4>), g, b, 0, dev->stream, a, ra, k, v, pos_ptr, A.part, A.n_splits); break;
    }
}

int launch_window_decode(candy_hip_device *dev, const WindowAttn &A, const int *pos_ptr) {
    if (A.f32) {
        if (int rc = launch_rope(dev, A, 1, 0, pos_ptr)) return rc;
        return launch_rows(dev, A, 1, 0, pos_ptr);
    }
    CANDY_REQUIRE(A.n_splits >= 1 && A.n_splits <= 64 && A.qk.copies == 1, "internal: attention launch");
    const int group = group_of(A.s);
    switch (lanes_per_row(A.row)) {
    case 4: launch_dec<4>(dev, A, group, pos_ptr); break;
    case 8: launch_dec<8>(dev, A, group, pos_ptr); break;
    case 16: launch_dec<16>(dev, A, group, pos_ptr); break;
    default: launch_dec<32>(dev, A, group, pos_ptr); break;
    }
    CANDY_LAUNCH_CHECK();
    hipLaunchKernelGGL(k_window_attn_merge, dim3((unsigned)A.s.n_heads), dim3(256), 0, dev->stream, window_args(A), A.part, A.n_splits,
                       (bf16 *)A.out);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

__global__ void k_store_pos(int *dst, int pos) { *dst = pos; }

}  // namespace candy

using namespace candy;

extern "C" {

int candy_hip_attn_row(int head_dim) { return attn_row(head_dim); }

int candy_hip_window_attention(candy_hip_device *dev, const candy_hip_attn_spec *spec, int act, const float *qk, int64_t n,
                               int32_t pos0, int32_t max_pos, void *k_cache, void *v_cache, const float *sink, int decode,
                               float *out) {
    CANDY_REQUIRE(dev && spec, "nil argument");
    if (int rc = check_attn_spec(*spec)) return rc;
    CANDY_REQUIRE(act == CANDY_HIP_ACT_BF16 || act == CANDY_HIP_ACT_F32, "unknown activation format %d", act);
    CANDY_REQUIRE(n >= 1 && n <= 1 << 20 && pos0 >= 0 && pos0 + n <= max_pos, "positions %d .. %lld outside the cache (max_pos %d)", pos0,
                  (long long)(pos0 + n - 1), max_pos);
    CANDY_REQUIRE(!decode || n == 1, "the decode kernels take one token");
    CANDY_REQUIRE(qk && k_cache && v_cache && out, "nil pointer");
    CANDY_REQUIRE(((uintptr_t)k_cache & 15) == 0 && ((uintptr_t)v_cache & 15) == 0, "caches must be 16-byte aligned");
    if (int rc = use_device(dev)) return rc;
    const bool f32 = act == CANDY_HIP_ACT_F32;
    WindowAttn A;
    A.s = *spec;
    A.row = attn_row(spec->head_dim);
    A.max_pos = max_pos;
    A.f32 = f32;
    A.n_splits = window_splits(dev, *spec, max_pos);
    const int width = spec->n_heads * spec->head_dim, half = spec->rope_dims / 2;
    const size_t es = f32 ? 4 : 2;
    auto al = [](size_t b) { return (b + 255) & ~(size_t)255; };
    const size_t q_b = al((size_t)n * spec->n_heads * A.row * es), o_b = al((size_t)n * width * es),
                 p_b = al(window_scratch_floats(*spec, A.n_splits) * 4), t_b = al((size_t)max_pos * half * 4 + 4);
    void *ws = nullptr;
    if (int rc = workspace(dev, q_b + o_b + p_b + 2 * t_b + 256, &ws)) return rc;
    uint8_t *w = (uint8_t *)ws;
    A.q = w; A.out = w + q_b; A.part = (float *)(w + q_b + o_b);
    float *ct = (float *)(w + q_b + o_b + p_b), *st = (float *)(w + q_b + o_b + p_b + t_b);
    int *pos = (int *)(w + q_b + o_b + p_b + 2 * t_b);
    std::vector<float> hc((size_t)max_pos * half + 1), hs((size_t)max_pos * half + 1);
    fill_rope_tables(*spec, max_pos, hc.data(), hs.data());
    if (int rc = candy_hip_h2d(dev, ct, hc.data(), (size_t)max_pos * half * 4)) return rc;
    if (int rc = candy_hip_h2d(dev, st, hs.data(), (size_t)max_pos * half * 4)) return rc;
    A.cos_t = ct; A.sin_t = st; A.sink = sink; A.k_cache = k_cache; A.v_cache = v_cache;
    A.qk.p = qk; A.qk.ld = (spec->n_heads + spec->n_kv_heads) * spec->head_dim;
    A.ldo = width; A.out_cols = width;
    if (decode) {
        hipLaunchKernelGGL(k_store_pos, dim3(1), dim3(1), 0, dev->stream, pos, (int)pos0);
        CANDY_LAUNCH_CHECK();
        if (int rc = launch_window_decode(dev, A, pos)) return rc;
    } else if (int rc = launch_window_prompt(dev, A, (int)n, pos0)) {
        return rc;
    }
    return launch_from_act(dev, f32, A.out, out, n, width, width);
}

}  // extern "C"
