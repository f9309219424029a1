// Latent attention: a position's cache row is a normed latent c and a rotated key part shared by all heads (layout and
// equations: include/candy_hip.h).
//   k_latent_rows          projected rows -> normed query latents, normed latent and rotated key part into the cache
//   k_latent_prompt        bfloat16 prompts on the matrix cores over expanded keys and values, 64 queries of a head per workgroup
//   k_latent_prompt_row    one wavefront per (query, head), vector ALU: f32 prompts, and heads too wide for the tiles
//   k_latent_query         decode: queries contracted with Wuk, rotated part turned, the new cache row appended
//   k_latent_decode        bfloat16 decode on the matrix cores: 16 heads against the cached rows, split over the positions
//   k_latent_decode_row    the same, one wavefront per (head, split), vector ALU: f32, and ranks too wide for the tiles
//   k_latent_merge         the splits and the sink -> the head's latent, contracted with Wuv
// Scores, weights and sums are f32; the matrix-core kernels meet attention weights (and, in decode, the contracted
// queries) as the sum of two bfloat16 parts.  (No counterpart in the reference, which has no attention layer.)
#include <algorithm>
#include <vector>

#include "dense.h"

namespace candy {

struct LatentArgs {
    const float *cos_t, *sin_t, *sink, *q_norm, *kv_norm;
    int H, dim, rot, half, vdim;      // padded widths per head; half: rot_dim / 2
    int q_rank, q_p, kv_rank, kv_p;   // as given and padded
    int row;                          // kv_p + rot
    int out_cols;
    int64_t ldo;
    float scale, eps;
};

__device__ __forceinline__ float partial_at(const Partial &p, size_t row, int i) {
    const float *s = p.p + row * (size_t)p.ld + i;
    float t = s[0];
    for (int c = 1; c < p.copies; ++c) t += s[(size_t)c * p.stride];
    return t;
}

// element j of a rotated part at position pos; at(i) gives its values before rotation
template <class F>
__device__ __forceinline__ float turned(const LatentArgs &a, int j, size_t pos, const F &at) {
    if (j >= 2 * a.half) return at(j);
    const int k = j < a.half ? j : j - a.half;
    const float c = a.cos_t[pos * a.half + k], s = a.sin_t[pos * a.half + k];
    return j < a.half ? at(j) * c - at(j + a.half) * s : at(j) * c + at(k) * s;
}

// One workgroup per token.  row: n values of the padded width in LDS -> normed by the first `rank`
__device__ __forceinline__ float rms_scale(const float *row, int rank, float eps, float *red) {
    float q = 0.0f;
    for (int i = threadIdx.x; i < rank; i += 256) q += row[i] * row[i];
    return 1.0f / sqrtf(block_sum(q, red) / (float)rank + eps);
}

template <class AT>
__device__ void append_row(const LatentArgs &a, const float *row, size_t pos, AT *cache, float *red) {
    const float r = rms_scale(row, a.kv_rank, a.eps, red);
    AT *dst = cache + pos * (size_t)a.row;
    for (int i = threadIdx.x; i < a.row; i += 256) {
        float v;
        if (i < a.kv_p) v = i < a.kv_rank ? row[i] * r * a.kv_norm[i] : 0.0f;
        else v = turned(a, i - a.kv_p, pos, [&](int j) { return row[a.kv_p + j]; });
        dst[i] = (AT)v;
    }
}

template <class AT>
__global__ __launch_bounds__(256) void k_latent_rows(const LatentArgs a, const Partial z, AT *__restrict__ cq, AT *__restrict__ cache,
                                                     int pos0, const int *pos_ptr) {
    extern __shared__ float row[];
    __shared__ float red[4];
    const int tid = threadIdx.x;
    const size_t t = blockIdx.x, pos = (size_t)(pos_ptr ? *pos_ptr : pos0) + t;
    const int width = a.q_p + (cache ? a.row : 0);
    for (int i = tid * 4; i < width; i += 1024) {   // every width is a multiple of four
        const float *s = z.p + t * (size_t)z.ld + i;
        f32x4 v = *(const f32x4 *)s;
        for (int c = 1; c < z.copies; ++c) v += *(const f32x4 *)(s + (size_t)c * z.stride);
        *(f32x4 *)&row[i] = v;
    }
    __syncthreads();
    if (cq) {
        const float r = rms_scale(row, a.q_rank, a.eps, red);
        for (int i = tid; i < a.q_p; i += 256) cq[t * a.q_p + i] = (AT)(i < a.q_rank ? row[i] * r * a.q_norm[i] : 0.0f);
    }
    if (cache) append_row(a, row + a.q_p, pos, cache, red);
}

// ------------------------------------------------------------------ prompts, bfloat16, matrix cores
// grid (heads, ceil(n / 64)), 4 wavefronts of 16 queries, keys in tiles of 64 through LDS; scores transposed (keys x
// queries), so that a lane holds scores of one query only and hands the weights to the second product from registers:
// its K index 8 g + e stands for key 4 g + e of one 16-key tile (e < 4) or of the next (e >= 4), and V is stored
// transposed in LDS in that key order.  DK and DV are upper bounds of the padded widths; what lies past them is zero.
template <int DK, int DV>
__global__ __launch_bounds__(256, 2) void k_latent_prompt(const LatentArgs a, const Partial qp, const bf16 *__restrict__ cache,
                                                          const bf16 *__restrict__ kv, int ldkv, bf16 *__restrict__ out, int n, int pos0) {
    constexpr int QT = 64, KT = 64, KP = DK + 8, VP = KT + 8, K8 = DK / 8, V8 = DV / 8;
    constexpr int K_IT = KT * K8 / 256, V_IT = (KT / 2 * V8 + 255) / 256;
    __shared__ __align__(16) bf16 s_k[KT * KP];
    __shared__ __align__(16) bf16 s_v[DV * VP];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int r16 = lane & 15, g = lane >> 4;
    const int h = blockIdx.x, i0 = (gridDim.y - 1 - blockIdx.y) * QT;   // the longest rows of keys first
    const int last = pos0 + min(i0 + QT, n) - 1;
    const int qi = i0 + 16 * wave + r16, qrow = min(qi, n - 1), qpos = pos0 + qrow;
    const int wq0 = pos0 + i0 + 16 * wave, wq1 = wq0 + 15;
    const bf16 *kh = kv + (size_t)h * a.dim, *vh = kv + (size_t)a.H * a.dim + (size_t)h * a.vdim, *kr = cache + a.kv_p;

    u32x4v kreg[K_IT], vreg[V_IT][2];
    const u32x4v none{0, 0, 0, 0};
    auto request = [&](int p0) __attribute__((always_inline)) {
#pragma unroll
        for (int it = 0; it < K_IT; ++it) {
            const int e = tid + it * 256, c = e % K8 * 8;
            const size_t p = (size_t)min(p0 + e / K8, last);
            kreg[it] = none;
            if (c < a.dim) kreg[it] = *(const u32x4v *)(kh + p * ldkv + c);
            else if (c < a.dim + a.rot) kreg[it] = *(const u32x4v *)(kr + p * a.row + c - a.dim);
        }
#pragma unroll
        for (int it = 0; it < V_IT; ++it) {
            const int e = tid + it * 256, kp = e & 31, c = (e >> 5) * 8;
            vreg[it][0] = vreg[it][1] = none;
            if (c < a.vdim) {
                vreg[it][0] = *(const u32x4v *)(vh + (size_t)min(p0 + 2 * kp, last) * ldkv + c);
                vreg[it][1] = *(const u32x4v *)(vh + (size_t)min(p0 + 2 * kp + 1, last) * ldkv + c);
            }
        }
    };
    request(0);
    bf16x8 qf[DK / 32];
#pragma unroll
    for (int ks = 0; ks < DK / 32; ++ks) {
        const int i = ks * 32 + g * 8, base = h * (a.dim + a.rot);
        float v[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
        if (i < a.dim) {
            for (int c = 0; c < qp.copies; ++c) {
                const float *s = qp.p + (size_t)c * qp.stride + (size_t)qrow * qp.ld + base + i;
                const f32x4 x0 = *(const f32x4 *)s, x1 = *(const f32x4 *)(s + 4);
#pragma unroll
                for (int e = 0; e < 4; ++e) { v[e] += x0[e]; v[4 + e] += x1[e]; }
            }
        } else if (i < a.dim + a.rot) {
#pragma unroll
            for (int e = 0; e < 8; ++e)
                v[e] = turned(a, i - a.dim + e, (size_t)qpos, [&](int j) { return partial_at(qp, (size_t)qrow, base + a.dim + j); });
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) qf[ks][e] = (bf16)v[e];
    }
    float m = a.sink ? a.sink[h] * LOG2E : LOW, l = a.sink && g == 0 ? 1.0f : 0.0f;  // l: summed over g at the end
    f32x4 o[DV / 16];
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    const float c_in = a.scale * LOG2E;
    for (int p0 = 0; p0 <= last; p0 += KT) {
        __syncthreads();  // the previous tile is consumed
#pragma unroll
        for (int it = 0; it < K_IT; ++it) {
            const int e = tid + it * 256;
            *(u32x4v *)&s_k[e / K8 * KP + e % K8 * 8] = kreg[it];
        }
#pragma unroll
        for (int it = 0; it < V_IT; ++it) {
            const int e = tid + it * 256, kp = e & 31, c = e >> 5;
            if (V_IT * 256 == KT / 2 * V8 || e < KT / 2 * V8) {
                const int k32 = 2 * kp & 31;   // key 16 hh + 4 gg + ee of its 32-key block sits at 8 gg + 4 hh + ee
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
        if (p0 > wq1) continue;  // nothing of the tile is visible to these 16 queries
        f32x4 s[4];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
            s[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < DK / 32; ++ks)
                s[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8 *)&s_k[(kt * 16 + r16) * KP + ks * 32 + g * 8], qf[ks],
                                                                s[kt], 0, 0, 0);
        }
        const bool whole = p0 + KT - 1 <= wq0;  // every key visible to every query
        float mx = MASKED;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                float z = s[kt][j] * c_in;
                if (!whole) z = p0 + kt * 16 + 4 * g + j <= pos0 + qi ? z : MASKED;
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
            for (int d = 0; d < DV / 16; ++d) o[d] *= corr;
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
            for (int d = 0; d < DV / 16; ++d) {
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
    bf16 *dst = out + (size_t)qi * a.ldo + (size_t)h * a.vdim;
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) {
        const int c = d * 16 + 4 * g;
        if (c < a.vdim) *(bf16x4 *)(dst + c) = __builtin_convertvector(o[d] * inv, bf16x4);
    }
    if (h == a.H - 1)
        for (int i = a.H * a.vdim + g; i < a.out_cols; i += 4) out[(size_t)qi * a.ldo + i] = (bf16)0.0f;
}

// ------------------------------------------------------------------ one wavefront per (query, head) or (head, split)
// Softmax over the positions p0 .. p0 + 63, p0 = first, first + stride, ..., up to pos.  q: this wavefront's query in LDS, in two parts: d1
// values against k1 (rows ld1 apart), d2 against k2; values: dv of v.  Lane i holds values i, i + 64, ...
template <class AT, int NC>
__device__ __forceinline__ void attend_row(const float *q, const AT *k1, int64_t ld1, int d1, const AT *k2, int64_t ld2, int d2,
                                           const AT *v, int64_t ldv, int dv, int pos, int first, int stride, float &m, float &l,
                                           float (&o)[NC]) {
    const int lane = threadIdx.x & 63;
    for (int p0 = first; p0 <= pos; p0 += stride) {
        const int p = p0 + lane;
        float s = MASKED;
        if (p <= pos) {
            const AT *a = k1 + (size_t)p * ld1, *b = k2 + (size_t)p * ld2;
            float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
            for (int i = 0; i < d1; i += 8) {
                float x[8];
                lds8(a + i, x);
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[e] = fmaf(q[i + e], x[e], acc[e]);
            }
            for (int i = 0; i < d2; i += 8) {
                float x[8];
                lds8(b + i, x);
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[e] = fmaf(q[d1 + i + e], x[e], acc[e]);
            }
            s = ((acc[0] + acc[1]) + (acc[2] + acc[3])) + ((acc[4] + acc[5]) + (acc[6] + acc[7]));
        }
        const float m_new = fmaxf(m, wave_max(s));
        const float corr = expf(m - m_new), w = p <= pos ? expf(s - m_new) : 0.0f;
        l = l * corr + wave_sum(w);
        m = m_new;
#pragma unroll
        for (int c = 0; c < NC; ++c) o[c] *= corr;
        const int cnt = min(64, pos - p0 + 1);
        for (int j = 0; j < cnt; ++j) {
            const float wj = __shfl(w, j, 64);
            const AT *vr = v + (size_t)(p0 + j) * ldv;
#pragma unroll
            for (int c = 0; c < NC; ++c)
                if (lane + 64 * c < dv) o[c] = fmaf(wj, (float)vr[lane + 64 * c], o[c]);
        }
    }
}

template <class AT, int NC>
__global__ __launch_bounds__(256) void k_latent_prompt_row(const LatentArgs a, const Partial qp, const AT *__restrict__ cache,
                                                           const AT *__restrict__ kv, int ldkv, AT *__restrict__ out, int n, int pos0) {
    extern __shared__ float row[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int t = blockIdx.x * 4 + wave, h = blockIdx.y, dk = a.dim + a.rot, base = h * dk;
    float *q = row + wave * dk;
    if (t < n)
        for (int i = lane; i < dk; i += 64) {
            const float v = i < a.dim ? partial_at(qp, (size_t)t, base + i)
                                      : turned(a, i - a.dim, (size_t)pos0 + t, [&](int j) { return partial_at(qp, (size_t)t, base + a.dim + j); });
            q[i] = (float)(AT)v * a.scale;
        }
    __syncthreads();
    if (t >= n) return;
    float m = a.sink ? a.sink[h] : LOW, l = a.sink ? 1.0f : 0.0f, o[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) o[c] = 0.0f;
    attend_row<AT, NC>(q, kv + (size_t)h * a.dim, ldkv, a.dim, cache + a.kv_p, a.row, a.rot,
                       kv + (size_t)a.H * a.dim + (size_t)h * a.vdim, ldkv, a.vdim, pos0 + t, 0, 64, m, l, o);
    AT *dst = out + (size_t)t * a.ldo;
#pragma unroll
    for (int c = 0; c < NC; ++c)
        if (lane + 64 * c < a.vdim) dst[(size_t)h * a.vdim + lane + 64 * c] = (AT)(o[c] / l);
    if (h == a.H - 1)
        for (int i = a.H * a.vdim + lane; i < a.out_cols; i += 64) dst[i] = (AT)0.0f;
}

// ------------------------------------------------------------------ decode
// grid (heads (+ 1: the new cache row), kv_p / 64): rows of Wuk^T of one head against its query, scaled into powers of
// two (SPLIT: as the sum of two bfloat16 parts, rows of the second H * row values behind the first) or plainly in f32.
template <class AT, bool SPLIT>
__global__ __launch_bounds__(256) void k_latent_query(const LatentArgs a, const Partial z, const float *__restrict__ q,
                                                      const bf16 *__restrict__ ukt, int ldd, AT *cache, void *__restrict__ qa,
                                                      const int *__restrict__ pos_ptr) {
    extern __shared__ float row[];
    __shared__ float red[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x;
    if (h == a.H) {
        if (blockIdx.y) return;
        for (int i = tid; i < a.row; i += 256) row[i] = z.p[a.q_p + i];
        __syncthreads();
        append_row(a, row, (size_t)*pos_ptr, cache, red);
        return;
    }
    const int dk = a.dim + a.rot, l16 = lane & 15;
    const int r0 = blockIdx.y * 64 + wave * 16 + (lane >> 4);
    const bf16 *w = ukt + ((size_t)h * a.kv_p + r0) * ldd;
    const float *qh = q + (size_t)h * dk;
    u32x4v first[4];
    if (l16 * 8 < ldd) {
#pragma unroll
        for (int it = 0; it < 4; ++it) first[it] = *(const u32x4v *)(w + (size_t)it * 4 * ldd + l16 * 8);
    }
    for (int i = tid; i < ldd; i += 256) row[i] = i < a.dim ? qh[i] : 0.0f;
    __syncthreads();
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k = l16 * 8; k < ldd; k += 128) {
        float x[8];
        lds8(row + k, x);
#pragma unroll
        for (int it = 0; it < 4; ++it) {
            float f[8];
            widen8(k < 128 ? first[it] : *(const u32x4v *)(w + (size_t)it * 4 * ldd + k), f);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[it] = fmaf(f[e], x[e], acc[it]);
        }
    }
    const float c = SPLIT ? a.scale * LOG2E : a.scale;
    auto put = [&](int i, float v) __attribute__((always_inline)) {
        const size_t at = (size_t)h * a.row + i;
        if (SPLIT) {
            const bf16 hi = (bf16)v;
            ((bf16 *)qa)[at] = hi;
            ((bf16 *)qa)[(size_t)a.H * a.row + at] = (bf16)(v - (float)hi);
        } else {
            ((float *)qa)[at] = v;
        }
    };
#pragma unroll
    for (int it = 0; it < 4; ++it) {
        const float v = lanes_sum<16>(acc[it]);
        if (l16 == 0) put(r0 + it * 4, v * c);
    }
    if (blockIdx.y == 0)
        for (int j = tid; j < a.rot; j += 256)
            put(a.kv_p + j, c * turned(a, j, (size_t)*pos_ptr, [&](int i) { return qh[a.dim + i]; }));
}

// grid (ceil(heads / 16), splits), tiles of 32 positions dealt to the splits round robin.  The tile's rows go to LDS
// once.  The 4 wavefronts share the first product's K (their sums meet in LDS), repeat the softmax over the tile's 32
// positions, and each take a quarter of the latent's columns in the second product, whose K index 8 g + e stands for key
// 4 g + e of the tile's first 16 (e < 4) or of the others.  NT: kv_p / 16 at most.
template <int NT>
__global__ __launch_bounds__(256) void k_latent_decode(const bf16 *__restrict__ qa, const bf16 *__restrict__ cache,
                                                       const int *__restrict__ pos_ptr, float *__restrict__ part, int H, int row, int kv_p,
                                                       int n_splits) {
    constexpr int KT = 32, WIDTH = NT * 16 + 128, NKS = (WIDTH / 32 + 3) / 4, P = WIDTH + 8, LOADS = KT * WIDTH / 8 / 256, ND = NT / 4;
    __shared__ __align__(16) bf16 tile[KT * P];
    __shared__ __align__(16) f32x4 sums[4][2][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int r16 = lane & 15, g = lane >> 4;
    const int h = blockIdx.x * 16 + r16, split = blockIdx.y, nks = row >> 5, chunks = row >> 3;
    const bf16 *q0 = qa + (size_t)min(h, H - 1) * row + g * 8, *q1 = q0 + (size_t)H * row;
    bf16x8 qh[NKS], ql[NKS];
#pragma unroll
    for (int i = 0; i < NKS; ++i) {
        const int ks = min(wave + 4 * i, nks - 1);
        qh[i] = *(const bf16x8 *)(q0 + ks * 32);
        ql[i] = *(const bf16x8 *)(q1 + ks * 32);
    }
    const int pos = *pos_ptr;
    u32x4v reg[LOADS];
    auto request = [&](int p0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < LOADS; ++i) {
            const int e = tid + i * 256, k = e / chunks;
            if (k < KT) reg[i] = *(const u32x4v *)(cache + (size_t)min(p0 + k, pos) * row + (e - k * chunks) * 8);
        }
    };
    if (split * KT <= pos) request(split * KT);
    float m = LOW, l = 0.0f;
    f32x4 o[ND];
#pragma unroll
    for (int d = 0; d < ND; ++d) o[d] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int step = n_splits * KT;
    for (int p0 = split * KT; p0 <= pos; p0 += step) {
#pragma unroll
        for (int i = 0; i < LOADS; ++i) {
            const int e = tid + i * 256, k = e / chunks;
            if (k < KT) *(u32x4v *)&tile[k * P + (e - k * chunks) * 8] = reg[i];
        }
        __syncthreads();
        if (p0 + step <= pos) request(p0 + step);
        f32x4 s[2];
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) s[kt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NKS; ++i) {
            const int ks = wave + 4 * i;
            if (ks >= nks) break;
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
                const bf16x8 kf = *(const bf16x8 *)&tile[(kt * 16 + r16) * P + ks * 32 + g * 8];
                s[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, ql[i], s[kt], 0, 0, 0);
                s[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qh[i], s[kt], 0, 0, 0);
            }
        }
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) sums[wave][kt][lane] = s[kt];
        __syncthreads();
        float mx = MASKED;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
            s[kt] = (sums[0][kt][lane] + sums[1][kt][lane]) + (sums[2][kt][lane] + sums[3][kt][lane]);
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                if (p0 + kt * 16 + 4 * g + j > pos) s[kt][j] = MASKED;
                mx = fmaxf(mx, s[kt][j]);
            }
        }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float m_new = fmaxf(m, mx), corr = __builtin_amdgcn_exp2f(m - m_new);
        m = m_new;
        float sum = 0.0f;
        bf16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float w = __builtin_amdgcn_exp2f(s[e >> 2][e & 3] - m_new);
            sum += w;
            hi[e] = (bf16)w;
            lo[e] = (bf16)(w - (float)hi[e]);
        }
        l = l * corr + sum;
#pragma unroll
        for (int d = 0; d < ND; ++d) {
            const int c = (wave + 4 * d) * 16;
            if (c >= kv_p) break;
            bf16x8 vt;
#pragma unroll
            for (int e = 0; e < 8; ++e) vt[e] = tile[((e >> 2) * 16 + 4 * g + (e & 3)) * P + c + r16];
            o[d] *= corr;
            o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, lo, o[d], 0, 0, 0);
            o[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vt, hi, o[d], 0, 0, 0);
        }
        __syncthreads();  // the tile and the sums are consumed
    }
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (h >= H) return;
    float *p = part + ((size_t)h * n_splits + split) * (kv_p + 4);
#pragma unroll
    for (int d = 0; d < ND; ++d) {
        const int c = (wave + 4 * d) * 16;
        if (c < kv_p) *(f32x4 *)(p + c + 4 * g) = o[d];
    }
    if (wave == 0 && g == 0) {
        p[kv_p] = m;
        p[kv_p + 1] = l;
    }
}

// grid (heads, ceil(splits / 4)): the same partial results from f32 queries; maxima in powers of two like there
template <class AT, int NC>
__global__ __launch_bounds__(256) void k_latent_decode_row(const LatentArgs a, const float *__restrict__ qa, const AT *__restrict__ cache,
                                                           const int *__restrict__ pos_ptr, float *__restrict__ part, int n_splits) {
    extern __shared__ float row[];
    const int lane = threadIdx.x & 63, h = blockIdx.x, split = blockIdx.y * 4 + (threadIdx.x >> 6);
    for (int i = threadIdx.x; i < a.row; i += 256) row[i] = qa[(size_t)h * a.row + i];
    __syncthreads();
    if (split >= n_splits) return;
    float m = LOW, l = 0.0f, o[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) o[c] = 0.0f;
    attend_row<AT, NC>(row, cache, a.row, a.row, cache, 0, 0, cache, a.row, a.kv_p, *pos_ptr, split * 64, n_splits * 64, m, l, o);
    float *p = part + ((size_t)h * n_splits + split) * (a.kv_p + 4);
#pragma unroll
    for (int c = 0; c < NC; ++c)
        if (lane + 64 * c < a.kv_p) p[lane + 64 * c] = o[c];
    if (lane == 0) {
        p[a.kv_p] = l > 0.0f ? m * LOG2E : LOW;
        p[a.kv_p + 1] = l;
    }
}

// grid (heads, vdim / 32): at most 64 splits, a lane each for the maxima; then 32 rows of the head's Wuv
template <class AT>
__global__ __launch_bounds__(256) void k_latent_merge(const LatentArgs a, const float *__restrict__ part, int n_splits,
                                                      const bf16 *__restrict__ uv, int ldw, AT *__restrict__ out) {
    extern __shared__ __align__(16) float lat[];   // [kv_p], then 256 float4
    __shared__ float factor[64];
    f32x4 *red = (f32x4 *)(lat + a.kv_p);
    const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15;
    const int r0 = blockIdx.y * 32 + wave * 8 + (lane >> 4);
    const bf16 *w = uv + ((size_t)h * a.vdim + r0) * ldw;
    constexpr int AHEAD = 4;   // 512 values of a row requested in front
    u32x4v wf[2][AHEAD];
#pragma unroll
    for (int it = 0; it < 2; ++it)
#pragma unroll
        for (int s = 0; s < AHEAD; ++s) wf[it][s] = *(const u32x4v *)(w + (size_t)it * 4 * ldw + min(s * 128 + l16 * 8, ldw - 8));
    const int pitch = a.kv_p + 4, C4 = a.kv_p >> 2, SG = 256 / C4;   // kv_p is at most 1024
    const float *p = part + (size_t)h * n_splits * pitch;
    float ms = LOW, ls = 0.0f;
    if (lane < n_splits) {
        ms = p[(size_t)lane * pitch + a.kv_p];
        ls = p[(size_t)lane * pitch + a.kv_p + 1];
    }
    const float sink = a.sink ? a.sink[h] * LOG2E : MASKED;
    const int sg = tid / C4, c4 = tid % C4;   // thread: splits sg, sg + SG, ... of four columns
    constexpr int FRONT = 16;
    f32x4 v[FRONT];
#pragma unroll
    for (int j = 0; j < FRONT; ++j) v[j] = *(const f32x4 *)(p + (size_t)min(sg + SG * j, n_splits - 1) * pitch + 4 * c4);
    __builtin_amdgcn_sched_barrier(0);  // every load above is requested before anything below waits
    const float m = fmaxf(wave_max(ms), sink);
    const float e = lane < n_splits ? __builtin_amdgcn_exp2f(ms - m) : 0.0f;
    const float f = e / (wave_sum(ls * e) + (a.sink ? __builtin_amdgcn_exp2f(sink - m) : 0.0f));
    if (wave == 0) factor[lane] = f;
    __syncthreads();
    f32x4 o{0.f, 0.f, 0.f, 0.f};
    if (sg < SG) {
#pragma unroll
        for (int j = 0; j < FRONT; ++j)
            if (sg + SG * j < n_splits) o += v[j] * factor[sg + SG * j];
#pragma unroll 8
        for (int s = sg + SG * FRONT; s < n_splits; s += SG) o += *(const f32x4 *)(p + (size_t)s * pitch + 4 * c4) * factor[s];
    }
    red[tid] = o;
    __syncthreads();
    if (tid < C4) {
        for (int s = 1; s < SG; ++s) o += red[s * C4 + tid];
        *(f32x4 *)(lat + 4 * tid) = o;
    }
    __syncthreads();
    float acc[2] = {0.f, 0.f};
    for (int k0 = 0; k0 < ldw; k0 += 128) {
        const int k = k0 + l16 * 8;
        if (k >= ldw) break;
        float x[8];
        lds8(lat + k, x);
#pragma unroll
        for (int it = 0; it < 2; ++it) {
            float g[8];
            u32x4v v;
            switch (k0 >> 7) {
            case 0: v = wf[it][0]; break;
            case 1: v = wf[it][1]; break;
            case 2: v = wf[it][2]; break;
            case 3: v = wf[it][3]; break;
            default: v = *(const u32x4v *)(w + (size_t)it * 4 * ldw + k);
            }
            widen8(v, g);
#pragma unroll
            for (int j = 0; j < 8; ++j) acc[it] = fmaf(g[j], x[j], acc[it]);
        }
    }
#pragma unroll
    for (int it = 0; it < 2; ++it) {
        const float v = lanes_sum<16>(acc[it]);
        if (l16 == 0) out[(size_t)h * a.vdim + r0 + it * 4] = (AT)v;
    }
    if (h == a.H - 1 && blockIdx.y == gridDim.y - 1)
        for (int i = a.H * a.vdim + tid; i < a.out_cols; i += 256) out[i] = (AT)0.0f;
}

// ------------------------------------------------------------------ host side
int check_latent_spec(const candy_hip_latent_spec &s) {
    CANDY_REQUIRE(s.n_heads > 0 && s.n_heads <= 4096, "invalid number of heads %d", s.n_heads);
    CANDY_REQUIRE(s.dim > 0 && s.rot_dim >= 0 && s.rot_dim % 2 == 0 && s.dim + s.rot_dim <= 960, "query widths %d + %d unsupported (even, 960 in all)",
                  s.dim, s.rot_dim);
    CANDY_REQUIRE(s.vdim > 0 && s.vdim <= 1024, "value width %d unsupported (1 .. 1024)", s.vdim);
    CANDY_REQUIRE(s.kv_rank > 0 && s.kv_rank <= 1024 && s.q_rank > 0 && s.q_rank <= 8192, "ranks %d / %d unsupported (kv up to 1024, q up to 8192)",
                  s.kv_rank, s.q_rank);
    CANDY_REQUIRE(s.rot_dim == 0 || s.rope_base > 0, "rope_base must be positive");
    return CANDY_HIP_OK;
}

static int latent_row(const candy_hip_latent_spec &s) { return (int)(pad64(s.kv_rank) + pad32(s.rot_dim)); }
// the matrix-core decode kernel holds rows of at most this many steps of 32 (k_latent_decode's NT: kv_p / 16 rounded up
// to a power of two, four steps for the rotated part)
static int decode_tiles(const candy_hip_latent_spec &s) {
    if (pad32(s.rot_dim) > 128) return 0;
    for (int nt : {4, 8, 16, 32})
        if (pad64(s.kv_rank) <= nt * 16) return nt;
    return 0;
}

int latent_splits(const candy_hip_device *dev, const candy_hip_latent_spec &s, int max_pos) {
    if (dev->opt.attn_splits > 0) return dev->opt.attn_splits;  // comparison runs
    const int64_t heads = (s.n_heads + 15) / 16;
    return (int)std::max<int64_t>(1, std::min<int64_t>({64, (max_pos + 31) / 32, 2 * (int64_t)dev->num_cus / heads}));
}
size_t latent_query_bytes(const candy_hip_latent_spec &s) { return (size_t)s.n_heads * latent_row(s) * 4; }
size_t latent_scratch_floats(const candy_hip_latent_spec &s, int n_splits) {
    return (size_t)s.n_heads * n_splits * (pad64(s.kv_rank) + 4);
}

static LatentArgs latent_args(const LatentAttn &A) {
    LatentArgs a;
    a.cos_t = A.cos_t; a.sin_t = A.sin_t; a.sink = A.sink; a.q_norm = A.q_norm; a.kv_norm = A.kv_norm;
    a.H = A.s.n_heads; a.dim = (int)pad32(A.s.dim); a.rot = (int)pad32(A.s.rot_dim); a.half = A.s.rot_dim / 2; a.vdim = (int)pad32(A.s.vdim);
    a.q_rank = A.s.q_rank; a.q_p = (int)pad64(A.s.q_rank); a.kv_rank = A.s.kv_rank; a.kv_p = (int)pad64(A.s.kv_rank);
    a.row = a.kv_p + a.rot;
    a.out_cols = A.out_cols; a.ldo = A.ldo;
    a.scale = A.s.scale; a.eps = A.eps;
    return a;
}

template <class AT>
static int latent_rows(candy_hip_device *dev, const LatentAttn &A, int n, int pos0, const int *pos_ptr) {
    const LatentArgs a = latent_args(A);
    CANDY_REQUIRE(A.down.ld % 4 == 0 && A.down.stride % 4 == 0 && ((uintptr_t)A.down.p & 15) == 0, "internal: unaligned projections");
    hipLaunchKernelGGL((k_latent_rows<AT>), dim3((unsigned)n), dim3(256), (size_t)(a.q_p + (A.own ? a.row : 0)) * 4, dev->stream, a, A.down,
                       (AT *)A.cq, A.own ? (AT *)A.cache : nullptr, pos0, pos_ptr);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}
int launch_latent_rows(candy_hip_device *dev, const LatentAttn &A, int n, int pos0, const int *pos_ptr) {
    return A.f32 ? latent_rows<float>(dev, A, n, pos0, pos_ptr) : latent_rows<bf16>(dev, A, n, pos0, pos_ptr);
}

static int row_chunks(int width) {
    for (int c : {1, 2, 4, 8, 16})
        if (width <= 64 * c) return c;
    return 0;
}

template <class AT>
static int prompt_rows(candy_hip_device *dev, const LatentAttn &A, int n, int pos0) {
    const LatentArgs a = latent_args(A);
    const dim3 g((unsigned)((n + 3) / 4), (unsigned)a.H), b(256);
    const size_t lds = (size_t)4 * (a.dim + a.rot) * 4;
#define CANDY_LPR(NC)                                                                                                             \
    case NC:                                                                                                                      \
        hipLaunchKernelGGL((k_latent_prompt_row<AT, NC>), g, b, lds, dev->stream, a, A.q, (const AT *)A.cache, (const AT *)A.kv,   \
                           (int)A.ukv->rows_pad, (AT *)A.out, n, pos0);                                                           \
        break
    switch (row_chunks(a.vdim)) {
        CANDY_LPR(1); CANDY_LPR(2); CANDY_LPR(4); CANDY_LPR(8); CANDY_LPR(16);
    default: return fail(CANDY_HIP_ERR_UNSUPPORTED, "no attention kernel for values of %d", a.vdim);
    }
#undef CANDY_LPR
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

template <int DK>
static bool prompt_tiles(candy_hip_device *dev, const LatentAttn &A, const LatentArgs &a, int n, int pos0) {
    const dim3 g((unsigned)a.H, (unsigned)((n + 63) / 64)), b(256);
#define CANDY_LP(DV)                                                                                                            \
    if (a.vdim <= DV) {                                                                                                         \
        hipLaunchKernelGGL((k_latent_prompt<DK, DV>), g, b, 0, dev->stream, a, A.q, (const bf16 *)A.cache, (const bf16 *)A.kv,   \
                           (int)A.ukv->rows_pad, (bf16 *)A.out, n, pos0);                                                       \
        return true;                                                                                                            \
    }
    CANDY_LP(64) CANDY_LP(128) CANDY_LP(256)
#undef CANDY_LP
    return false;
}

int launch_latent_prompt(candy_hip_device *dev, const LatentAttn &A, int n, int pos0) {
    const LatentArgs a = latent_args(A);
    CANDY_REQUIRE(A.ukv->rows == (int64_t)a.H * (a.dim + a.vdim) && A.ukv->ld == a.kv_p && (n + 63) / 64 <= 65535, "internal: attention launch");
    // keys and values of every position so far, one contraction with the cached latents
    DenseLaunch D;
    D.w = A.ukv; D.x = A.cache; D.ldx = a.row; D.f32 = A.f32; D.m = pos0 + n; D.epi = CANDY_HIP_EPI_ACT;
    D.y = A.kv; D.ldy = D.n_store = A.ukv->rows_pad;
    if (int rc = launch_dense(dev, D)) return rc;
    if (A.f32) return prompt_rows<float>(dev, A, n, pos0);
    CANDY_REQUIRE(A.q.ld % 4 == 0 && A.q.stride % 4 == 0 && ((uintptr_t)A.q.p & 15) == 0, "internal: unaligned queries");
    const int dk = a.dim + a.rot;
    bool done = false;
    if (dk <= 64) done = prompt_tiles<64>(dev, A, a, n, pos0);
    else if (dk <= 96) done = prompt_tiles<96>(dev, A, a, n, pos0);
    else if (dk <= 128) done = prompt_tiles<128>(dev, A, a, n, pos0);
    else if (dk <= 192) done = prompt_tiles<192>(dev, A, a, n, pos0);
    else if (dk <= 256) done = prompt_tiles<256>(dev, A, a, n, pos0);
    if (!done) return prompt_rows<bf16>(dev, A, n, pos0);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

template <class AT>
static int decode_rows(candy_hip_device *dev, const LatentAttn &A, const LatentArgs &a, const int *pos_ptr) {
    const dim3 g((unsigned)a.H, (unsigned)((A.n_splits + 3) / 4)), b(256);
#define CANDY_LDR(NC)                                                                                                         \
    case NC:                                                                                                                  \
        hipLaunchKernelGGL((k_latent_decode_row<AT, NC>), g, b, (size_t)a.row * 4, dev->stream, a, (const float *)A.qa,        \
                           (const AT *)A.cache, pos_ptr, A.part, A.n_splits);                                                 \
        break
    switch (row_chunks(a.kv_p)) {
        CANDY_LDR(1); CANDY_LDR(2); CANDY_LDR(4); CANDY_LDR(8); CANDY_LDR(16);
    default: return fail(CANDY_HIP_ERR_UNSUPPORTED, "no attention kernel for latents of %d", a.kv_p);
    }
#undef CANDY_LDR
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

template <class AT, bool SPLIT>
static void decode_query(candy_hip_device *dev, const LatentAttn &A, const LatentArgs &a, const int *pos_ptr) {
    hipLaunchKernelGGL((k_latent_query<AT, SPLIT>), dim3((unsigned)(a.H + (A.own ? 1 : 0)), (unsigned)(a.kv_p / 64)), dim3(256),
                       (size_t)std::max<int64_t>(a.row, A.ukt->ld) * 4, dev->stream, a, A.down, A.q.p, (const bf16 *)A.ukt->data,
                       (int)A.ukt->ld, (AT *)A.cache, A.qa, pos_ptr);
}

template <class AT>
static int decode_merge(candy_hip_device *dev, const LatentAttn &A, const LatentArgs &a) {
    const int ldw = (int)A.ukv->ld;
    hipLaunchKernelGGL((k_latent_merge<AT>), dim3((unsigned)a.H, (unsigned)(a.vdim / 32)), dim3(256), (size_t)a.kv_p * 4 + 4096, dev->stream, a,
                       A.part, A.n_splits, (const bf16 *)A.ukv->data + (size_t)a.H * a.dim * ldw, ldw, (AT *)A.out);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

int launch_latent_decode(candy_hip_device *dev, const LatentAttn &A, const int *pos_ptr) {
    const LatentArgs a = latent_args(A);
    CANDY_REQUIRE(A.n_splits >= 1 && A.n_splits <= 64 && A.q.copies == 1 && (!A.own || A.down.copies == 1) &&
                      A.ukt->rows == (int64_t)a.H * a.kv_p && A.ukv->rows == (int64_t)a.H * (a.dim + a.vdim) && A.ukv->ld == a.kv_p,
                  "internal: attention launch");
    const int nt = A.f32 ? 0 : decode_tiles(A.s);
    if (A.f32) decode_query<float, false>(dev, A, a, pos_ptr);
    else if (nt) decode_query<bf16, true>(dev, A, a, pos_ptr);
    else decode_query<bf16, false>(dev, A, a, pos_ptr);
    CANDY_LAUNCH_CHECK();
    if (nt) {
        const dim3 g((unsigned)((a.H + 15) / 16), (unsigned)A.n_splits), b(256);
#define CANDY_LD(NT)                                                                                                                \
    case NT:                                                                                                                        \
        hipLaunchKernelGGL((k_latent_decode<NT>), g, b, 0, dev->stream, (const bf16 *)A.qa, (const bf16 *)A.cache, pos_ptr, A.part,  \
                           a.H, a.row, a.kv_p, A.n_splits);                                                                         \
        break
        switch (nt) {
            CANDY_LD(4); CANDY_LD(8); CANDY_LD(16); CANDY_LD(32);
        }
#undef CANDY_LD
        CANDY_LAUNCH_CHECK();
    } else if (int rc = A.f32 ? decode_rows<float>(dev, A, a, pos_ptr) : decode_rows<bf16>(dev, A, a, pos_ptr)) {
        return rc;
    }
    return A.f32 ? decode_merge<float>(dev, A, a) : decode_merge<bf16>(dev, A, a);
}

}  // namespace candy

using namespace candy;

extern "C" {

int32_t candy_hip_pad32(int32_t n) { return (int32_t)pad32(n); }
int32_t candy_hip_pad64(int32_t n) { return (int32_t)pad64(n); }
int32_t candy_hip_latent_row(const candy_hip_latent_spec *spec) { return spec && check_latent_spec(*spec) == CANDY_HIP_OK ? latent_row(*spec) : 0; }

int candy_hip_latent_attention(candy_hip_device *dev, const candy_hip_latent_spec *spec, int act, const float *q, const float *dkv,
                               const float *kv_norm, float eps, const candy_hip_dense *ukv, const candy_hip_dense *ukt,
                               const float *sink, int64_t n, int32_t pos0, int32_t max_pos, void *cache, int decode, float *out) {
    CANDY_REQUIRE(dev && spec, "nil argument");
    if (int rc = check_latent_spec(*spec)) return rc;
    CANDY_REQUIRE(act == CANDY_HIP_ACT_BF16 || act == CANDY_HIP_ACT_F32, "unknown activation format %d", act);
    CANDY_REQUIRE(n >= 1 && n <= 1 << 20 && pos0 >= 0 && pos0 + n <= max_pos, "positions %d .. %lld outside the cache (max_pos %d)", pos0,
                  (long long)(pos0 + n - 1), max_pos);
    CANDY_REQUIRE(!decode || n == 1, "the decode kernels take one token");
    CANDY_REQUIRE(q && ukv && ukt && cache && out && (!dkv || kv_norm), "nil pointer");
    CANDY_REQUIRE(((uintptr_t)cache & 15) == 0 && ((uintptr_t)q & 15) == 0 && ((uintptr_t)dkv & 15) == 0, "arrays must be 16-byte aligned");
    const bool f32 = act == CANDY_HIP_ACT_F32;
    LatentAttn A;
    A.s = *spec;
    A.s.q_rank = 0;   // no query latent in front of the projected rows here
    const LatentArgs a = latent_args(A);
    CANDY_REQUIRE(ukv->dev == dev && ukt->dev == dev && ukv->rows == (int64_t)a.H * (a.dim + a.vdim) && ukv->cols == spec->kv_rank &&
                      ukt->rows == (int64_t)a.H * a.kv_p && ukt->cols == spec->dim,
                  "weights do not fit the spec");
    if (int rc = use_device(dev)) return rc;
    A.max_pos = max_pos; A.f32 = f32; A.n_splits = latent_splits(dev, *spec, max_pos);
    const int width = a.H * a.vdim;
    const size_t es = f32 ? 4 : 2;
    auto al = [](size_t b) { return (b + 255) & ~(size_t)255; };
    const size_t kv_b = al((size_t)max_pos * ukv->rows_pad * es), o_b = al((size_t)n * width * es), qa_b = al(latent_query_bytes(*spec)),
                 p_b = al(latent_scratch_floats(*spec, A.n_splits) * 4), t_b = al((size_t)max_pos * a.half * 4 + 4);
    void *ws = nullptr;
    if (int rc = workspace(dev, kv_b + o_b + qa_b + p_b + 2 * t_b + 256, &ws)) return rc;
    uint8_t *w = (uint8_t *)ws;
    A.kv = w; A.out = w + kv_b; A.qa = w + kv_b + o_b; A.part = (float *)(w + kv_b + o_b + qa_b);
    float *ct = (float *)(w + kv_b + o_b + qa_b + p_b), *st = (float *)((uint8_t *)ct + t_b);
    int *pos = (int *)((uint8_t *)st + t_b);
    candy_hip_attn_spec turn{};
    turn.rope_dims = spec->rot_dim;
    turn.rope_base = spec->rope_base;
    std::vector<float> hc((size_t)max_pos * a.half + 1), hs((size_t)max_pos * a.half + 1);
    fill_rope_tables(turn, max_pos, hc.data(), hs.data());
    if (int rc = candy_hip_h2d(dev, ct, hc.data(), (size_t)max_pos * a.half * 4)) return rc;
    if (int rc = candy_hip_h2d(dev, st, hs.data(), (size_t)max_pos * a.half * 4)) return rc;
    if (int rc = candy_hip_h2d(dev, pos, &pos0, sizeof(int))) return rc;
    A.cos_t = ct; A.sin_t = st; A.sink = sink; A.kv_norm = kv_norm; A.eps = eps; A.cache = cache; A.own = dkv != nullptr;
    A.ukv = ukv; A.ukt = ukt;
    A.q.p = q; A.q.ld = a.H * (a.dim + a.rot);
    A.down.p = dkv; A.down.ld = a.row;
    A.ldo = width; A.out_cols = width;
    if (decode) {
        if (int rc = launch_latent_decode(dev, A, pos)) return rc;
    } else {
        if (dkv)
            if (int rc = launch_latent_rows(dev, A, (int)n, pos0, nullptr)) return rc;
        if (int rc = launch_latent_prompt(dev, A, (int)n, pos0)) return rc;
    }
    return launch_from_act(dev, f32, A.out, out, n, width, width);
}

}  // extern "C"
