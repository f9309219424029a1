// bfloat16 weights [rows, cols]: upload, row gather and the contraction y = epilogue(x . W^T).
//   k_dense_mv      one activation row: every weight row is streamed once by one wavefront, the activations wait in LDS
//                   (bfloat16 or f32 activations; HBM-bound).  Optional prologue: the norms in front of the contraction.
//   k_dense_mm      prompt batches, bfloat16 activations: v_mfma_f32_16x16x32_bf16 over LDS tiles filled by direct
//                   global-to-LDS loads, two stages; optionally split along K
//   k_dense_mm_f32  prompt batches, f32 activations: v_mfma_f32_16x16x4_f32, weights widened exactly
// Prompt batches also come with block-diagonal weights, and with their rows dealt to experts (GroupedRows).
// Weights are stored with both sides padded to multiples of 64 by zeros, so no kernel has a ragged edge in K, and the
// padded rows come out as epilogue(0) = 0.  (No counterpart in the reference, which has no bfloat16.)
#include <algorithm>

#include "dense.h"

namespace candy {

constexpr int EPI_NONE = CANDY_HIP_EPI_NONE, EPI_RELU2 = CANDY_HIP_EPI_SQUARED_RELU, EPI_CAP = CANDY_HIP_EPI_SOFTCAP,
              EPI_ACT = CANDY_HIP_EPI_ACT;
constexpr bool to_act(int epi) { return epi == EPI_RELU2 || epi == EPI_ACT; }  // the result is in the activation format

struct EpiArgs {
    float scale, cap;
};

template <int EPI>
__device__ __forceinline__ float epilogue(float z, const EpiArgs &e) {
    if (EPI == EPI_RELU2) {
        const float r = fmaxf(z, 0.0f);
        return r * r;
    }
    if (EPI == EPI_CAP) {
        z *= e.scale;
        return e.cap > 0.0f ? e.cap * tanhf(z / e.cap) : z;
    }
    return z;
}

// ------------------------------------------------------------------ one row
// The norms in front of the contraction (launch_norm_chain's arithmetic), for a kernel that runs them in its prologue.
struct NormPro {
    const float *x, *y, *post_w, *post_b, *step, *pre_w, *pre_b;
    float *x_out;
    float mult, eps;
    int cols, rms;
};

__device__ __forceinline__ float pro_sum(float v, float *red) {
    v = wave_sum(v);
    __syncthreads();  // the last use of red is over
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    const int n = blockDim.x >> 6;
    float t = red[0];
    for (int w = 1; w < n; ++w) t += red[w];
    return t;
}

template <class AT> constexpr int mv_lds_values() { return sizeof(AT) == 2 ? 16384 : 8192; }  // 32 KB: whole steps
template <int R> constexpr int mv_unroll() { return 8 / R; }                                  // 8 KB requested per step

// One workgroup of W wavefronts per CU where the rows go round (launch_mv picks W and R so that they do), R weight rows
// per wavefront.  The next step's weights are requested before the current ones are multiplied, the first ones before
// the activations are staged.  NV > 0: the activations are made here, by the norm chain in front of the contraction
// (NV float4 per thread); every workgroup repeats it, workgroup 0 writes the new residual row.
template <class AT, int R, int EPI, int NV>
__global__ __launch_bounds__(1024) void k_dense_mv(const AT *__restrict__ x, const bf16 *__restrict__ W, void *__restrict__ yv,
                                                   int K, int rows, int n_store, const EpiArgs ea, const NormPro np) {
    constexpr int U = mv_unroll<R>(), STEP = U * 512, CH = mv_lds_values<AT>();
    __shared__ __align__(16) AT xs[CH];
    __shared__ float red[16];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int threads = blockDim.x;
    const int row0 = (blockIdx.x * (threads >> 6) + wave) * R;
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.0f;
    const bf16 *wr[R];
#pragma unroll
    for (int r = 0; r < R; ++r) wr[r] = W + (size_t)min(row0 + r, rows - 1) * K;
    auto fetch = [&](u32x4v (&w)[R][U], int k0) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = min(k0 + u * 512 + lane * 8, K - 8);  // past the row: any value of it, times x = 0
#pragma unroll
            for (int r = 0; r < R; ++r) w[r][u] = __builtin_nontemporal_load((const u32x4v *)(wr[r] + k));
        }
    };
    auto multiply = [&](const u32x4v (&w)[R][U], int k0) __attribute__((always_inline)) {
        const AT *xp = xs + (k0 & (CH - 1)) + lane * 8;
#pragma unroll
        for (int u = 0; u < U; ++u) {
            float xf[8];
            lds8(xp + u * 512, xf);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float wf[8];
                widen8(w[r][u], wf);
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[r] = fmaf(wf[e], xf[e], acc[r]);
            }
        }
    };
    auto stage = [&](int k0) __attribute__((always_inline)) {
        if (k0) __syncthreads();  // the previous chunk is consumed
        const int n = min(CH, (K - k0 + STEP - 1) / STEP * STEP);
        constexpr int PER = 16 / sizeof(AT);
        for (int i = tid * PER; i < n; i += threads * PER)
            *(u32x4v *)&xs[i] = k0 + i < K ? *(const u32x4v *)(x + k0 + i) : u32x4v{0, 0, 0, 0};
        __syncthreads();
    };
    u32x4v wa[R][U], wb[R][U];
    if constexpr (NV > 0) {
        f32x4 xv[NV], yv4[NV];
        const f32x4 zero{0.f, 0.f, 0.f, 0.f};
        auto load = [&](const float *p, f32x4 (&d)[NV]) __attribute__((always_inline)) {
#pragma unroll
            for (int i = 0; i < NV; ++i) d[i] = (tid + threads * i) * 4 < K ? *(const f32x4 *)(p + (tid + threads * i) * 4) : zero;
        };
        f32x4 wv[NV], bv[NV], pw[NV], pb[NV];
#pragma unroll
        for (int i = 0; i < NV; ++i) bv[i] = pb[i] = zero;
        load(np.x, xv);
        if (np.y) {
            load(np.y, yv4);
            load(np.post_w, pw);
            if (np.post_b) load(np.post_b, pb);
        }
        if (np.pre_w) load(np.pre_w, wv);
        if (np.pre_b) load(np.pre_b, bv);
        fetch(wa, 0);
        const float inv_n = 1.0f / (float)np.cols;
        auto normalize = [&](f32x4 (&d)[NV], const f32x4 (&w)[NV], const f32x4 (&b)[NV]) __attribute__((always_inline)) {
            float mean = 0.0f;
            if (!np.rms) {
                float s = 0.0f;
#pragma unroll
                for (int i = 0; i < NV; ++i) s += (d[i][0] + d[i][1]) + (d[i][2] + d[i][3]);
                mean = pro_sum(s, red) * inv_n;
            }
            float q = 0.0f;
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    d[i][j] = (tid + threads * i) * 4 + j < np.cols ? d[i][j] - mean : 0.0f;
                    q += d[i][j] * d[i][j];
                }
            const float rstd = 1.0f / sqrtf(pro_sum(q, red) * inv_n + np.eps);
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) d[i][j] = d[i][j] * rstd * w[i][j] + b[i][j];  // w = b = 0 past the row
        };
        if (np.y) {
            normalize(yv4, pw, pb);
#pragma unroll
            for (int i = 0; i < NV; ++i) xv[i] += np.mult * yv4[i];
        }
        if (np.step) {
            load(np.step, yv4);
#pragma unroll
            for (int i = 0; i < NV; ++i) xv[i] += yv4[i];
        }
        if (np.x_out && blockIdx.x == 0) {
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if ((tid + threads * i) * 4 < K) *(f32x4 *)(np.x_out + (tid + threads * i) * 4) = xv[i];
        }
        if (np.pre_w) normalize(xv, wv, bv);
        typedef AT at4 __attribute__((ext_vector_type(4)));
        const int n = (K + STEP - 1) / STEP * STEP;
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if ((tid + threads * i) * 4 < n) *(at4 *)&xs[(tid + threads * i) * 4] = __builtin_convertvector(xv[i], at4);
        for (int i = (tid + threads * NV) * 4; i < n; i += threads * 4) *(at4 *)&xs[i] = __builtin_convertvector(zero, at4);
        __syncthreads();
    } else {
        fetch(wa, 0);
    }
    for (int k0 = 0; k0 < K; k0 += 2 * STEP) {
        if (NV == 0 && (k0 & (CH - 1)) == 0) stage(k0);
        if (k0 + STEP < K) fetch(wb, k0 + STEP);
        multiply(wa, k0);
        if (k0 + STEP >= K) break;
        if (k0 + 2 * STEP < K) fetch(wa, k0 + 2 * STEP);
        multiply(wb, k0 + STEP);
    }
    float mine = 0.0f;
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const float t = wave_sum(acc[r]);
        if (lane == r) mine = t;
    }
    if (lane < R && row0 + lane < n_store) {
        const float z = epilogue<EPI>(mine, ea);
        if (to_act(EPI)) ((AT *)yv)[row0 + lane] = (AT)z;
        else ((float *)yv)[row0 + lane] = z;
    }
}

// ------------------------------------------------------------------ prompt batches, bfloat16
// Tile: BN = 128 weight rows x BM activation rows, 64 values of K per stage.  A row of a stage is 128 bytes = eight
// 16-byte chunks; chunk c of row r sits in slot c ^ ((r >> 1) & 7), so that the 16 rows a fragment read touches spread
// over all banks.  A direct load writes 64 consecutive 16-byte slots, so the permutation is in the addresses it reads.
// GROUPED: the row tiles come from a list in device memory (of BM rows at most each), one expert's weights per tile.
template <int BM, int EPI, bool GROUPED>
__global__ __launch_bounds__(256, 2) void k_dense_mm(const bf16 *__restrict__ W, const bf16 *__restrict__ X, void *__restrict__ yv,
                                                     int M, int Np, int ld, int ldx, int k_slice, int64_t ldy, int n_store,
                                                     size_t split_stride, int m_tiles, int n_tiles, int block_rows, const EpiArgs ea,
                                                     const GroupedRows gr) {
    constexpr int BN = 128, BK = 64, ROWS = BN + BM, LOADS = ROWS / 32;
    constexpr int TN = 4, TM = BM / 32;
    __shared__ __align__(16) u32x4v s[2][ROWS * 8];
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // each XCD takes a run of neighbouring tiles (workgroups are dealt to the XCDs round robin); the activation tiles of
    // one weight tile are neighbours
    if (GROUPED) m_tiles = *gr.n_tiles;
    const int total = m_tiles * n_tiles;
    int t = blockIdx.x;
    if (GROUPED && t >= total) return;
    {
        const int per = total >> 3, full = per << 3;
        if (t < full) t = (t & 7) * per + (t >> 3);
    }
    int n0 = (t / m_tiles) * BN, m0 = (t % m_tiles) * BM;
    const int *perm = nullptr;
    if (GROUPED) {
        // expert by expert; within one, its row tiles of one weight tile are neighbours
        GroupTile tile = gr.tiles[t / n_tiles];
        const int local = t - tile.tile0 * n_tiles, nt = local / tile.of_expert;
        n0 = nt * BN;
        tile = gr.tiles[tile.tile0 + local - nt * tile.of_expert];
        W += (size_t)tile.expert * Np * ld;
        perm = gr.perm + tile.first;
        M = tile.count;
        m0 = 0;
    }
    if (block_rows) X += (size_t)(n0 / block_rows) * ld;
    const int kbeg = blockIdx.y * k_slice, kend = min(kbeg + k_slice, ld);
    const bf16 *src[LOADS];
#pragma unroll
    for (int i = 0; i < LOADS; ++i) {
        const int r = (wave + 4 * i) * 8 + (lane >> 3);
        const int c = (lane & 7) ^ ((r >> 1) & 7);
        int xr = min(m0 + max(r - BN, 0), M - 1);
        if (GROUPED) xr = perm[xr] / gr.x_div;
        src[i] = (r < BN ? W + (size_t)min(n0 + r, Np - 1) * ld : X + (size_t)xr * ldx) + kbeg + c * 8;
    }
    auto load = [&](int stage) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < LOADS; ++i) {
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)src[i],
                                             (__attribute__((address_space(3))) void *)&s[stage][(wave + 4 * i) * 64], 16, 0, 0);
            src[i] += BK;
        }
    };
    f32x4 acc[TN][TM];
#pragma unroll
    for (int i = 0; i < TN; ++i)
#pragma unroll
        for (int j = 0; j < TM; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int wn = (wave >> 1) * 64, wm = BN + (wave & 1) * (BM / 2);
    const int r16 = lane & 15, g = lane >> 4;
    const int sw = (r16 >> 1) & 7;  // every tile starts at a multiple of 16 rows: the same swizzle for all of a lane's reads
    auto compute = [&](int stage) __attribute__((always_inline)) {
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
            bf16x8 a[TN], b[TM];
            const int slot = (kk * 4 + g) ^ sw;
#pragma unroll
            for (int i = 0; i < TN; ++i) a[i] = __builtin_bit_cast(bf16x8, s[stage][(wn + i * 16 + r16) * 8 + slot]);
#pragma unroll
            for (int j = 0; j < TM; ++j) b[j] = __builtin_bit_cast(bf16x8, s[stage][(wm + j * 16 + r16) * 8 + slot]);
#pragma unroll
            for (int i = 0; i < TN; ++i)
#pragma unroll
                for (int j = 0; j < TM; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[i], b[j], acc[i][j], 0, 0, 0);
        }
    };
    const int n_it = (kend - kbeg) / BK;
    load(0);
    for (int it = 0; it < n_it; ++it) {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();  // the stage has landed for every wavefront, and the other one is consumed
        if (it + 1 < n_it) load((it + 1) & 1);
        compute(it & 1);
    }
    // C layout: column r16 is the activation row, rows 4g .. 4g+3 are four neighbouring outputs of it
#pragma unroll
    for (int j = 0; j < TM; ++j) {
        int m = m0 + wm - BN + j * 16 + r16;
        if (m >= M) continue;
        if (GROUPED) m = perm[m];
#pragma unroll
        for (int i = 0; i < TN; ++i) {
            const int n = n0 + wn + i * 16 + 4 * g;
            f32x4 z = acc[i][j];
#pragma unroll
            for (int e = 0; e < 4; ++e) z[e] = epilogue<EPI>(z[e], ea);
            if (to_act(EPI)) {
                if (n < n_store) *(bf16x4 *)((bf16 *)yv + (size_t)m * ldy + n) = __builtin_convertvector(z, bf16x4);
            } else if (EPI == EPI_NONE) {
                float *y = (float *)yv + blockIdx.y * split_stride + (size_t)m * ldy + n;
                if (n + 3 < n_store && (ldy & 3) == 0) *(f32x4 *)y = z;
                else
                    for (int e = 0; e < 4; ++e)
                        if (n + e < n_store) y[e] = z[e];
            } else {
                float *y = (float *)yv + (size_t)m * ldy + n;
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (n + e < n_store) y[e] = z[e];
            }
        }
    }
}

// ------------------------------------------------------------------ prompt batches, f32 activations
template <int EPI, bool GROUPED>
__global__ __launch_bounds__(256) void k_dense_mm_f32(const bf16 *__restrict__ W, const float *__restrict__ X, float *__restrict__ yv,
                                                      int M, int ld, int ldx, int64_t ldy, int n_store, int block_rows,
                                                      const EpiArgs ea, const GroupedRows gr) {
    constexpr int B = 64, BK = 32, P = BK + 4;
    __shared__ __align__(16) float sw[B * P], sx[B * P];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int n0 = blockIdx.x * B;
    int m0 = blockIdx.y * B;
    const int *perm = nullptr;
    if (GROUPED) {
        if ((int)blockIdx.y >= *gr.n_tiles) return;
        const GroupTile tile = gr.tiles[blockIdx.y];
        W += (size_t)tile.expert * gr.expert_rows * ld;
        perm = gr.perm + tile.first;
        M = tile.count;
        m0 = 0;
    }
    if (block_rows) X += (size_t)(n0 / block_rows) * ld;
    const int r16 = lane & 15, g = lane >> 4;
    const int wn = (wave >> 1) * 32, wm = (wave & 1) * 32;
    f32x4 acc[2][2];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int lr = tid >> 2, lc = (tid & 3) * 8;  // a row of the stage, 8 of its 32 values
    int xr = min(m0 + lr, M - 1);
    if (GROUPED) xr = perm[xr] / gr.x_div;
    for (int k0 = 0; k0 < ld; k0 += BK) {
        float wf[8], xf[8];
        widen8(*(const u32x4v *)(W + (size_t)(n0 + lr) * ld + k0 + lc), wf);
        lds8(X + (size_t)xr * ldx + k0 + lc, xf);
        __syncthreads();
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            sw[lr * P + lc + e] = wf[e];
            sx[lr * P + lc + e] = xf[e];
        }
        __syncthreads();
#pragma unroll
        for (int kk = 0; kk < BK; kk += 4) {
            float a[2], b[2];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                a[i] = sw[(wn + i * 16 + r16) * P + kk + g];
                b[i] = sx[(wm + i * 16 + r16) * P + kk + g];
            }
#pragma unroll
            for (int i = 0; i < 2; ++i)
#pragma unroll
                for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[j], acc[i][j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        int m = m0 + wm + j * 16 + r16;
        if (m >= M) continue;
        if (GROUPED) m = perm[m];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int n = n0 + wn + i * 16 + 4 * g + e;
                if (n < n_store) yv[(size_t)m * ldy + n] = epilogue<EPI>(acc[i][j][e], ea);
            }
    }
}

// ------------------------------------------------------------------ launches
// Rows over wavefronts: with up to 64 rows per CU one workgroup per CU takes them all, its shape the one that leaves the
// fewest slots empty (the more wavefronts the better, from eight on); longer weights take many workgroups of 8 x 4.
MvShape mv_shape(const candy_hip_device *dev, int64_t rows) {
    const int64_t per_cu = (rows + dev->num_cus - 1) / dev->num_cus;
    if (per_cu > 64) return {8, 4};
    if (per_cu <= 8) return {8, 1};
    MvShape best{16, 4};
    int64_t best_cost = 1 << 30;
    for (int r : {1, 2, 4})
        for (int w = 8; w <= 16; ++w) {
            const int64_t slots = (int64_t)w * r;
            if (slots < per_cu) continue;
            const int64_t cost = (slots - per_cu) * 64 - w;
            if (cost < best_cost) { best_cost = cost; best = {w, r}; }
        }
    return best;
}

template <class AT, int R, int EPI>
static void launch_mv_nv(candy_hip_device *dev, const DenseLaunch &L, int waves, int nv, const NormPro &np) {
    const int64_t per_wg = (int64_t)waves * R;
    const dim3 g((unsigned)((L.n_store + per_wg - 1) / per_wg)), b((unsigned)(64 * waves));
    const EpiArgs ea{L.scale, L.cap};
    const AT *x = (const AT *)L.x;
    const bf16 *W = (const bf16 *)L.w->data;
    const int K = (int)L.w->ld, rows = (int)L.w->rows_pad, ns = (int)L.n_store;
    if constexpr (sizeof(AT) == 2 || (R == 1 && EPI == EPI_NONE)) {
        switch (nv) {
        case 1: hipLaunchKernelGGL((k_dense_mv<AT, R, EPI, 1>), g, b, 0, dev->stream, x, W, L.y, K, rows, ns, ea, np); return;
        case 2: hipLaunchKernelGGL((k_dense_mv<AT, R, EPI, 2>), g, b, 0, dev->stream, x, W, L.y, K, rows, ns, ea, np); return;
        default: break;
        }
    }
    hipLaunchKernelGGL((k_dense_mv<AT, R, EPI, 0>), g, b, 0, dev->stream, x, W, L.y, K, rows, ns, ea, np);
}

template <class AT, int R>
static void launch_mv_epi(candy_hip_device *dev, const DenseLaunch &L, int waves, int nv, const NormPro &np) {
    switch (L.epi) {
    case EPI_RELU2: launch_mv_nv<AT, R, EPI_RELU2>(dev, L, waves, nv, np); break;
    case EPI_CAP: launch_mv_nv<AT, R, EPI_CAP>(dev, L, waves, nv, np); break;
    case EPI_ACT: launch_mv_nv<AT, R, EPI_ACT>(dev, L, waves, nv, np); break;
    default: launch_mv_nv<AT, R, EPI_NONE>(dev, L, waves, nv, np); break;
    }
}

template <class AT>
static int launch_mv(candy_hip_device *dev, const DenseLaunch &L, const MvShape &s, int nv = 0, const NormPro &np = NormPro{}) {
    switch (s.rows) {
    case 1: launch_mv_epi<AT, 1>(dev, L, s.waves, nv, np); break;
    case 2: launch_mv_epi<AT, 2>(dev, L, s.waves, nv, np); break;
    default: launch_mv_epi<AT, 4>(dev, L, s.waves, nv, np); break;
    }
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

int launch_dense_norm(candy_hip_device *dev, const DenseLaunch &L, const NormArgs &A) {
    // every workgroup repeats the norms: one per CU, or the launch of their own is the cheaper one
    const MvShape s = mv_shape(dev, L.n_store);
    const int per = 256 * s.waves, nv = (int)((L.w->ld + per - 1) / per);
    if (L.m != 1 || (L.f32 && (s.rows != 1 || L.epi != EPI_NONE)) || A.rows != 1 || A.y.copies != 1 || A.slots || A.row_ids ||
        A.x == A.x_out || nv > 2 || L.w->ld > (L.f32 ? mv_lds_values<float>() : mv_lds_values<bf16>()) || L.n_store > 64 * (int64_t)dev->num_cus)
        return CANDY_HIP_ERR_UNSUPPORTED;
    CANDY_REQUIRE(pad64(A.cols) == L.w->ld, "internal: norm and contraction of different widths");
    if (L.partial) *L.partial = Partial{(const float *)L.y, 1, 0, (int)L.ldy};
    const NormPro np{A.x, A.y.p, A.post_w, A.post_b, A.step, A.pre_w, A.pre_b, A.x_out, A.mult, A.eps, A.cols, A.rms};
    return L.f32 ? launch_mv<float>(dev, L, s, nv, np) : launch_mv<bf16>(dev, L, s, nv, np);
}

template <int BM>
static int launch_mm(candy_hip_device *dev, const DenseLaunch &L) {
    const int m_tiles = (L.m + BM - 1) / BM, n_tiles = (int)((L.w->rows_pad + 127) / 128);
    const int64_t tiles = (int64_t)m_tiles * n_tiles;
    CANDY_REQUIRE(tiles <= 0x7FFFFFFF, "matrix too large");
    const int K = (int)L.w->ld;
    int splits = 1;
    void *y = L.y;
    int64_t ldy = L.ldy, n_store = L.n_store;
    size_t stride = 0;
    if (L.partial) {
        // two workgroups fit a CU; a slice keeps at least 512 values of K
        const int64_t room = 2 * (int64_t)dev->num_cus / tiles;
        splits = (int)std::max<int64_t>(1, std::min<int64_t>(std::min<int64_t>(room, 8), K / 512));
        if (splits > 1) {
            ldy = n_store = L.w->rows_pad;
            stride = (size_t)L.m * ldy;
            if (int rc = splitk_workspace(dev, stride * splits * sizeof(float), &y)) return rc;
        }
    }
    const int k_slice = (int)pad64((K + splits - 1) / splits);
    splits = (K + k_slice - 1) / k_slice;
    if (L.partial) {
        L.partial->p = (const float *)y;
        L.partial->copies = splits;
        L.partial->stride = stride;
        L.partial->ld = (int)ldy;
    }
    const dim3 g((unsigned)tiles, (unsigned)splits), b(256);
    const EpiArgs ea{L.scale, L.cap};
    const bf16 *W = (const bf16 *)L.w->data, *X = (const bf16 *)L.x;
#define CANDY_MM(EPI)                                                                                                     \
    hipLaunchKernelGGL((k_dense_mm<BM, EPI, false>), g, b, 0, dev->stream, W, X, y, L.m, (int)L.w->rows_pad, K, (int)L.ldx,   \
                       k_slice, ldy, (int)n_store, stride, m_tiles, n_tiles, L.block_rows, ea, GroupedRows{})
    switch (L.epi) {
    case EPI_RELU2: CANDY_MM(EPI_RELU2); break;
    case EPI_CAP: CANDY_MM(EPI_CAP); break;
    case EPI_ACT: CANDY_MM(EPI_ACT); break;
    default: CANDY_MM(EPI_NONE); break;
    }
#undef CANDY_MM
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

// Rows dealt to experts: the grid has room for max_tiles row tiles, workgroups past the list's end leave at once.
template <int BM>
static int launch_mm_grouped(candy_hip_device *dev, const DenseLaunch &L) {
    const GroupedRows &gr = *L.group;
    const int n_tiles = (gr.expert_rows + 127) / 128, K = (int)L.w->ld;
    const int64_t tiles = (int64_t)gr.max_tiles * n_tiles;
    CANDY_REQUIRE(tiles <= 0x7FFFFFFF, "matrix too large");
    const dim3 g((unsigned)tiles), b(256);
    const EpiArgs ea{L.scale, L.cap};
    const bf16 *W = (const bf16 *)L.w->data, *X = (const bf16 *)L.x;
#define CANDY_MMG(EPI)                                                                                                       \
    hipLaunchKernelGGL((k_dense_mm<BM, EPI, true>), g, b, 0, dev->stream, W, X, L.y, L.m, gr.expert_rows, K, (int)L.ldx, K,  \
                       L.ldy, (int)L.n_store, (size_t)0, 0, n_tiles, 0, ea, gr)
    if (L.epi == EPI_RELU2) CANDY_MMG(EPI_RELU2);
    else CANDY_MMG(EPI_NONE);
#undef CANDY_MMG
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

int launch_dense(candy_hip_device *dev, const DenseLaunch &L) {
    const candy_hip_dense *w = L.w;
    CANDY_REQUIRE(L.m > 0 && w->rows_pad <= 0x7FFFFFFF && w->ld <= 0x7FFFFFFF && L.ldx >= w->ld && L.ldx <= 0x7FFFFFFF,
                  "internal: dense contraction of a shape the kernels do not take");
    CANDY_REQUIRE(L.n_store <= w->rows_pad && L.ldy >= L.n_store, "internal: dense output row too short");
    const int64_t out_rows = L.group ? L.group->expert_rows : w->rows_pad;
    CANDY_REQUIRE(!to_act(L.epi) || (L.n_store == out_rows && (L.ldy & 63) == 0), "internal: activation rows must be padded");
    CANDY_REQUIRE(L.block_rows == 0 || (!L.partial && L.block_rows % 128 == 0 && w->rows_pad % L.block_rows == 0 &&
                                        L.ldx >= w->rows_pad / L.block_rows * w->ld), "internal: block-diagonal contraction");
    if (L.group) {
        CANDY_REQUIRE((L.epi == EPI_NONE || L.epi == EPI_RELU2) && !L.partial && !L.block_rows && L.group->expert_rows % 64 == 0 &&
                          w->rows % L.group->expert_rows == 0 && L.group->max_tiles <= 65535,
                      "internal: grouped contraction");
        if (!L.f32 && L.group->tile_rows == 128) return launch_mm_grouped<128>(dev, L);
        CANDY_REQUIRE(L.group->tile_rows == 64, "internal: row tiles of 64");
        if (!L.f32) return launch_mm_grouped<64>(dev, L);
    }
    if (L.partial) {
        L.partial->p = (const float *)L.y;
        L.partial->copies = 1;
        L.partial->stride = 0;
        L.partial->ld = (int)L.ldy;
    }
    if (L.m == 1 && !L.group && !L.block_rows) {
        const MvShape s = mv_shape(dev, L.n_store);
        return L.f32 ? launch_mv<float>(dev, L, s) : launch_mv<bf16>(dev, L, s);
    }
    if (!L.f32) return L.m <= 64 ? launch_mm<64>(dev, L) : launch_mm<128>(dev, L);
    const dim3 g((unsigned)(out_rows / 64), (unsigned)(L.group ? L.group->max_tiles : (L.m + 63) / 64)), b(256);
    CANDY_REQUIRE((L.m + 63) / 64 <= 65535, "prompt too long for one pass");
    const EpiArgs ea{L.scale, L.cap};
    const bf16 *W = (const bf16 *)w->data;
    const float *X = (const float *)L.x;
#define CANDY_MM32(EPI)                                                                                                 \
    do {                                                                                                                \
        if (L.group)                                                                                                    \
            hipLaunchKernelGGL((k_dense_mm_f32<EPI, true>), g, b, 0, dev->stream, W, X, (float *)L.y, L.m, (int)w->ld,  \
                               (int)L.ldx, L.ldy, (int)L.n_store, 0, ea, *L.group);                                     \
        else                                                                                                            \
            hipLaunchKernelGGL((k_dense_mm_f32<EPI, false>), g, b, 0, dev->stream, W, X, (float *)L.y, L.m, (int)w->ld, \
                               (int)L.ldx, L.ldy, (int)L.n_store, L.block_rows, ea, GroupedRows{});                     \
    } while (0)
    switch (L.epi) {
    case EPI_RELU2: CANDY_MM32(EPI_RELU2); break;
    case EPI_CAP: CANDY_MM32(EPI_CAP); break;
    default: CANDY_MM32(EPI_NONE); break;  // ACT: f32 is the activation format
    }
#undef CANDY_MM32
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

// rows ids[i] of a bfloat16 table, widened and scaled; an id outside the table raises the handle's fault word and gives zeros
__global__ __launch_bounds__(256) void k_dense_gather(const bf16 *__restrict__ W, int64_t rows, int64_t ld,
                                                      const int64_t *__restrict__ ids, float *__restrict__ out, int64_t ldo,
                                                      float scale, int *fault) {
    const int64_t id = ids[blockIdx.y];
    const int64_t c = ((int64_t)blockIdx.x * 256 + threadIdx.x) * 8;
    if (c >= ld) return;
    float f[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (id >= 0 && id < rows) widen8(*(const u32x4v *)(W + id * ld + c), f);
    else if (c == 0) *fault = 1;
    float *o = out + (int64_t)blockIdx.y * ldo + c;
    *(f32x4 *)o = f32x4{f[0], f[1], f[2], f[3]} * scale;
    *(f32x4 *)(o + 4) = f32x4{f[4], f[5], f[6], f[7]} * scale;
}

int launch_dense_gather(candy_hip_device *dev, const candy_hip_dense *w, const int64_t *ids, int64_t n, float *out, int64_t ldo,
                        float scale) {
    for (int64_t i0 = 0; i0 < n; i0 += 65535) {
        const int64_t part = std::min<int64_t>(n - i0, 65535);
        hipLaunchKernelGGL(k_dense_gather, dim3((unsigned)((w->ld / 8 + 255) / 256), (unsigned)part), dim3(256), 0, dev->stream,
                           (const bf16 *)w->data, w->rows, w->ld, ids + i0, out + i0 * ldo, ldo, scale, dev->fault);
        CANDY_LAUNCH_CHECK();
    }
    return CANDY_HIP_OK;
}

// f32 rows -> activation rows of ld values, zero past cols
template <class AT>
__global__ __launch_bounds__(256) void k_to_act(const float *__restrict__ src, AT *__restrict__ dst, int64_t rows, int64_t cols, int64_t ld) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= rows * ld) return;
    const int64_t r = i / ld, c = i % ld;
    dst[i] = c < cols ? (AT)src[r * cols + c] : (AT)0.0f;
}
// activation rows -> dense f32
template <class AT>
__global__ __launch_bounds__(256) void k_from_act(const AT *__restrict__ src, float *__restrict__ dst, int64_t rows, int64_t cols, int64_t ld) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= rows * cols) return;
    dst[i] = (float)src[i / cols * ld + i % cols];
}

int launch_to_act(candy_hip_device *dev, bool f32, const float *src, void *dst, int64_t rows, int64_t cols, int64_t ld) {
    const int64_t grid = (rows * ld + 255) / 256;
    CANDY_REQUIRE(grid <= 0x7FFFFFFF, "matrix too large");
    if (f32) hipLaunchKernelGGL((k_to_act<float>), dim3((unsigned)grid), dim3(256), 0, dev->stream, src, (float *)dst, rows, cols, ld);
    else hipLaunchKernelGGL((k_to_act<bf16>), dim3((unsigned)grid), dim3(256), 0, dev->stream, src, (bf16 *)dst, rows, cols, ld);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}
int launch_from_act(candy_hip_device *dev, bool f32, const void *src, float *dst, int64_t rows, int64_t cols, int64_t ld) {
    const int64_t grid = (rows * cols + 255) / 256;
    CANDY_REQUIRE(grid <= 0x7FFFFFFF, "matrix too large");
    if (f32) hipLaunchKernelGGL((k_from_act<float>), dim3((unsigned)grid), dim3(256), 0, dev->stream, (const float *)src, dst, rows, cols, ld);
    else hipLaunchKernelGGL((k_from_act<bf16>), dim3((unsigned)grid), dim3(256), 0, dev->stream, (const bf16 *)src, dst, rows, cols, ld);
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}

}  // namespace candy

using namespace candy;

extern "C" {

int candy_hip_dense_upload(candy_hip_device *dev, int64_t rows, int64_t cols, const uint16_t *host_bf16, candy_hip_dense **out) {
    CANDY_REQUIRE(out, "out is nil");
    *out = nullptr;
    CANDY_REQUIRE(dev, "device handle is nil");
    CANDY_REQUIRE(rows > 0 && cols > 0 && rows <= 0x7FFFFF00 && cols <= 0x7FFFFF00, "invalid matrix dimensions %lld x %lld",
                  (long long)rows, (long long)cols);
    CANDY_REQUIRE(host_bf16, "host weight is nil");
    if (int rc = use_device(dev)) return rc;
    const int64_t rp = pad64(rows), ld = pad64(cols);
    void *d = nullptr;
    const size_t bytes = (size_t)rp * ld * 2;
    if (int rc = candy_hip_alloc(dev, bytes, &d)) return rc;
    int rc = CANDY_HIP_OK;
    if (rp != rows || ld != cols) rc = candy_hip_zero(dev, d, bytes);
    if (!rc) {
        hipError_t e = hipMemcpy2DAsync(d, (size_t)ld * 2, host_bf16, (size_t)cols * 2, (size_t)cols * 2, (size_t)rows,
                                        hipMemcpyHostToDevice, dev->stream);
        if (e == hipSuccess) e = hipStreamSynchronize(dev->stream);
        if (e != hipSuccess) rc = fail(CANDY_HIP_ERR_HIP, "weight upload failed: %s", hipGetErrorString(e));
    }
    if (rc) {
        (void)candy_hip_free(dev, d);
        return rc;
    }
    candy_hip_dense *w = new candy_hip_dense();
    w->dev = dev; w->rows = rows; w->cols = cols; w->rows_pad = rp; w->ld = ld; w->data = d;
    *out = w;
    return CANDY_HIP_OK;
}

int candy_hip_dense_free(candy_hip_dense *w) {
    if (!w) return CANDY_HIP_OK;
    const int rc = candy_hip_free(w->dev, w->data);
    delete w;
    return rc;
}

int candy_hip_dense_info(const candy_hip_dense *w, int64_t *rows, int64_t *cols, size_t *nbytes) {
    CANDY_REQUIRE(w, "weight is nil");
    if (rows) *rows = w->rows;
    if (cols) *cols = w->cols;
    if (nbytes) *nbytes = (size_t)w->rows_pad * w->ld * 2;
    return CANDY_HIP_OK;
}

int candy_hip_dense_matmul(candy_hip_device *dev, const candy_hip_dense *w, const float *dev_x, int64_t m, int act, int epilogue,
                           float scale, float cap, float *dev_y) {
    CANDY_REQUIRE(w, "rhs weight is nil");
    CANDY_REQUIRE(dev && w->dev == dev, "rhs storage must live on the same HIP device");
    CANDY_REQUIRE(m >= 0 && m <= 1 << 20, "invalid matrix dimensions");
    CANDY_REQUIRE(act == CANDY_HIP_ACT_BF16 || act == CANDY_HIP_ACT_F32, "unknown activation format %d", act);
    CANDY_REQUIRE(epilogue >= EPI_NONE && epilogue <= EPI_ACT, "unknown epilogue %d", epilogue);
    if (m == 0) return CANDY_HIP_OK;
    CANDY_REQUIRE(dev_x && dev_y, "nil pointer");
    if (int rc = use_device(dev)) return rc;
    const bool f32 = act == CANDY_HIP_ACT_F32;
    const size_t x_bytes = (size_t)m * w->ld * 4, y_bytes = (size_t)m * w->rows_pad * 4;
    void *ws = nullptr;
    if (int rc = workspace(dev, x_bytes + y_bytes, &ws)) return rc;
    if (int rc = launch_to_act(dev, f32, dev_x, ws, m, w->cols, w->ld)) return rc;
    DenseLaunch L;
    L.w = w; L.x = ws; L.ldx = w->ld; L.f32 = f32; L.m = (int)m; L.epi = epilogue; L.scale = scale; L.cap = cap;
    if (!to_act(epilogue)) {
        L.y = dev_y; L.ldy = L.n_store = w->rows;
        return launch_dense(dev, L);
    }
    L.y = (uint8_t *)ws + x_bytes; L.ldy = L.n_store = w->rows_pad;
    if (int rc = launch_dense(dev, L)) return rc;
    return launch_from_act(dev, f32, L.y, dev_y, m, w->rows, w->rows_pad);
}

int candy_hip_dense_sweep(candy_hip_device *dev, const candy_hip_dense *const *ws, int n_ws, const float *dev_x, int64_t m,
                          int epilogue, int iters, float *elapsed_ms) {
    CANDY_REQUIRE(dev && ws && n_ws > 0 && dev_x && elapsed_ms && iters > 0 && m > 0 && m <= 1 << 20, "nil argument");
    CANDY_REQUIRE(epilogue >= EPI_NONE && epilogue <= EPI_ACT, "unknown epilogue %d", epilogue);
    for (int i = 0; i < n_ws; ++i)
        CANDY_REQUIRE(ws[i] && ws[i]->dev == dev && ws[i]->rows == ws[0]->rows && ws[i]->cols == ws[0]->cols,
                      "weights of one sweep share a device and a shape");
    if (int rc = use_device(dev)) return rc;
    const candy_hip_dense *w = ws[0];
    const size_t x_bytes = (size_t)m * w->ld * 2;
    void *buf = nullptr;
    if (int rc = workspace(dev, x_bytes + (size_t)m * w->rows_pad * 4, &buf)) return rc;
    if (int rc = launch_to_act(dev, false, dev_x, buf, m, w->cols, w->ld)) return rc;
    DenseLaunch L;
    Partial part;
    L.x = buf; L.ldx = w->ld; L.m = (int)m; L.epi = epilogue; L.scale = 1.0f; L.cap = 30.0f;
    L.y = (uint8_t *)buf + x_bytes; L.ldy = L.n_store = w->rows_pad;
    if (epilogue == EPI_NONE) L.partial = &part;
    CANDY_HIP_TRY(hipEventRecord(dev->ev_start, dev->stream));
    for (int i = 0; i < iters; ++i) {
        L.w = ws[i % n_ws];
        if (int rc = launch_dense(dev, L)) return rc;
    }
    CANDY_HIP_TRY(hipEventRecord(dev->ev_stop, dev->stream));
    CANDY_HIP_TRY(hipEventSynchronize(dev->ev_stop));
    CANDY_HIP_TRY(hipEventElapsedTime(elapsed_ms, dev->ev_start, dev->ev_stop));
    return CANDY_HIP_OK;
}

}  // extern "C"
