// Routed experts with squared-ReLU feed-forwards (equations and layouts: include/candy_hip.h).
//   prompts: k_route        router scores of 16 tokens in f32 on the matrix cores (activations as the sum of three bfloat16
//                           parts, which is exact), softmax, the choice and its weights
//            k_deal         slots (token, choice) sorted by expert, and the list of row tiles
//            the experts' contractions over their rows, and the shared expert's (dense.hip); k_norm_chain sums the slots
//   decode:  the router as a contraction of one row (dense.hip)
//            k_expert_up    choice in the prologue; the chosen experts' and the shared one's rows, squared ReLU, weighted
//            k_expert_down  one contraction over the concatenation of their inner activations
// (No counterpart in the reference, which has no routed layer.)
#include <algorithm>

#include "dense.h"

namespace candy {

// What the choice orders scores by: every value has its place, so that the choice names `top` different experts even where
// a model's numbers have gone wrong.
__device__ __forceinline__ float ordered(float z) { return z == z ? z : -INFINITY; }

// One wavefront, lane e holding score e of a token's E <= 64 (ordered()): lane k leaves with the k-th choice and its weight.
__device__ __forceinline__ void choose64(float v, int E, int top, int &id, float &weight) {
    const int lane = threadIdx.x & 63;
    uint64_t left = E == 64 ? ~0ull : (1ull << E) - 1;
    if (lane >= E) v = -INFINITY;
    float best = wave_max(v), mine = -INFINITY;
    const float mx = fmaxf(best, LOW), sum = wave_sum(lane < E ? expf(v - mx) : 0.0f);
    id = 0;
    for (int k = 0; k < top; ++k) {
        if (k) best = wave_max(v);
        const int e = __ffsll((unsigned long long)(__ballot(v == best) & left)) - 1;   // not empty: `left` has top - k members
        left &= ~(1ull << e);
        if (lane == k) { id = e; mine = best; }
        if (lane == e) v = -INFINITY;
    }
    const float s = lane < top ? expf(mine - mx) / sum : 0.0f;
    weight = s / (wave_sum(s) + 1e-20f);
}

// The same for any number of scores z[0 .. E) in LDS; choices and weights in order of their scores.
__device__ __forceinline__ void choose(const float *z, int E, int top, int *ids, float *weights) {
    const int lane = threadIdx.x & 63;
    if (E <= 64) {
        int id;
        float w;
        choose64(lane < E ? z[lane] : 0.0f, E, top, id, w);
        if (lane < top) {
            ids[lane] = id;
            weights[lane] = w;
        }
        return;
    }
    float mx = LOW;
    for (int e = lane; e < E; e += 64) mx = fmaxf(mx, z[e]);
    mx = wave_max(mx);
    float sum = 0.0f;
    for (int e = lane; e < E; e += 64) sum += expf(z[e] - mx);
    sum = wave_sum(sum);
    float chosen = 0.0f;
    for (int e0 = 0; e0 < E; e0 += 64) {
        const int e = e0 + lane;
        const float mine = e < E ? z[e] : 0.0f;
        int rank = 0;
#pragma unroll 8
        for (int f = 0; f < E; ++f) rank += z[f] > mine || (z[f] == mine && f < e);
        if (e < E && rank < top) {
            const float s = expf(mine - mx) / sum;
            ids[rank] = e;
            weights[rank] = s;
            chosen += s;
        }
    }
    chosen = wave_sum(chosen) + 1e-20f;
    __builtin_amdgcn_wave_barrier();
    for (int k = lane; k < top; k += 64) weights[k] /= chosen;
}

// ------------------------------------------------------------------ prompts
constexpr int ROUTE_T = 16, ROUTE_W = 8, ROUTE_U = 4;   // tokens and wavefronts of a workgroup, K steps requested together
// grid ceil(n / 16), 8 wavefronts that share K; 64 experts per round
__global__ __launch_bounds__(64 * ROUTE_W) void k_route(const float *__restrict__ x, int64_t ldx, const bf16 *__restrict__ W, int ld, int E,
                                                        int top, int n, int *__restrict__ ids, float *__restrict__ weights) {
    extern __shared__ __align__(16) float z[];        // [16][E] scores, then [4][64][17] sums of pairs of wavefronts
    const int Ep = E | 1;                              // odd pitch
    float *red = z + ROUTE_T * Ep;
    int *s_ids = (int *)red;                           // once the scores stand: [16][top], [16][top]
    float *s_w = red + ROUTE_T * top;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
    const int t0 = blockIdx.x * ROUTE_T, steps = ld >> 5;
    const float *xr = x + (size_t)min(t0 + r16, n - 1) * ldx + g * 8;
    for (int e0 = 0; e0 < E; e0 += 64) {
        f32x4 acc[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
        const bf16 *w = W + (size_t)(e0 + r16) * ld + g * 8;
        const int strips = min(4, (E - e0 + 15) >> 4);
        for (int s0 = wave; s0 < steps; s0 += ROUTE_W * ROUTE_U) {
            f32x4 xv[ROUTE_U][2];
            bf16x8 wv[ROUTE_U][4];
#pragma unroll
            for (int u = 0; u < ROUTE_U; ++u) {
                const int k = min(s0 + u * ROUTE_W, steps - 1) * 32;
                xv[u][0] = *(const f32x4 *)(xr + k);
                xv[u][1] = *(const f32x4 *)(xr + k + 4);
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (i < strips) wv[u][i] = *(const bf16x8 *)(w + (size_t)i * 16 * ld + k);
            }
#pragma unroll
            for (int u = 0; u < ROUTE_U; ++u) {
                if (s0 + u * ROUTE_W >= steps) break;
                bf16x8 part[3];
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    const float f = xv[u][j >> 2][j & 3];
                    part[0][j] = (bf16)f;
                    const float r1 = f - (float)part[0][j];
                    part[1][j] = (bf16)r1;
                    part[2][j] = (bf16)(r1 - (float)part[1][j]);
                }
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (i < strips) {
#pragma unroll
                        for (int p = 2; p >= 0; --p) acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u][i], part[p], acc[i], 0, 0, 0);
                    }
            }
        }
        // lane: token r16, experts e0 + 16 i + 4 g + j
        for (int half = 1; half >= 0; --half) {   // the second four wavefronts' sums, then the first four's on top
            if (wave >> 2 == half) {
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        float *s = &red[((wave & 3) * 64 + i * 16 + 4 * g + j) * 17 + r16];
                        *s = half ? acc[i][j] : *s + acc[i][j];
                    }
            }
            __syncthreads();
        }
        for (int i = tid; i < 64 * ROUTE_T; i += 64 * ROUTE_W) {
            const int t = i & 15, e = i >> 4;
            if (e0 + e >= E) continue;
            float sum = 0.0f;
#pragma unroll
            for (int v = 0; v < ROUTE_W / 2; ++v) sum += red[(v * 64 + e) * 17 + t];
            z[t * Ep + e0 + e] = ordered(sum);
        }
        __syncthreads();
    }
    for (int t = wave; t < ROUTE_T; t += ROUTE_W) choose(z + t * Ep, E, top, s_ids + t * top, s_w + t * top);
    __syncthreads();
    for (int i = tid; i < ROUTE_T * top; i += 64 * ROUTE_W)
        if (t0 + i / top < n) {
            ids[(size_t)t0 * top + i] = s_ids[i];
            weights[(size_t)t0 * top + i] = s_w[i];
        }
}

constexpr int MAX_EXPERTS = 1024;
// One workgroup of 1024: perm[0 .. count) = the slots, expert by expert; tiles of at most `rows` of one expert each.
__global__ __launch_bounds__(1024) void k_deal(const int *__restrict__ ids, int count, int E, int rows, int *__restrict__ perm,
                                               GroupTile *__restrict__ tiles, int *__restrict__ n_tiles) {
    __shared__ int members[MAX_EXPERTS], end[2][MAX_EXPERTS], tile_end[2][MAX_EXPERTS];
    const int tid = threadIdx.x;
    members[tid] = 0;
    __syncthreads();
    constexpr int AHEAD = 4;
    for (int i0 = tid; i0 < count; i0 += 1024 * AHEAD) {
        int e[AHEAD];
#pragma unroll
        for (int k = 0; k < AHEAD; ++k) e[k] = ids[min(i0 + 1024 * k, count - 1)];
#pragma unroll
        for (int k = 0; k < AHEAD; ++k)
            if (i0 + 1024 * k < count) atomicAdd(&members[e[k]], 1);
    }
    __syncthreads();
    const int mine = members[tid], my_tiles = (mine + rows - 1) / rows;
    int cur = 0;
    end[0][tid] = mine;
    tile_end[0][tid] = my_tiles;
    __syncthreads();
    for (int d = 1; d < MAX_EXPERTS; d <<= 1) {   // inclusive sums
        end[cur ^ 1][tid] = end[cur][tid] + (tid >= d ? end[cur][tid - d] : 0);
        tile_end[cur ^ 1][tid] = tile_end[cur][tid] + (tid >= d ? tile_end[cur][tid - d] : 0);
        cur ^= 1;
        __syncthreads();
    }
    const int begin = end[cur][tid] - mine, tile0 = tile_end[cur][tid] - my_tiles;
    for (int k = 0; k < my_tiles; ++k) tiles[tile0 + k] = GroupTile{tid, begin + k * rows, min(rows, mine - k * rows), (uint16_t)tile0, (uint16_t)my_tiles};
    if (tid == MAX_EXPERTS - 1) *n_tiles = tile_end[cur][tid];
    members[tid] = begin;
    __syncthreads();
    for (int i0 = tid; i0 < count; i0 += 1024 * AHEAD) {
        int e[AHEAD];
#pragma unroll
        for (int k = 0; k < AHEAD; ++k) e[k] = ids[min(i0 + 1024 * k, count - 1)];
#pragma unroll
        for (int k = 0; k < AHEAD; ++k)
            if (i0 + 1024 * k < count) perm[atomicAdd(&members[e[k]], 1)] = i0 + 1024 * k;
    }
}

// ------------------------------------------------------------------ decode
struct RowArgs {
    const bf16 *W, *shared;   // up: [E * rows_e][ld], [rows_s][ld]; down: [E * d_p][rows_e], [d_p][rows_s]
    int E, top, rows_e, rows_s, ld;   // rows_e / rows_s: padded inner widths of an expert and of the shared one
};

constexpr int EXP_U = 4;   // 16-byte requests per row in flight

// Rows of the concatenated up matrices, R per wavefront.  FEW: at most 64 experts, every wavefront makes the choice for
// itself and requests its weights before the activations are staged.  LDS: x; else also the scores and the choice.
template <class AT, int R, bool FEW>
__global__ __launch_bounds__(1024) void k_expert_up(const RowArgs a, const float *__restrict__ x, const float *__restrict__ logits,
                                                    AT *__restrict__ act, int *__restrict__ sel) {
    extern __shared__ __align__(16) uint8_t lds[];
    AT *xs = (AT *)lds;
    float *z = (float *)(xs + a.ld), *gate = z + a.E;
    int *ids = (int *)(gate + a.top);
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), threads = blockDim.x;
    const int total = a.top * a.rows_e + a.rows_s, row0 = (blockIdx.x * (threads >> 6) + wave) * R;
    int my_id = 0;
    float my_weight = 0.0f;
    auto stage = [&]() __attribute__((always_inline)) {
        typedef AT at4 __attribute__((ext_vector_type(4)));
        for (int i = tid * 4; i < a.ld; i += threads * 4) *(at4 *)&xs[i] = __builtin_convertvector(*(const f32x4 *)(x + i), at4);
    };
    if (FEW) {
        choose64(ordered(logits[min(lane, a.E - 1)]), a.E, a.top, my_id, my_weight);
        if (blockIdx.x == 0 && wave == 0 && lane < a.top) sel[lane] = my_id;
    } else {
        for (int e = tid; e < a.E; e += threads) z[e] = ordered(logits[e]);
        stage();
        __syncthreads();
        if (wave == 0) {
            choose(z, a.E, a.top, ids, gate);
            if (blockIdx.x == 0)
                for (int k = lane; k < a.top; k += 64) sel[k] = ids[k];
        }
        __syncthreads();
    }
    const bf16 *w[R];
    float scale[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int row = min(row0 + r, total - 1), k = row / a.rows_e;
        if (k < a.top) {
            const int id = FEW ? __builtin_amdgcn_readlane(my_id, k) : ids[k];
            w[r] = a.W + ((size_t)id * a.rows_e + (row - k * a.rows_e)) * a.ld;
            scale[r] = FEW ? __int_as_float(__builtin_amdgcn_readlane(__float_as_int(my_weight), k)) : gate[k];
        } else {
            w[r] = a.shared + (size_t)(row - a.top * a.rows_e) * a.ld;
            scale[r] = 1.0f;
        }
    }
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.0f;
    for (int k0 = 0; k0 < a.ld; k0 += EXP_U * 512) {
        u32x4v v[R][EXP_U];
#pragma unroll
        for (int u = 0; u < EXP_U; ++u)
#pragma unroll
            for (int r = 0; r < R; ++r) v[r][u] = __builtin_nontemporal_load((const u32x4v *)(w[r] + min(k0 + u * 512 + lane * 8, a.ld - 8)));
        if (FEW && k0 == 0) {
            stage();
            __syncthreads();
        }
#pragma unroll
        for (int u = 0; u < EXP_U; ++u) {
            const int k = k0 + u * 512 + lane * 8;
            if (k >= a.ld) continue;
            float xf[8];
            lds8(xs + k, xf);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float f[8];
                widen8(v[r][u], f);
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[r] = fmaf(f[e], xf[e], acc[r]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const float t = fmaxf(wave_sum(acc[r]), 0.0f);
        if (lane == r && row0 + r < total) act[row0 + r] = (AT)(t * t * scale[r]);
    }
}

// Rows of the result: an expert's inner activations meet its down matrix, all of them one long sum.  LDS: the
// activations, and per 64 of them where their weights start.
template <class AT, int R>
__global__ __launch_bounds__(1024) void k_expert_down(const RowArgs a, int d_p, const AT *__restrict__ act, const int *__restrict__ sel,
                                                      float *__restrict__ y) {
    extern __shared__ __align__(16) uint8_t lds[];
    const int K = a.top * a.rows_e + a.rows_s, chunks = K >> 6;
    const bf16 **base = (const bf16 **)lds;
    int *pitch = (int *)(base + chunks);
    AT *xs = (AT *)(pitch + ((chunks + 3) & ~3));
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), threads = blockDim.x;
    const int row0 = (blockIdx.x * (threads >> 6) + wave) * R;
    for (int i = tid; i < chunks; i += threads) {
        const int k = (i << 6) / a.rows_e;
        if (k < a.top) {
            base[i] = a.W + (size_t)sel[k] * d_p * a.rows_e + ((i << 6) - k * a.rows_e);
            pitch[i] = a.rows_e;
        } else {
            base[i] = a.shared + ((i << 6) - a.top * a.rows_e);
            pitch[i] = a.rows_s;
        }
    }
    constexpr int PER = 16 / sizeof(AT);
    for (int i = tid * PER; i < K; i += threads * PER) *(u32x4v *)&xs[i] = *(const u32x4v *)(act + i);
    __syncthreads();
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.0f;
    for (int k0 = 0; k0 < K; k0 += EXP_U * 512) {
        u32x4v v[R][EXP_U];
#pragma unroll
        for (int u = 0; u < EXP_U; ++u) {
            const int k = min(k0 + u * 512 + lane * 8, K - 8), c = k >> 6;
            const bf16 *p = base[c] + (k & 63);
#pragma unroll
            for (int r = 0; r < R; ++r) v[r][u] = __builtin_nontemporal_load((const u32x4v *)(p + (size_t)min(row0 + r, d_p - 1) * pitch[c]));
        }
#pragma unroll
        for (int u = 0; u < EXP_U; ++u) {
            const int k = k0 + u * 512 + lane * 8;
            if (k >= K) continue;
            float xf[8];
            lds8(xs + k, xf);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                float f[8];
                widen8(v[r][u], f);
#pragma unroll
                for (int e = 0; e < 8; ++e) acc[r] = fmaf(f[e], xf[e], acc[r]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const float t = wave_sum(acc[r]);
        if (lane == r && row0 + r < d_p) y[row0 + r] = t;
    }
}

// ------------------------------------------------------------------ host side
int expert_row_values(const candy_hip_expert_spec &s) { return (int)(s.top * pad64(s.d_ff) + pad64(s.shared_ff)); }

// LDS of the one-row kernels
static size_t up_lds(const candy_hip_expert_spec &s, int64_t ld, size_t es) { return (size_t)ld * es + (size_t)(s.n_experts + 2 * s.top) * 4; }
static size_t down_lds(const candy_hip_expert_spec &s, size_t es) {
    const size_t K = (size_t)expert_row_values(s), chunks = K / 64;
    return chunks * 8 + ((chunks + 3) & ~(size_t)3) * 4 + K * es;
}
static size_t route_lds(const candy_hip_expert_spec &s) {
    return ((size_t)ROUTE_T * (s.n_experts | 1) + std::max<size_t>(ROUTE_W / 2 * 64 * 17, 2 * ROUTE_T * (size_t)s.top)) * 4;
}

int check_expert_spec(const candy_hip_expert_spec &s, int d) {
    CANDY_REQUIRE(s.n_experts > 0 && s.n_experts <= MAX_EXPERTS / 2 && s.top > 0 && s.top <= s.n_experts, "choice of %d out of %d experts unsupported",
                  s.top, s.n_experts);
    CANDY_REQUIRE(s.d_ff > 0 && s.shared_ff >= 0 && s.d_ff <= 1 << 20 && s.shared_ff <= 1 << 20, "invalid expert widths %d / %d", s.d_ff, s.shared_ff);
    // one workgroup keeps a row's activations in the 64 KB of LDS a launch gets without asking
    CANDY_REQUIRE(up_lds(s, pad64(d), 4) <= 65536 && (int64_t)s.top * pad64(s.d_ff) + pad64(s.shared_ff) <= 1 << 24 && down_lds(s, 2) <= 65536,
                  "%d experts of %d (+ %d) at width %d are too wide for one row's kernels", s.top, s.d_ff, s.shared_ff, d);
    CANDY_REQUIRE(route_lds(s) <= 65536, "too many experts (%d)", s.n_experts);
    return CANDY_HIP_OK;
}

static int deal_rows(const candy_hip_expert_spec &s, int n, bool f32) {
    return !f32 && (int64_t)n * s.top >= 96 * (int64_t)s.n_experts ? 128 : 64;
}
static int deal_max_tiles(const candy_hip_expert_spec &s, int n, int rows) {
    const int64_t count = (int64_t)n * s.top;
    // an expert with members has at most one tile that is not full
    return (int)(count / rows + std::min<int64_t>(s.n_experts, count));
}
static size_t deal_perm(const candy_hip_expert_spec &s, int n) { return ((size_t)n * s.top + 4 + 3) & ~(size_t)3; }
size_t expert_list_ints(const candy_hip_expert_spec &s, int n) { return deal_perm(s, n) + 4 * (size_t)deal_max_tiles(s, n, 64); }

int launch_experts_prompt(candy_hip_device *dev, const ExpertLayer &A, int n) {
    const candy_hip_expert_spec &s = A.s;
    const int rows = deal_rows(s, n, A.f32);
    hipLaunchKernelGGL(k_route, dim3((unsigned)((n + ROUTE_T - 1) / ROUTE_T)), dim3(64 * ROUTE_W), route_lds(s), dev->stream, A.x, A.ldx,
                       (const bf16 *)A.w.router->data, (int)A.w.router->ld, s.n_experts, s.top, n, A.ids, A.weights);
    CANDY_LAUNCH_CHECK();
    int *n_tiles = A.list, *perm = A.list + 4;
    GroupTile *tiles = (GroupTile *)(A.list + deal_perm(s, n));
    CANDY_REQUIRE((int64_t)n * s.top <= 0x7FFFFFFF / 2, "prompt too long for one pass");
    hipLaunchKernelGGL(k_deal, dim3(1), dim3(1024), 0, dev->stream, A.ids, n * s.top, s.n_experts, rows, perm, tiles, n_tiles);
    CANDY_LAUNCH_CHECK();
    GroupedRows gr;
    gr.perm = perm; gr.tiles = tiles; gr.n_tiles = n_tiles; gr.max_tiles = deal_max_tiles(s, n, rows); gr.tile_rows = rows;
    const int64_t ff = pad64(s.d_ff), d = pad64(A.d);
    DenseLaunch D;
    D.f32 = A.f32; D.m = n * s.top; D.group = &gr;
    gr.x_div = s.top; gr.expert_rows = (int)ff;
    D.w = A.w.up; D.x = A.x_act; D.ldx = A.ld_act; D.epi = CANDY_HIP_EPI_SQUARED_RELU; D.y = A.act; D.ldy = D.n_store = ff;
    if (int rc = launch_dense(dev, D)) return rc;
    gr.x_div = 1; gr.expert_rows = (int)d;
    D.w = A.w.down; D.x = A.act; D.ldx = ff; D.epi = CANDY_HIP_EPI_NONE; D.y = A.slots; D.ldy = D.n_store = d;
    if (int rc = launch_dense(dev, D)) return rc;
    if (!s.shared_ff) return CANDY_HIP_OK;
    DenseLaunch S;
    S.f32 = A.f32; S.m = n;
    S.w = A.w.shared_up; S.x = A.x_act; S.ldx = A.ld_act; S.epi = CANDY_HIP_EPI_SQUARED_RELU; S.y = A.shared_act;
    S.ldy = S.n_store = A.w.shared_up->rows_pad;
    if (int rc = launch_dense(dev, S)) return rc;
    S.w = A.w.shared_down; S.x = A.shared_act; S.ldx = A.w.shared_down->ld; S.epi = CANDY_HIP_EPI_NONE; S.y = A.y; S.ldy = A.ldy;
    S.n_store = A.w.shared_down->rows_pad; S.partial = A.shared;
    return launch_dense(dev, S);
}

template <class AT>
static int experts_row(candy_hip_device *dev, const ExpertLayer &A) {
    const candy_hip_expert_spec &s = A.s;
    const int64_t d = pad64(A.d);
    RowArgs u;
    u.E = s.n_experts; u.top = s.top; u.rows_e = (int)pad64(s.d_ff); u.rows_s = (int)pad64(s.shared_ff); u.ld = (int)d;
    u.W = (const bf16 *)A.w.up->data;
    u.shared = s.shared_ff ? (const bf16 *)A.w.shared_up->data : nullptr;
    const int total = expert_row_values(s);
    AT *act = (AT *)A.act;
    const MvShape su = mv_shape(dev, total), sd = mv_shape(dev, d);
    const dim3 gu((unsigned)((total + su.waves * su.rows - 1) / (su.waves * su.rows))), bu((unsigned)(64 * su.waves));
    const size_t lu = up_lds(s, d, sizeof(AT)), ldn = down_lds(s, sizeof(AT));
    CANDY_REQUIRE(lu <= 65536 && ldn <= 163840, "experts too wide for this activation format");
#define CANDY_UP(R)                                                                                                          \
    do {                                                                                                                     \
        if (s.n_experts <= 64) hipLaunchKernelGGL((k_expert_up<AT, R, true>), gu, bu, lu, dev->stream, u, A.x, A.logits, act, A.ids); \
        else hipLaunchKernelGGL((k_expert_up<AT, R, false>), gu, bu, lu, dev->stream, u, A.x, A.logits, act, A.ids);          \
    } while (0)
    switch (su.rows) {
    case 1: CANDY_UP(1); break;
    case 2: CANDY_UP(2); break;
    default: CANDY_UP(4); break;
    }
#undef CANDY_UP
    CANDY_LAUNCH_CHECK();
    u.W = (const bf16 *)A.w.down->data;
    u.shared = s.shared_ff ? (const bf16 *)A.w.shared_down->data : nullptr;
    const dim3 gd((unsigned)((d + sd.waves * sd.rows - 1) / (sd.waves * sd.rows))), bd((unsigned)(64 * sd.waves));
    switch (sd.rows) {
    case 1: hipLaunchKernelGGL((k_expert_down<AT, 1>), gd, bd, ldn, dev->stream, u, (int)d, act, A.ids, A.y); break;
    case 2: hipLaunchKernelGGL((k_expert_down<AT, 2>), gd, bd, ldn, dev->stream, u, (int)d, act, A.ids, A.y); break;
    default: hipLaunchKernelGGL((k_expert_down<AT, 4>), gd, bd, ldn, dev->stream, u, (int)d, act, A.ids, A.y); break;
    }
    CANDY_LAUNCH_CHECK();
    return CANDY_HIP_OK;
}
int launch_experts_row(candy_hip_device *dev, const ExpertLayer &A) {
    return A.f32 ? experts_row<float>(dev, A) : experts_row<bf16>(dev, A);
}

int check_expert_weights(const candy_hip_device *dev, const candy_hip_expert_spec &s, const candy_hip_expert_weights &w, int64_t d) {
    auto fits = [&](const candy_hip_dense *m, int64_t rows, int64_t cols) { return m && m->dev == dev && m->rows == rows && m->cols == cols; };
    CANDY_REQUIRE(fits(w.router, s.n_experts, d) && fits(w.up, s.n_experts * pad64(s.d_ff), d) &&
                      fits(w.down, s.n_experts * pad64(d), s.d_ff) &&
                      (s.shared_ff == 0 || (fits(w.shared_up, s.shared_ff, d) && fits(w.shared_down, d, s.shared_ff))),
                  "expert weights do not fit the spec");
    return CANDY_HIP_OK;
}

// sum of the slots and the shared row, for the entry point below
__global__ __launch_bounds__(256) void k_slot_sum(const float *slots, const float *weights, const Partial shared, int top, int d, int64_t ld,
                                                  float *out, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n * d) return;
    const int64_t t = i / d, c = i % d;
    float s = 0.0f;
    if (shared.p)
        for (int k = 0; k < shared.copies; ++k) s += shared.p[(size_t)k * shared.stride + t * shared.ld + c];
    for (int k = 0; k < top; ++k) s += weights[t * top + k] * slots[(t * top + k) * ld + c];
    out[i] = s;
}

}  // namespace candy

using namespace candy;

extern "C" int candy_hip_experts(candy_hip_device *dev, const candy_hip_expert_spec *spec, int act, const candy_hip_expert_weights *w,
                                 const float *x, int64_t n, int decode, float *out, int32_t *ids, float *weights) {
    CANDY_REQUIRE(dev && spec && w && w->router && x && out, "nil argument");
    const int64_t d = w->router->cols, ld = pad64(d);
    CANDY_REQUIRE(act == CANDY_HIP_ACT_BF16 || act == CANDY_HIP_ACT_F32, "unknown activation format %d", act);
    if (int rc = check_expert_spec(*spec, (int)d)) return rc;
    if (int rc = check_expert_weights(dev, *spec, *w, d)) return rc;
    CANDY_REQUIRE(n >= 1 && n <= 1 << 16 && (!decode || n == 1), "invalid number of rows %lld", (long long)n);
    if (int rc = use_device(dev)) return rc;
    const bool f32 = act == CANDY_HIP_ACT_F32;
    const size_t es = f32 ? 4 : 2, N = (size_t)n, slots = N * spec->top;
    auto al = [](size_t b) { return (b + 255) & ~(size_t)255; };
    size_t at = 0;
    auto take = [&](size_t bytes) { const size_t p = at; at += al(bytes); return p; };
    const size_t o_x = take(N * ld * 4), o_xa = take(N * ld * es), o_id = take(slots * 4), o_w = take(slots * 4),
                 o_act = take(std::max<size_t>(slots * pad64(spec->d_ff), expert_row_values(*spec)) * es),
                 o_sact = take(N * pad64(spec->shared_ff) * es + 4), o_list = take(expert_list_ints(*spec, (int)n) * 4),
                 o_slots = take(slots * ld * 4), o_y = take(N * ld * 4), o_lg = take(w->router->rows_pad * 4);
    void *ws = nullptr;
    if (int rc = workspace(dev, at, &ws)) return rc;
    uint8_t *b = (uint8_t *)ws;
    if (int rc = launch_to_act(dev, true, x, b + o_x, n, d, ld)) return rc;
    if (int rc = launch_to_act(dev, f32, x, b + o_xa, n, d, ld)) return rc;
    ExpertLayer A;
    Partial shared;
    A.s = *spec; A.w = *w; A.d = (int)d; A.f32 = f32;
    A.x = (const float *)(b + o_x); A.ldx = ld; A.x_act = b + o_xa; A.ld_act = ld;
    A.ids = (int *)(b + o_id); A.weights = (float *)(b + o_w); A.act = b + o_act; A.shared_act = b + o_sact; A.list = (int *)(b + o_list);
    A.slots = (float *)(b + o_slots); A.y = (float *)(b + o_y); A.ldy = ld; A.shared = &shared;
    if (decode) {
        CANDY_REQUIRE(!ids && !weights, "the decode kernels keep the weights to themselves");
        DenseLaunch D;
        D.w = w->router; D.x = A.x; D.ldx = ld; D.f32 = true; D.m = 1; D.y = b + o_lg; D.ldy = D.n_store = w->router->rows_pad;
        if (int rc = launch_dense(dev, D)) return rc;
        A.logits = (const float *)(b + o_lg);
        if (int rc = launch_experts_row(dev, A)) return rc;
        return candy_hip_d2d(dev, out, A.y, (size_t)d * 4);
    }
    if (int rc = launch_experts_prompt(dev, A, (int)n)) return rc;
    hipLaunchKernelGGL(k_slot_sum, dim3((unsigned)((n * d + 255) / 256)), dim3(256), 0, dev->stream, A.slots, A.weights, shared, spec->top, (int)d,
                       ld, out, n);
    CANDY_LAUNCH_CHECK();
    if (ids)
        if (int rc = candy_hip_d2d(dev, ids, A.ids, slots * 4)) return rc;
    return weights ? candy_hip_d2d(dev, weights, A.weights, slots * 4) : CANDY_HIP_OK;
}
