// Mixture of experts without a host round trip: router (fp32 logits, sigmoid or softmax scores, top-k), a one-workgroup
// sort of the (token, choice) pairs by expert into 32-row tiles, a grouped GEMM over those tiles on the matrix cores, and
// the combine that sums a token's rows (plus an optional gated shared expert).
//
//   route    logits = W_r h (fp32);  score = sigmoid(logit);  the k largest -> idx[T][k], weight[T][k]
//   align    pairs p = t * k + j sorted by expert; every expert's run padded to a multiple of the tile rows (32, long steps 128):
//            sorted[pos] = p or -1, tile_expert[pos / tile rows], pos_of_pair[p] = pos, n_tiles
//   gemm     out[pos][n] = sum_c A[row(pos)][c] * s(pos) * W[expert(pos)][n][c]        (s = 1 or the routing weight, applied
//            to the INPUT row and rounded to T like any other GEMM operand), optionally silu(gate) * up over a stacked
//            [gate | up] weight or the square of relu of a plain one
//   combine  y[t] = sum_j rows[pos_of_pair[t k + j]] * (w[t][j] or 1) + g[t] * shared[t]
//
// The number of tiles is data dependent; the grid is sized for the worst case (T k + E * (tile rows - 1) rows) and tiles past
// n_tiles leave at once.
#include <type_traits>
#include "common.h"
#include "mfma_frag.h"
#include "route_top.h"

namespace {

constexpr int TM = 32;        // rows per tile = one 32x32 MFMA block
constexpr int TM_LONG = 128;  // rows per tile of long steps (moe_gemm_tiled_kernel)

template <typename T> __device__ __forceinline__ float ldf(const T* p) { return (float)*p; }

// ---- router -----------------------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void moe_route_kernel(const T* __restrict__ h, int64_t ld_h, const float* __restrict__ wr,
                                                        const float* __restrict__ wg, int32_t* __restrict__ idx,
                                                        float* __restrict__ weight, float* __restrict__ shared_gate, int W, int E,
                                                        int k, const float* __restrict__ router_b, int softmax_top,
                                                        const float* __restrict__ correction, int n_groups, int keep_groups,
                                                        float renorm_eps) {
    extern __shared__ float sm[];
    float* hs = sm;          // [W]
    float* logit = sm + W;   // [E + 1]
    float* choice = logit + E + 1;  // [E] (softmax_top 2 only)
    const int64_t t = blockIdx.x;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = blockDim.x >> 6;
    for (int c = threadIdx.x; c < W; c += blockDim.x) hs[c] = ldf(h + t * ld_h + c);
    __syncthreads();
    const int rows = E + (wg ? 1 : 0);
    for (int e = wave; e < rows; e += nw) {
        const float* w = e < E ? wr + (int64_t)e * W : wg;
        float s = 0.f;
        if ((W & 3) == 0) {  // 16-byte loads, several in flight
#pragma unroll 4
            for (int c = lane * 4; c < W; c += 256) {
                const f32x4 wv = *reinterpret_cast<const f32x4*>(w + c);
                const f32x4 hv = *reinterpret_cast<const f32x4*>(hs + c);
                s += wv[0] * hv[0] + wv[1] * hv[1] + wv[2] * hv[2] + wv[3] * hv[3];
            }
        } else {
            for (int c = lane; c < W; c += 64) s += hs[c] * w[c];
        }
        s = wave_sum(s);
        if (lane == 0) logit[e] = s + ((router_b && e < E) ? router_b[e] : 0.f);
    }
    __syncthreads();
    if (softmax_top != 2 && k <= 64) {
        if (wave != 0) return;
        if (lane == 0 && wg) shared_gate[t] = 1.f / (1.f + expf(-logit[E]));
        route_top_wave(logit, E, k, softmax_top, idx + t * k, weight + t * k);
        return;
    }
    if (threadIdx.x == 0) {
        if (wg) shared_gate[t] = 1.f / (1.f + expf(-logit[E]));
        if (softmax_top == 2) {
            // scores = softmax over ALL experts; experts are chosen by score + correction among the keep_groups groups of
            // neighbours whose best choice score is largest (the others count as -inf); weights = the chosen scores / their sum
            float top = -INFINITY, sum = 0.f;
            for (int e = 0; e < E; ++e) top = fmaxf(top, logit[e]);
            for (int e = 0; e < E; ++e) sum += (logit[e] = expf(logit[e] - top));
            for (int e = 0; e < E; ++e) {
                logit[e] /= sum;
                choice[e] = logit[e] + (correction ? correction[e] : 0.f);
            }
            if (n_groups > 1 && keep_groups < n_groups) {
                const int per = E / n_groups;
                // a group is dropped when at least keep_groups others beat it (ties go to the lower index)
                for (int g = 0; g < n_groups; ++g) {
                    float best = -INFINITY;
                    for (int e = g * per; e < (g + 1) * per; ++e) best = fmaxf(best, choice[e]);
                    hs[g] = best;  // the row is no longer needed
                }
                for (int g = 0; g < n_groups; ++g) {
                    int ahead = 0;
                    for (int o = 0; o < n_groups; ++o) ahead += (hs[o] > hs[g] || (hs[o] == hs[g] && o < g)) ? 1 : 0;
                    if (ahead >= keep_groups)
                        for (int e = g * per; e < (g + 1) * per; ++e) choice[e] = -INFINITY;
                }
            }
            float wsum = 0.f;
            for (int j = 0; j < k; ++j) {
                int best = -1;
                float bv = -INFINITY;
                for (int e = 0; e < E; ++e)
                    if (choice[e] > bv) {
                        bv = choice[e];
                        best = e;
                    }
                if (best < 0) {  // fewer allowed experts than k, or NaN scores: the first index not taken yet
                    best = 0;
                    for (int e = E - 1; e >= 0; --e) {
                        bool taken = false;
                        for (int i = 0; i < j; ++i) taken |= idx[t * k + i] == e;
                        if (!taken) best = e;
                    }
                }
                idx[t * k + j] = best;
                weight[t * k + j] = logit[best];
                wsum += logit[best];
                choice[best] = -INFINITY;
            }
            for (int j = 0; j < k; ++j) weight[t * k + j] /= (wsum + renorm_eps);
            return;
        }
        // k passes of selection; ties go to the lower index
        for (int j = 0; j < k; ++j) {
            int best = -1;
            float bv = -INFINITY;
            for (int e = 0; e < E; ++e) {
                const float v = logit[e];
                if (v > bv) {
                    bv = v;
                    best = e;
                }
            }
            if (best < 0) best = 0;  // NaN logits: still a valid index
            idx[t * k + j] = best;
            // softmax_top: the chosen logits are softmaxed among themselves below (the first one is the largest)
            weight[t * k + j] = softmax_top ? bv : 1.f / (1.f + expf(-bv));
            logit[best] = -INFINITY;
        }
        if (softmax_top) {
            const float top = weight[t * k];
            float sum = 0.f;
            for (int j = 0; j < k; ++j) sum += expf(weight[t * k + j] - top);
            for (int j = 0; j < k; ++j) weight[t * k + j] = expf(weight[t * k + j] - top) / sum;
        }
    }
}

// Choice among logits that are there already (tgis_narrow_product): a wave per token, four tokens per workgroup.
__global__ __launch_bounds__(256) void moe_choose_kernel(const float* __restrict__ logits, int64_t rows, int E, int k, int groups, int keep,
                                                         float scale, int32_t* __restrict__ idx, float* __restrict__ weight) {
    extern __shared__ float sm[];  // [4][E + groups]
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int64_t t = (int64_t)blockIdx.x * 4 + wave;
    if (t >= rows) return;  // the whole wave; no workgroup barrier follows
    float* mine = sm + wave * (E + groups);
    for (int e = lane; e < E; e += 64) mine[e] = logits[t * E + e];
    route_grouped_sigmoid_wave(mine, mine + E, E, k, groups, keep, scale, idx + t * k, weight + t * k);
}

// ---- align: one workgroup ---------------------------------------------------------------------------------------------
__global__ __launch_bounds__(1024) void moe_align_kernel(const int32_t* __restrict__ idx, int64_t n_pairs, int E,
                                                         int32_t* __restrict__ sorted, int64_t cap, int32_t* __restrict__ tile_expert,
                                                         int32_t* __restrict__ pos_of_pair, int32_t* __restrict__ n_tiles, int tm) {
    extern __shared__ int32_t si[];
    int32_t* count = si;            // [E]
    int32_t* start = si + E;        // [E + 1]
    int32_t* cursor = si + 2 * E + 1;  // [E]
    for (int e = threadIdx.x; e < E; e += blockDim.x) count[e] = cursor[e] = 0;
    for (int64_t i = threadIdx.x; i < cap; i += blockDim.x) sorted[i] = -1;
    __syncthreads();
    for (int64_t p = threadIdx.x; p < n_pairs; p += blockDim.x) atomicAdd(&count[idx[p]], 1);
    __syncthreads();
    if (threadIdx.x == 0) {
        int32_t at = 0;
        for (int e = 0; e < E; ++e) {
            start[e] = at;
            at += (count[e] + tm - 1) / tm * tm;
        }
        start[E] = at;
        *n_tiles = at / tm;
    }
    __syncthreads();
    for (int e = threadIdx.x; e < E; e += blockDim.x)
        for (int32_t tl = start[e] / tm; tl < start[e + 1] / tm; ++tl) tile_expert[tl] = e;
    // arrival order within an expert: the rows of a tile are independent of each other, so the order changes no result
    for (int64_t p = threadIdx.x; p < n_pairs; p += blockDim.x) {
        const int e = idx[p];
        const int32_t pos = start[e] + atomicAdd(&cursor[e], 1);
        sorted[pos] = (int32_t)p;
        pos_of_pair[p] = pos;
    }
}

// ---- grouped GEMM -----------------------------------------------------------------------------------------------------
// Workgroup = 4 waves = one 32-row tile x 128 output columns; a wave owns 32 columns (GLU: 32 gate + the 32 matching up
// columns).  Operands come straight from global memory / L2 in MFMA fragment order: lane l holds row (l % 32) and 8 (bf16)
// or 4 (fp32) consecutive k at offset (l / 32) * that — a 16-byte load for A and for B.
//
// Weights come as an IMAGE in that order: per expert [block of 32 weight rows][step of 16 (fp32: 8) k][lane][8 (4) elements], rows
// and k padded with zeros, GLU: the gate rows' blocks, then the up rows' — a step of a block is 1 KiB in one piece, so a decode
// step streams an expert's weights in whole lines.
//
// Two shapes of workgroup:
//   many tiles (prompts): wave w owns row tile 4 y + w and 64 output columns (GLU: 64 gate + the 64 matching up columns).  The
//     four waves walk the same weight rows at the same time, so an expert's weights come from L2 once per four row tiles
//     instead of once per tile, and a wave's A fragment feeds two (GLU: four) products;
//   few tiles (decode, KW > 1): KW waves split K for ONE 32-row x 32-column block and meet in LDS, so that a launch with a
//     handful of tiles still has enough waves in flight to stream the expert weights.
//
// GLU 1: silu(gate) * up.  GLU 2 (clamped unit): g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(alpha g) (u + 1).
template <int GLU> __device__ __forceinline__ float gated(float g, float u, float alpha, float limit) {
    if (GLU == 1) return g / (1.f + expf(-g)) * u;
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return g / (1.f + expf(-alpha * g)) * (u + 1.f);
}

// what a plain product (GLU 0) becomes where it is written: act 1 the square of relu
__device__ __forceinline__ float plain_out(float v, int act) {
    const float p = fmaxf(v, 0.f);
    return act ? p * p : v;
}

template <typename T> __device__ __forceinline__ int64_t image_block(int64_t K) {  // elements of a block of 32 weight rows
    return (K + Frag<T>::KSTEP - 1) / Frag<T>::KSTEP * (64 * Frag<T>::PER);
}

template <typename T, int GLU, int KW>
__global__ __launch_bounds__(KW > 4 ? 512 : 256) void moe_gemm_kernel(const T* __restrict__ A, int64_t ld_a, const int32_t* __restrict__ sorted,
                                                       int pair_div, const float* __restrict__ pair_scale,
                                                       const int32_t* __restrict__ tile_expert, const int32_t* __restrict__ n_tiles,
                                                       const T* __restrict__ Wt, int64_t N, int64_t K,
                                                       T* __restrict__ out, int64_t ld_out, float alpha, float limit, int act) {
    constexpr bool KSPLIT = KW > 1;
    using F = Frag<T>;
    using V = typename F::V;
    constexpr int NB = KSPLIT ? 1 : 2;  // 32-column blocks per wave
    __shared__ float part[KSPLIT ? KW * (GLU ? 2 : 1) * 16 * 64 : 1];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int tile = KSPLIT ? blockIdx.y : blockIdx.y * 4 + wave;
    if (tile >= *n_tiles) return;  // KSPLIT: the whole workgroup
    const int row = lane & 31, half = lane >> 5;
    const int64_t n0 = (int64_t)blockIdx.x * 32 * NB;
    const int64_t pos = (int64_t)tile * TM + row;
    const int64_t block = image_block<T>(K), nblocks = (N + 31) >> 5;
    const T* W = Wt + (int64_t)tile_expert[tile] * nblocks * (GLU ? 2 : 1) * block;
    // A row of this lane
    int64_t arow = pos;
    float scale = 1.f;
    bool live = true;
    if (sorted) {
        const int32_t p = sorted[pos];
        live = p >= 0;
        if (pair_div > 0) arow = live ? p / pair_div : 0;
        if (pair_scale) scale = live ? pair_scale[p] : 0.f;
    }
    const T* ap = A + arow * ld_a + half * F::PER;
    const T* bp[NB];
    const T* bp2[NB];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
        const int64_t nblk = min((n0 >> 5) + nb, nblocks - 1);  // clamped: a block past the last is computed and dropped
        bp[nb] = W + nblk * block + lane * F::PER;
        bp2[nb] = GLU ? W + (nblocks + nblk) * block + lane * F::PER : nullptr;
    }
    f32x16 acc[NB], acc2[NB];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) acc[nb] = acc2[nb] = f32x16{};
    // this wave's k range, in whole steps
    const int64_t steps = (K + F::KSTEP - 1) / F::KSTEP;
    const int64_t s0 = KSPLIT ? steps * wave / KW : 0, s1 = KSPLIT ? steps * (wave + 1) / KW : steps;
    // U steps' fragments are asked for before the first product of them: a wave streams several KiB of weights at a time
    constexpr int U = KSPLIT ? 4 : 2;
    auto steps_of = [&](auto count, int64_t st) {
        constexpr int N_ = decltype(count)::value;
        V a[N_], bw[N_][NB], bw2[N_][NB];
#pragma unroll
        for (int u = 0; u < N_; ++u) {
            const int64_t kk = (st + u) * F::KSTEP;
            // K is a multiple of PER: a fragment is whole or absent.  Padding rows are not fetched: a decode step has a few live rows
            // per tile, and their lines are as many as the weights' otherwise
            const bool in = live && kk + half * F::PER + F::PER <= K;
            a[u] = in ? *reinterpret_cast<const V*>(ap + kk) : F::zero();
#pragma unroll
            for (int nb = 0; nb < NB; ++nb) {
                bw[u][nb] = *reinterpret_cast<const V*>(bp[nb] + (st + u) * (64 * F::PER));
                if (GLU) bw2[u][nb] = *reinterpret_cast<const V*>(bp2[nb] + (st + u) * (64 * F::PER));
            }
        }
#pragma unroll
        for (int u = 0; u < N_; ++u) {
            if (pair_scale) a[u] = F::scaled(a[u], scale);
#pragma unroll
            for (int nb = 0; nb < NB; ++nb) {
                F::mma(a[u], bw[u][nb], acc[nb]);
                if (GLU) F::mma(a[u], bw2[u][nb], acc2[nb]);
            }
        }
    };
    int64_t st = s0;
    for (; st + U <= s1; st += U) steps_of(std::integral_constant<int, U>{}, st);
    if (U >= 4 && st + 2 <= s1) {
        steps_of(std::integral_constant<int, 2>{}, st);
        st += 2;
    }
    if (st < s1) steps_of(std::integral_constant<int, 1>{}, st);
    // accumulator i of lane l: A row (i / 4) * 8 + (l / 32) * 4 + i % 4, B row (= output column) l % 32
    if (KSPLIT) {
        constexpr int NA = GLU ? 2 : 1;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            part[((wave * NA + 0) * 16 + i) * 64 + lane] = acc[0][i];
            if (GLU) part[((wave * NA + 1) * 16 + i) * 64 + lane] = acc2[0][i];
        }
        __syncthreads();
        if (n0 + row >= N) return;
        // wave w finishes accumulators 16 / KW * w and on
#pragma unroll
        for (int q = 0; q < 16 / KW; ++q) {
            const int i = wave * (16 / KW) + q;
            float v = 0.f, v2 = 0.f;
#pragma unroll
            for (int w = 0; w < KW; ++w) {
                v += part[((w * NA + 0) * 16 + i) * 64 + lane];
                if (GLU) v2 += part[((w * NA + 1) * 16 + i) * 64 + lane];
            }
            v = GLU ? gated<GLU>(v, v2, alpha, limit) : plain_out(v, act);
            const int m = (i >> 2) * 8 + half * 4 + (i & 3);
            out[((int64_t)tile * TM + m) * ld_out + n0 + row] = (T)v;
        }
        return;
    }
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
        const int64_t n = n0 + nb * 32 + row;
        if (n < N) {
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const int m = (i >> 2) * 8 + half * 4 + (i & 3);
                float v = acc[nb][i];
                v = GLU ? gated<GLU>(v, acc2[nb][i], alpha, limit) : plain_out(v, act);
                out[((int64_t)tile * TM + m) * ld_out + n] = (T)v;
            }
        }
    }
}

// ---- grouped GEMM of long steps -----------------------------------------------------------------------------------------
// Workgroup = 4 waves (2 x 2) = one 128-row tile x BN weight rows (GLU: BN / 2 gate rows and the matching up rows); a wave owns
// 64 rows x BN / 2 weight rows: 2 x BN / 64 accumulators of 32x32.  Both operands go through LDS in slices of 32 k, two slices
// deep: the next slice is on its way to registers while the matrix cores work on the current one, one barrier per slice.  A slice
// row is four 16-byte pieces, stored at piece ^ swz(row) so that the fragment reads of neighbouring rows fall on different banks.
// Workgroups are dealt so that an XCD (one in eight workgroup ids) works on eight row tiles x a run of column blocks at a time:
// what they read again is in its own L2.
template <typename T, int GLU, int BN>
__global__ __launch_bounds__(256, 2) void moe_gemm_tiled_kernel(const T* __restrict__ A, int64_t ld_a, const int32_t* __restrict__ sorted,
                                                                int pair_div, const float* __restrict__ pair_scale,
                                                                const int32_t* __restrict__ tile_expert, const int32_t* __restrict__ n_tiles,
                                                                const T* __restrict__ Wt, int64_t N, int64_t K,
                                                                T* __restrict__ out, int64_t ld_out, float alpha, float limit, int ncb, int act) {
    using V = typename Frag<T>::V;
    constexpr int BK = 32, AL = TM_LONG * 4 / 256, BL = BN * 4 / 256, NJ = BN / 64;
    constexpr int HALF = BN / 2;                      // weight rows of a wave
    constexpr int OUTC = GLU ? BN / 2 : BN;           // output columns of the workgroup
    __shared__ __attribute__((aligned(16))) T as[2][TM_LONG * BK];
    __shared__ __attribute__((aligned(16))) T bs[2][BN * BK];
    const int total = *n_tiles * ncb;
    const int chunk = (total + 7) >> 3;
    const int lin = (int)(blockIdx.x & 7) * chunk + (int)(blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= chunk || lin >= total) return;  // the whole workgroup
    // groups of eight row tiles; inside a group the row tile moves fastest
    const int group = lin / (8 * ncb), in_group = lin - group * 8 * ncb;
    const int rows_here = min(8, *n_tiles - group * 8);
    const int tile = group * 8 + in_group % rows_here, cb = in_group / rows_here;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
    const int wr = wave >> 1, wc = wave & 1, r = lane & 31, half = lane >> 5;
    const int64_t block = image_block<T>(K), nblocks = (N + 31) >> 5;
    const T* W = Wt + (int64_t)tile_expert[tile] * nblocks * (GLU ? 2 : 1) * block;
    const int64_t n0 = (int64_t)cb * OUTC;
    auto swz = [](int row) { return ((row >> 1) ^ (row >> 3)) & 3; };
    const T* ap[AL];
    float asc[AL];
    int aoff[AL];
#pragma unroll
    for (int i = 0; i < AL; ++i) {
        const int e = tid + i * 256, row = e >> 2, piece = e & 3;
        const int64_t pos = (int64_t)tile * TM_LONG + row;
        int64_t arow = pos;
        asc[i] = 1.f;
        if (sorted) {
            const int32_t p = sorted[pos];
            if (pair_div > 0) arow = p >= 0 ? p / pair_div : 0;
            if (pair_scale) asc[i] = p >= 0 ? pair_scale[p] : 0.f;
        }
        ap[i] = A + arow * ld_a + piece * 8;
        aoff[i] = row * BK + ((piece ^ swz(row)) * 8);
    }
    const T* bp[BL];
    int boff[BL];
#pragma unroll
    for (int i = 0; i < BL; ++i) {
        // the image's order: 32 rows of one piece lie side by side
        const int e = tid + i * 256, rb = e >> 7, piece = (e >> 5) & 3, row = rb * 32 + (e & 31);
        int64_t nblk;
        if (GLU) {  // a wave's blocks: HALF / 64 of gate rows, then the matching up rows'
            constexpr int PB = HALF / 32;
            const int w = rb / PB, x = rb % PB;
            nblk = (n0 >> 5) + w * (PB / 2) + x % (PB / 2);
            nblk = min(nblk, nblocks - 1) + (x >= PB / 2 ? nblocks : 0);
        } else {
            nblk = min((n0 >> 5) + rb, nblocks - 1);  // clamped: a block past the last is computed and dropped
        }
        bp[i] = W + nblk * block + ((piece >> 1) * 64 + (piece & 1) * 32 + (e & 31)) * 8;
        boff[i] = row * BK + ((piece ^ swz(row)) * 8);
    }
    f32x16 acc[2][NJ];
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < NJ; ++j) acc[i][j] = f32x16{};
    V ar[AL], br[BL];
    auto fetch = [&](int64_t k) {
#pragma unroll
        for (int i = 0; i < AL; ++i) ar[i] = *reinterpret_cast<const V*>(ap[i] + k);
#pragma unroll
        for (int i = 0; i < BL; ++i) br[i] = *reinterpret_cast<const V*>(bp[i] + k * 32);  // two steps of 512 elements per slice
    };
    auto store = [&](int buf) {
#pragma unroll
        for (int i = 0; i < AL; ++i) *reinterpret_cast<V*>(&as[buf][aoff[i]]) = pair_scale ? Frag<T>::scaled(ar[i], asc[i]) : ar[i];
#pragma unroll
        for (int i = 0; i < BL; ++i) *reinterpret_cast<V*>(&bs[buf][boff[i]]) = br[i];
    };
    fetch(0);
    store(0);
    __syncthreads();
    int buf = 0;
    for (int64_t k = 0; k < K; k += BK, buf ^= 1) {
        const bool more = k + BK < K;
        if (more) fetch(k + BK);
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            V a[2], b[NJ];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                const int row = wr * 64 + i * 32 + r;
                a[i] = *reinterpret_cast<const V*>(&as[buf][row * BK + (((s * 2 + half) ^ swz(row)) * 8)]);
            }
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                const int row = wc * HALF + j * 32 + r;
                b[j] = *reinterpret_cast<const V*>(&bs[buf][row * BK + (((s * 2 + half) ^ swz(row)) * 8)]);
            }
#pragma unroll
            for (int i = 0; i < 2; ++i)
#pragma unroll
                for (int j = 0; j < NJ; ++j) Frag<T>::mma(a[i], b[j], acc[i][j]);
        }
        if (more) store(buf ^ 1);  // its last readers passed the barrier at the end of the slice before
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < (GLU ? NJ / 2 : NJ); ++j) {
            const int64_t n = n0 + (GLU ? wc * (HALF / 2) : wc * HALF) + j * 32 + r;
            if (n >= N) continue;
#pragma unroll
            for (int q = 0; q < 16; ++q) {
                const int64_t row = (int64_t)tile * TM_LONG + wr * 64 + i * 32 + (q >> 2) * 8 + half * 4 + (q & 3);
                float v = acc[i][j][q];
                v = GLU ? gated<GLU ? GLU : 1>(v, acc[i][GLU ? j + NJ / 2 : j][q], alpha, limit) : plain_out(v, act);
                out[row * ld_out + n] = (T)v;
            }
        }
}

template <typename T>
void launch_gemm_tiled(int glu, int act, float alpha, float limit, const void* A, int64_t ld_a, const int32_t* sorted, int pair_div,
                       const float* pair_scale, const int32_t* tile_expert, const int32_t* n_tiles, const void* Wt,
                       int64_t N, int64_t K, void* out, int64_t ld_out, int64_t max_tiles, hipStream_t st) {
#define TGIS_MOE_TILED(GLU, BN)                                                                                                        \
    do {                                                                                                                               \
        const int ncb = (int)cdiv64(N, GLU ? BN / 2 : BN);                                                                             \
        hipLaunchKernelGGL((moe_gemm_tiled_kernel<T, GLU, BN>), dim3((unsigned)((max_tiles * ncb + 7) / 8 * 8)), dim3(256), 0, st,     \
                           (const T*)A, ld_a, sorted, pair_div, pair_scale, tile_expert, n_tiles, (const T*)Wt, N, K,   \
                           (T*)out, ld_out, alpha, limit, ncb, act);                                                                   \
    } while (0)
    if (glu == 2)
        TGIS_MOE_TILED(2, 256);
    else if (glu)
        TGIS_MOE_TILED(1, 256);
    else
        TGIS_MOE_TILED(0, 256);
#undef TGIS_MOE_TILED
}

// ---- combine: one workgroup per token -----------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void moe_combine_kernel(const T* __restrict__ rows, int64_t ld_rows, const int32_t* __restrict__ pos_of_pair,
                                                          const float* __restrict__ pair_weight, int k, const T* __restrict__ shared,
                                                          int64_t ld_shared, const float* __restrict__ shared_gate, T* __restrict__ out,
                                                          int64_t ld_out, int64_t W) {
    const int64_t t = blockIdx.x;
    const float g = shared ? (shared_gate ? shared_gate[t] : 1.f) : 0.f;
    const int64_t c = (int64_t)blockIdx.y * blockDim.x + threadIdx.x;  // grid (token, 256-column block)
    if (c >= W) return;
    float s = 0.f;
    for (int j = 0; j < k; ++j) {
        const float w = pair_weight ? pair_weight[t * k + j] : 1.f;
        s += w * ldf(rows + (int64_t)pos_of_pair[t * k + j] * ld_rows + c);
    }
    if (shared) s += g * ldf(shared + t * ld_shared + c);
    out[t * ld_out + c] = (T)s;
}

template <typename T>
void launch_gemm(int glu, int act, float alpha, float limit, const void* A, int64_t ld_a, const int32_t* sorted, int pair_div, const float* pair_scale,
                 const int32_t* tile_expert, const int32_t* n_tiles, const void* Wt, int64_t N, int64_t K,
                 void* out, int64_t ld_out, int64_t max_tiles, hipStream_t st) {
    const bool ksplit = max_tiles * cdiv64(N, 128) < 1024;
    // few blocks (narrow experts): eight waves per block, or the launch is over before the memory system is busy
    const bool deep = ksplit && max_tiles * cdiv64(N, 32) < 1024 && K >= 1024;
    dim3 grid((unsigned)(ksplit ? cdiv64(N, 32) : cdiv64(N, 64)), (unsigned)(ksplit ? max_tiles : cdiv64(max_tiles, 4)));
#define TGIS_MOE_LAUNCH(GLU, KW)                                                                                                       \
    hipLaunchKernelGGL((moe_gemm_kernel<T, GLU, KW>), grid, dim3(KW > 4 ? 512 : 256), 0, st, (const T*)A, ld_a, sorted, pair_div, pair_scale, \
                       tile_expert, n_tiles, (const T*)Wt, N, K, (T*)out, ld_out, alpha, limit, act)
#define TGIS_MOE_GLU(KW)                     \
    do {                                     \
        if (glu == 2)                        \
            TGIS_MOE_LAUNCH(2, KW);          \
        else if (glu)                        \
            TGIS_MOE_LAUNCH(1, KW);          \
        else                                 \
            TGIS_MOE_LAUNCH(0, KW);          \
    } while (0)
    if (deep)
        TGIS_MOE_GLU(8);
    else if (ksplit)
        TGIS_MOE_GLU(4);
    else
        TGIS_MOE_GLU(1);
#undef TGIS_MOE_GLU
#undef TGIS_MOE_LAUNCH
}

}  // namespace

static bool dtype3(int d) { return d == TGIS_F16 || d == TGIS_BF16 || d == TGIS_F32; }

static int64_t row_capacity(int64_t n_pairs, int64_t E, int64_t tm) { return (n_pairs + E * (tm - 1) + tm - 1) / tm * tm; }
extern "C" int64_t tgis_moe_row_capacity(int64_t n_pairs, int64_t E, int tile_rows) { return row_capacity(n_pairs, E, tile_rows); }

// Rows per tile a mixture of n_pairs (token, choice) pairs over E experts should be aligned to: 128 where the experts' runs are long
// enough to fill such tiles and both products' inner widths fit the LDS-staged kernel (two-byte dtypes, multiples of 32), else 32.
extern "C" int tgis_moe_tile_rows(int64_t n_pairs, int64_t E, int64_t W, int64_t ff, int dtype) {
    return dtype != TGIS_F32 && n_pairs >= 96 * E && W % 32 == 0 && ff % 32 == 0 ? TM_LONG : TM;
}

static int moe_route_impl(const void* h, int64_t ld_h, const float* router_w, const float* shared_gate_w, int32_t* idx,
                          float* weight, float* shared_gate, int64_t T, int64_t W, int E, int k, int dtype, void* stream,
                          const float* router_b, int softmax_top, const float* correction = nullptr, int n_groups = 1,
                          int keep_groups = 1, float renorm_eps = 0.f) {
    TGIS_CHECK_ARG(h && router_w && idx && weight && (!shared_gate_w || shared_gate), "tgis_moe_route: null tensor");
    TGIS_CHECK_ARG(n_groups >= 1 && keep_groups >= 1 && keep_groups <= n_groups && E % n_groups == 0 && n_groups <= W,
                   "tgis_moe_route: %d experts do not form %d equal groups", E, n_groups);
    TGIS_CHECK_ARG(E >= 1 && k >= 1 && k <= E && W >= 1 && ld_h >= W && dtype3(dtype), "tgis_moe_route: bad arguments");
    const size_t lds = ((size_t)W + 2 * E + 1) * sizeof(float);
    TGIS_CHECK_ARG(lds <= 64 * 1024, "tgis_moe_route: width + experts need %ld bytes of LDS", (long)lds);
    if (T == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    if (dtype == TGIS_F16)
        hipLaunchKernelGGL(moe_route_kernel<f16>, dim3((unsigned)T), dim3(256), lds, st, (const f16*)h, ld_h, router_w, shared_gate_w, idx, weight, shared_gate, (int)W, E, k, router_b, softmax_top, correction, n_groups, keep_groups, renorm_eps);
    else if (dtype == TGIS_BF16)
        hipLaunchKernelGGL(moe_route_kernel<bf16>, dim3((unsigned)T), dim3(256), lds, st, (const bf16*)h, ld_h, router_w, shared_gate_w, idx, weight, shared_gate, (int)W, E, k, router_b, softmax_top, correction, n_groups, keep_groups, renorm_eps);
    else
        hipLaunchKernelGGL(moe_route_kernel<float>, dim3((unsigned)T), dim3(256), lds, st, (const float*)h, ld_h, router_w, shared_gate_w, idx, weight, shared_gate, (int)W, E, k, router_b, softmax_top, correction, n_groups, keep_groups, renorm_eps);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}

extern "C" int tgis_moe_route(const void* h, int64_t ld_h, const float* router_w, const float* shared_gate_w, int32_t* idx,
                              float* weight, float* shared_gate, int64_t T, int64_t W, int E, int k, int dtype, void* stream) {
    return moe_route_impl(h, ld_h, router_w, shared_gate_w, idx, weight, shared_gate, T, W, E, k, dtype, stream, nullptr, 0);
}

// The same with a bias on the router logits (router_b [E] fp32 or NULL) and a choice of weights: softmax_top 0: the sigmoid of
// each chosen logit; 1: the softmax over the chosen logits only.
extern "C" int tgis_moe_route_ext(const void* h, int64_t ld_h, const float* router_w, const float* router_b, const float* shared_gate_w,
                                  int softmax_top, int32_t* idx, float* weight, float* shared_gate, int64_t T, int64_t W, int E, int k,
                                  int dtype, void* stream) {
    return moe_route_impl(h, ld_h, router_w, shared_gate_w, idx, weight, shared_gate, T, W, E, k, dtype, stream, router_b, softmax_top ? 1 : 0);
}

// Softmax scores over all experts; choice by score + correction [E] (fp32 or NULL) among the keep_groups best of n_groups equal
// groups of neighbouring experts (a group's rank is its largest choice score); weights = chosen scores / (their sum + renorm_eps).
extern "C" int tgis_moe_route_grouped(const void* h, int64_t ld_h, const float* router_w, const float* correction, int n_groups,
                                      int keep_groups, float renorm_eps, int32_t* idx, float* weight, int64_t T, int64_t W, int E, int k,
                                      int dtype, void* stream) {
    return moe_route_impl(h, ld_h, router_w, nullptr, idx, weight, nullptr, T, W, E, k, dtype, stream, nullptr, 2, correction, n_groups,
                          keep_groups, renorm_eps);
}

// The choice alone, from logits [T][E] fp32: scores are their sigmoids; experts come from the `keep` best of `groups` equal groups of
// neighbours (a group counts by the sum of its two largest scores); weights = chosen scores * scale.
extern "C" int tgis_moe_choose(const float* logits, int64_t T, int E, int k, int groups, int keep, float scale, int32_t* idx, float* weight,
                               void* stream) {
    TGIS_CHECK_ARG(logits && idx && weight && E >= 1 && E <= 2048 && k >= 1 && k <= 64 && groups >= 1 && E % groups == 0 && keep >= 1 && keep <= groups &&
                       (int64_t)keep * (E / groups) >= k,
                   "tgis_moe_choose: cannot choose %d of %d experts in the best %d of %d groups", k, E, keep, groups);
    if (T == 0) return TGIS_OK;
    hipLaunchKernelGGL(moe_choose_kernel, dim3((unsigned)cdiv64(T, 4)), dim3(256), (size_t)4 * (E + groups) * sizeof(float), (hipStream_t)stream, logits,
                       T, E, k, groups, keep, scale, idx, weight);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}

extern "C" int tgis_moe_align(const int32_t* idx, int64_t n_pairs, int E, int32_t* sorted, int64_t capacity, int32_t* tile_expert,
                              int32_t* pos_of_pair, int32_t* n_tiles, int tile_rows, void* stream) {
    TGIS_CHECK_ARG(idx && sorted && tile_expert && pos_of_pair && n_tiles, "tgis_moe_align: null tensor");
    TGIS_CHECK_ARG(tile_rows == TM || tile_rows == TM_LONG, "tgis_moe_align: tiles of %d or %d rows", TM, TM_LONG);
    TGIS_CHECK_ARG(E >= 1 && E <= 4096 && n_pairs >= 0 && capacity >= row_capacity(n_pairs, E, tile_rows) && capacity % tile_rows == 0,
                   "tgis_moe_align: capacity %ld below tgis_moe_row_capacity", (long)capacity);
    const int threads = n_pairs <= 1024 && capacity <= 4096 ? 256 : 1024;  // decode: barriers of four waves instead of sixteen
    hipLaunchKernelGGL(moe_align_kernel, dim3(1), dim3(threads), (size_t)(3 * E + 1) * sizeof(int32_t), (hipStream_t)stream, idx, n_pairs,
                       E, sorted, capacity, tile_expert, pos_of_pair, n_tiles, tile_rows);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}

extern "C" int tgis_moe_gemm(const void* A, int64_t ld_a, const int32_t* sorted, int pair_div, const float* pair_scale,
                             const int32_t* tile_expert, const int32_t* n_tiles, const void* image, int64_t N, int64_t K, int glu,
                             float alpha, float limit, void* out, int64_t ld_out, int64_t capacity, int tile_rows, int dtype, void* stream) {
    TGIS_CHECK_ARG(A && tile_expert && n_tiles && image && out, "tgis_moe_gemm: null tensor");
    TGIS_CHECK_ARG(dtype3(dtype) && glu >= 0 && glu <= 3, "tgis_moe_gemm: bad dtype or glu");
    const int act = glu == 3 ? 1 : 0;  // a plain weight whose product is squared where it is positive
    if (act) glu = 0;
    const int per = dtype == TGIS_F32 ? 4 : 8;
    TGIS_CHECK_ARG(N >= 1 && K >= per && K % per == 0 && ld_a % per == 0 && ld_a >= K && ld_out >= N,
                   "tgis_moe_gemm: K (%ld) and the A row stride (%ld) must be multiples of %d", (long)K, (long)ld_a, per);
    TGIS_CHECK_ARG((((uintptr_t)A) & 15) == 0 && (((uintptr_t)image) & 15) == 0, "tgis_moe_gemm: operands must be 16-byte aligned");
    TGIS_CHECK_ARG(!sorted || pair_div >= 0, "tgis_moe_gemm: gathered rows need pair_div >= 1, rows in place pair_div 0");
    TGIS_CHECK_ARG(!pair_scale || sorted, "tgis_moe_gemm: a per-pair scale needs the sorted pair list");
    TGIS_CHECK_ARG((tile_rows == TM || tile_rows == TM_LONG) && capacity % tile_rows == 0, "tgis_moe_gemm: tiles of %d or %d rows", TM, TM_LONG);
    if (capacity == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_MOE_GEMM, st);
    const int64_t tiles = capacity / tile_rows;
    if (tile_rows == TM_LONG) {
        TGIS_CHECK_ARG(dtype != TGIS_F32 && K % 32 == 0 && tiles * cdiv64(N, 128) < (1ll << 30),
                       "tgis_moe_gemm: 128-row tiles take two-byte dtypes and K a multiple of 32 (got %ld)", (long)K);
        if (dtype == TGIS_F16)
            launch_gemm_tiled<f16>(glu, act, alpha, limit, A, ld_a, sorted, pair_div, pair_scale, tile_expert, n_tiles, image, N, K, out, ld_out, tiles, st);
        else
            launch_gemm_tiled<bf16>(glu, act, alpha, limit, A, ld_a, sorted, pair_div, pair_scale, tile_expert, n_tiles, image, N, K, out, ld_out, tiles, st);
        TGIS_CHECK_LAUNCH();
        return TGIS_OK;
    }
    TGIS_CHECK_ARG(tiles <= 65535, "tgis_moe_gemm: %ld tiles exceed one grid", (long)tiles);
    if (dtype == TGIS_F16)
        launch_gemm<f16>(glu, act, alpha, limit, A, ld_a, sorted, pair_div, pair_scale, tile_expert, n_tiles, image, N, K, out, ld_out, tiles, st);
    else if (dtype == TGIS_BF16)
        launch_gemm<bf16>(glu, act, alpha, limit, A, ld_a, sorted, pair_div, pair_scale, tile_expert, n_tiles, image, N, K, out, ld_out, tiles, st);
    else
        launch_gemm<float>(glu, act, alpha, limit, A, ld_a, sorted, pair_div, pair_scale, tile_expert, n_tiles, image, N, K, out, ld_out, tiles, st);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}

extern "C" int tgis_moe_combine(const void* rows, int64_t ld_rows, const int32_t* pos_of_pair, const float* pair_weight, int k,
                                const void* shared, int64_t ld_shared, const float* shared_gate, void* out, int64_t ld_out, int64_t T,
                                int64_t W, int dtype, void* stream) {
    TGIS_CHECK_ARG(rows && pos_of_pair && out && k >= 1 && W >= 1 && ld_rows >= W && ld_out >= W && (!shared || ld_shared >= W),
                   "tgis_moe_combine: bad arguments");
    TGIS_CHECK_ARG(dtype3(dtype), "tgis_moe_combine: bad dtype");
    if (T == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    if (dtype == TGIS_F16)
        hipLaunchKernelGGL(moe_combine_kernel<f16>, dim3((unsigned)T, (unsigned)cdiv64(W, 256)), dim3(256), 0, st, (const f16*)rows, ld_rows, pos_of_pair, pair_weight, k, (const f16*)shared, ld_shared, shared_gate, (f16*)out, ld_out, W);
    else if (dtype == TGIS_BF16)
        hipLaunchKernelGGL(moe_combine_kernel<bf16>, dim3((unsigned)T, (unsigned)cdiv64(W, 256)), dim3(256), 0, st, (const bf16*)rows, ld_rows, pos_of_pair, pair_weight, k, (const bf16*)shared, ld_shared, shared_gate, (bf16*)out, ld_out, W);
    else
        hipLaunchKernelGGL(moe_combine_kernel<float>, dim3((unsigned)T, (unsigned)cdiv64(W, 256)), dim3(256), 0, st, (const float*)rows, ld_rows, pos_of_pair, pair_weight, k, (const float*)shared, ld_shared, shared_gate, (float*)out, ld_out, W);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}
