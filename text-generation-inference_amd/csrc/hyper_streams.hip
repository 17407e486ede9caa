// Several fp32 residual streams per token ("hyper-connections"): a sublayer f reads a weighted sum of the s streams and its
// result is spread over all of them while they are mixed,
//
//     u = sum_a c_in[a] X_a;    y = f(u / sqrt(mean u^2 + eps) * g);    X'_b = sum_a M[a][b] X_a + c_out[b] y
//
// One launch per sublayer boundary: it applies the update of the sublayer that just ran and makes the normed input of the next
// one (in front of the first sublayer the streams are s copies of the scaled embedding row, which it looks up itself).  y
// arrives as the projection left it: a tensor of T, the fp32 split-K slabs of the GEMM, or the unsummed expert rows of a
// mixture with their weights and a gated shared row.  Where the next sublayer is a mixture its router runs here too: the normed
// row is in LDS already (and has not been rounded to T).
//
// Layout: X [token][stream][W].  A workgroup per token; a column's s values stay in registers between the mix and the next
// sublayer's sum, whose row waits in LDS for the mean of squares.
#include "common.h"
#include "route_top.h"
#include "sublayer_result.h"

namespace {

constexpr int MAX_STREAMS = 8;

// The router of the sublayer that comes (w null: none): logits w h and sg h in fp32, the choice and the weights of route_top.h.
struct NextRouter {
    const float* w;   // [E][W]
    const float* sg;  // [W] or null
    int E, k, softmax_top;
    int32_t* idx;     // [tokens][k]
    float* weight;    // [tokens][k]
    float* shared_gate;  // [tokens]
};

// cur: [s * s mix (from, to) | s out] of the sublayer that ran (kind > 0); next: [s in | gain] of the one that comes.
template <typename T, int S, int V>
__global__ __launch_bounds__(512) void hyper_update_kernel(const float* x, const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                           float emb_scale, int64_t vocab, float* x_out, SublayerResult r,
                                                           const float* __restrict__ cur, const float* __restrict__ next, T* __restrict__ h,
                                                           int64_t W, float eps, NextRouter nr) {
    extern __shared__ float urow[];  // [W] (router: + E + 1 logits)
    __shared__ float red[8];
    const int64_t row = blockIdx.x;
    const int64_t tok = ids ? min(max(ids[row], (int64_t)0), vocab - 1) : 0;
    float cin[S], cout[S], mix[S][S];
#pragma unroll
    for (int a = 0; a < S; ++a) {
        cin[a] = next[a];
        cout[a] = r.kind ? cur[S * S + a] : 0.f;
#pragma unroll
        for (int b = 0; b < S; ++b) mix[a][b] = r.kind ? cur[a * S + b] : 0.f;
    }
    float ss = 0.f;
    for (int64_t c = (int64_t)threadIdx.x * V; c < W; c += (int64_t)blockDim.x * V) {
        f32x4 X[S], N[S];
        if (ids) {
            const f32x4 e = LdV<T, V>::ld(table + tok * W + c) * emb_scale;
#pragma unroll
            for (int a = 0; a < S; ++a) X[a] = e;
        } else {
#pragma unroll
            for (int a = 0; a < S; ++a) X[a] = LdV<float, V>::ld(x + (row * S + a) * W + c);
        }
        if (r.kind) {
            const f32x4 y = result_at<T, V>(r, row, c);
#pragma unroll
            for (int b = 0; b < S; ++b) {
                N[b] = y * cout[b];
#pragma unroll
                for (int a = 0; a < S; ++a) N[b] += X[a] * mix[a][b];
            }
        } else {
#pragma unroll
            for (int a = 0; a < S; ++a) N[a] = X[a];
        }
        f32x4 u = {};
#pragma unroll
        for (int a = 0; a < S; ++a) {
            if (x_out) LdV<float, V>::st(x_out + (row * S + a) * W + c, N[a]);
            u += N[a] * cin[a];
        }
#pragma unroll
        for (int i = 0; i < V; ++i) {
            urow[c + i] = u[i];
            ss += u[i] * u[i];
        }
    }
    ss = block_sum(ss, red);
    const float f = next[S] / sqrtf(ss / (float)W + eps);
    // a thread reads back what it wrote itself
    for (int64_t c = (int64_t)threadIdx.x * V; c < W; c += (int64_t)blockDim.x * V) {
        f32x4 u = {};
#pragma unroll
        for (int i = 0; i < V; ++i) u[i] = urow[c + i] * f;
        LdV<T, V>::st(h + row * W + c, u);
        if (nr.w) {
#pragma unroll
            for (int i = 0; i < V; ++i) urow[c + i] = u[i];
        }
    }
    if (!nr.w) return;
    __syncthreads();
    float* logit = urow + W;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = blockDim.x >> 6;
    for (int e = wave; e < nr.E + (nr.sg ? 1 : 0); e += nw) {
        const float* w = e < nr.E ? nr.w + (int64_t)e * W : nr.sg;
        float s = 0.f;
        if (V == 4) {
#pragma unroll 4
            for (int64_t c = lane * 4; c < W; c += 256) {
                const f32x4 wv = *reinterpret_cast<const f32x4*>(w + c);
                const f32x4 hv = *reinterpret_cast<const f32x4*>(urow + c);
                s += wv[0] * hv[0] + wv[1] * hv[1] + wv[2] * hv[2] + wv[3] * hv[3];
            }
        } else {
            for (int64_t c = lane; c < W; c += 64) s += w[c] * urow[c];
        }
        s = wave_sum(s);
        if (lane == 0) logit[e] = s;
    }
    __syncthreads();
    if (wave != 0) return;
    if (nr.sg && lane == 0) nr.shared_gate[row] = 1.f / (1.f + expf(-logit[nr.E]));
    route_top_wave(logit, nr.E, nr.k, nr.softmax_top, nr.idx + row * nr.k, nr.weight + row * nr.k);
}

template <typename T, int S>
void launch_s(bool vec, const float* x, const int64_t* ids, const void* table, float emb_scale, int64_t vocab, float* x_out,
              const SublayerResult& r, const float* cur, const float* next, void* h, int64_t rows, int64_t W, float eps, const NextRouter& nr, hipStream_t st) {
    const int64_t lanes = vec ? W / 4 : W;
    const size_t lds = ((size_t)W + (nr.w ? nr.E + 1 : 0)) * 4;
    const int nt = (int)(lanes >= 512 ? 512 : (lanes + 63) / 64 * 64);
    if (vec)
        hipLaunchKernelGGL((hyper_update_kernel<T, S, 4>), dim3((unsigned)rows), dim3(nt), lds, st, x, ids, (const T*)table, emb_scale,
                           vocab, x_out, r, cur, next, (T*)h, W, eps, nr);
    else
        hipLaunchKernelGGL((hyper_update_kernel<T, S, 1>), dim3((unsigned)rows), dim3(nt), lds, st, x, ids, (const T*)table, emb_scale,
                           vocab, x_out, r, cur, next, (T*)h, W, eps, nr);
}

template <typename T>
void launch_t(int S, bool vec, const float* x, const int64_t* ids, const void* table, float emb_scale, int64_t vocab, float* x_out,
              const SublayerResult& r, const float* cur, const float* next, void* h, int64_t rows, int64_t W, float eps, const NextRouter& nr, hipStream_t st) {
#define TGIS_HYPER(N) \
    case N: return launch_s<T, N>(vec, x, ids, table, emb_scale, vocab, x_out, r, cur, next, h, rows, W, eps, nr, st)
    switch (S) {
        TGIS_HYPER(1);
        TGIS_HYPER(2);
        TGIS_HYPER(3);
        TGIS_HYPER(4);
        TGIS_HYPER(5);
        TGIS_HYPER(6);
        TGIS_HYPER(7);
        TGIS_HYPER(8);
    }
#undef TGIS_HYPER
}

}  // namespace

extern "C" int tgis_hyper_update(const float* x, const int64_t* ids, const void* table, int64_t vocab, float emb_scale, float* x_out,
                                 int kind, const void* y, int64_t ld_y, int slabs, const int32_t* pos, const float* weight, int k,
                                 const void* shared, int64_t ld_shared, int shared_slabs, const float* shared_gate, const float* cur,
                                 const float* next, void* h, int64_t rows, int64_t W, int streams, float eps, const float* router_w,
                                 const float* router_sg, int E, int top, int softmax_top, int32_t* idx, float* route_weight,
                                 float* route_gate, int dtype, void* stream) {
    TGIS_CHECK_ARG(dtype == TGIS_F16 || dtype == TGIS_BF16 || dtype == TGIS_F32, "tgis_hyper_update: bad dtype");
    TGIS_CHECK_ARG((x != nullptr) != (ids != nullptr) && next && h && (!ids || (table && vocab >= 1 && kind == 0)),
                   "tgis_hyper_update: streams, or token ids and their table (and then no sublayer result)");
    TGIS_CHECK_ARG(!router_w || (E >= 1 && top >= 1 && top <= E && top <= 64 && idx && route_weight && (!router_sg || route_gate)),
                   "tgis_hyper_update: a router chooses 1 .. min(E, 64) of E experts (got %d of %d)", top, E);
    TGIS_CHECK_ARG(streams >= 1 && streams <= MAX_STREAMS && W >= 1 && (W + (router_w ? E + 1 : 0)) * 4 <= 64 * 1024,
                   "tgis_hyper_update: 1 .. %d streams of up to 16384 channels and logits (got %d of %ld)", MAX_STREAMS, streams, (long)W);
    TGIS_CHECK_ARG(kind >= 0 && kind <= 3 && (kind == 0 || (y && cur && ld_y >= W)) && (kind != 2 || slabs >= 1) && (kind != 3 || (pos && k >= 1)) &&
                       (!shared || (kind == 3 && ld_shared >= W && shared_slabs >= 0)),
                   "tgis_hyper_update: bad sublayer result (kind %d)", kind);
    if (rows == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_NORM, st);
    NextRouter nr{router_w, router_sg, E, top, softmax_top, idx, route_weight, route_gate};
    SublayerResult r{kind, y, ld_y, slabs, pos, weight, k, shared, ld_shared, shared_slabs, shared_gate};
    auto al = [](const void* p, size_t n) { return ((uintptr_t)p % n) == 0; };
    const size_t e4 = dtype == TGIS_F32 ? 16 : 8;
    const bool vec = W % 4 == 0 && al(x, 16) && al(x_out, 16) && al(table, e4) && al(h, e4) && al(router_w, 16) && al(router_sg, 16) && (kind == 0 || ld_y % 4 == 0) &&
                     al(y, kind == 2 ? 16 : e4) && (!shared || (ld_shared % 4 == 0 && al(shared, shared_slabs > 0 ? 16 : e4)));
    if (dtype == TGIS_F16)
        launch_t<f16>(streams, vec, x, ids, table, emb_scale, vocab, x_out, r, cur, next, h, rows, W, eps, nr, st);
    else if (dtype == TGIS_BF16)
        launch_t<bf16>(streams, vec, x, ids, table, emb_scale, vocab, x_out, r, cur, next, h, rows, W, eps, nr, st);
    else
        launch_t<float>(streams, vec, x, ids, table, emb_scale, vocab, x_out, r, cur, next, h, rows, W, eps, nr, st);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}
