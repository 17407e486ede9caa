// Residual stream of designs that norm AFTER the sum: both sublayers of a layer read the stream itself and
//
//     x <- N(c x + y) * w           N(z) = z / sqrt(mean z^2 + eps), y what the sublayer left, c one constant of the model
//
// One launch per sublayer boundary: the sum, the norm, the stream in fp32 and its rounding to the activation dtype T (the operand of
// the next projections), optionally one more norm behind it (the end of the stack).  In front of the first sublayer the stream is the
// scaled embedding row, looked up here.  y arrives as the projection left it (sublayer_result.h).
//
// A sublayer that comes may need a few fp32 products of the stream — the logits of a router, the input and forget gates of a
// matrix memory.  On steps of few tokens they are made here, from the row in LDS (rounded to T, like any operand), and a router's
// experts are chosen by one wave of the same workgroup; long steps take tgis_narrow_product (matrix cores) and tgis_moe_choose.
#include "common.h"
#include "route_top.h"
#include "sublayer_result.h"
#include "wave_dpp.h"

namespace {

// Products the next sublayer wants of the row (w null: none).  idx null: they are the result (out [tokens][R]); else they are the
// logits of a grouped sigmoid router.
struct RowProducts {
    const void* w;   // [R][W] of the activation dtype
    int R;
    float* out;
    int32_t* idx;    // [tokens][k]
    float* weight;   // [tokens][k]
    int k, groups, keep;
    float scale;
};

// the sum over a workgroup of up to eight waves, in every thread
__device__ __forceinline__ float group_sum(float v, float* red) {
    v = wave_total(v);
    const int wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();  // red may still be read from the call before
    if ((threadIdx.x & 63) == 0) red[wave] = v;
    __syncthreads();
    float s = 0.f;
    for (int i = 0; i < nw; ++i) s += red[i];
    return s;
}

// eight consecutive elements of a row of products' weights
__device__ __forceinline__ void load8(const float* p, f32x4& a, f32x4& b) {
    a = Vec4<float>::ld(p);
    b = Vec4<float>::ld(p + 4);
}
template <typename T> __device__ __forceinline__ void load8(const T* p, f32x4& a, f32x4& b) {
    const typename VecT<T>::x8 v = *reinterpret_cast<const typename VecT<T>::x8*>(p);
    a = f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
    b = f32x4{(float)v[4], (float)v[5], (float)v[6], (float)v[7]};
}
__device__ __forceinline__ float dot4(f32x4 a, f32x4 b) { return a[0] * b[0] + a[1] * b[1] + a[2] * b[2] + a[3] * b[3]; }

// The products of the row in LDS, two rows of weights per wave at a time; then the choice of a router by wave 0.
template <typename T, bool VEC>
__device__ __forceinline__ void row_products(const float* urow, float* dots, int64_t row, int64_t W, const RowProducts& rp) {
    __syncthreads();
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = blockDim.x >> 6;
    const T* w = reinterpret_cast<const T*>(rp.w);
    for (int e = wave; e < rp.R; e += 2 * nw) {
        const bool two = e + nw < rp.R;
        const T* w0 = w + (int64_t)e * W;
        const T* w1 = two ? w0 + (int64_t)nw * W : w0;
        float s0 = 0.f, s1 = 0.f;
        if (VEC && (W & 7) == 0) {
#pragma unroll 4
            for (int64_t c = lane * 8; c < W; c += 512) {
                f32x4 a0, b0, a1, b1;
                load8(w0 + c, a0, b0);
                load8(w1 + c, a1, b1);
                const f32x4 x = Vec4<float>::ld(urow + c), y = Vec4<float>::ld(urow + c + 4);
                s0 += dot4(a0, x) + dot4(b0, y);
                s1 += dot4(a1, x) + dot4(b1, y);
            }
        } else {
            for (int64_t c = lane; c < W; c += 64) {
                s0 += Elem<T>::ld(w0 + c) * urow[c];
                s1 += Elem<T>::ld(w1 + c) * urow[c];
            }
        }
        s0 = wave_total(s0);
        s1 = wave_total(s1);
        if (lane == 0) {
            float* out = rp.idx ? dots : rp.out + row * rp.R;
            out[e] = s0;
            if (two) out[e + nw] = s1;
        }
    }
    if (!rp.idx) return;
    __syncthreads();
    if (wave != 0) return;
    route_grouped_sigmoid_wave(dots, dots + rp.R, rp.R, rp.k, rp.groups, rp.keep, rp.scale, rp.idx + row * rp.k, rp.weight + row * rp.k);
}

template <typename T, int V>
__global__ __launch_bounds__(512) void post_norm_kernel(const float* x, const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                        float emb_scale, int64_t vocab, float alpha, float* x_out, SublayerResult r,
                                                        const float* __restrict__ w, const float* __restrict__ w2, T* __restrict__ h,
                                                        int64_t W, float eps, RowProducts rp) {
    extern __shared__ __attribute__((aligned(16))) float urow[];  // [W] (+ products and group ranks)
    __shared__ float red[8];
    const int64_t row = blockIdx.x;
    const int64_t tok = ids ? min(max(ids[row], (int64_t)0), vocab - 1) : 0;
    const int64_t step = (int64_t)blockDim.x * V;
    float ss = 0.f;
    for (int64_t c = (int64_t)threadIdx.x * V; c < W; c += step) {
        f32x4 v = ids ? LdV<T, V>::ld(table + tok * W + c) * emb_scale : LdV<float, V>::ld(x + row * W + c);
        if (r.kind) v = v * alpha + result_at<T, V>(r, row, c);
#pragma unroll
        for (int i = 0; i < V; ++i) {
            urow[c + i] = v[i];
            ss += v[i] * v[i];
        }
    }
    // from here on a thread reads back what it wrote itself
    if (w) {
        ss = group_sum(ss, red);
        const float rinv = 1.f / sqrtf(ss / (float)W + eps);
        ss = 0.f;
        for (int64_t c = (int64_t)threadIdx.x * V; c < W; c += step) {
            const f32x4 g = LdV<float, V>::ld(w + c);
#pragma unroll
            for (int i = 0; i < V; ++i) {
                const float v = urow[c + i] * rinv * g[i];
                urow[c + i] = v;
                ss += v * v;
            }
        }
    }
    float rinv2 = 1.f;
    if (w2) {
        ss = group_sum(ss, red);
        rinv2 = 1.f / sqrtf(ss / (float)W + eps);
    }
    for (int64_t c = (int64_t)threadIdx.x * V; c < W; c += step) {
        f32x4 v = {};
#pragma unroll
        for (int i = 0; i < V; ++i) v[i] = urow[c + i];
        if (x_out) LdV<float, V>::st(x_out + row * W + c, v);
        if (w2) {
            const f32x4 g = LdV<float, V>::ld(w2 + c);
            v = v * rinv2 * g;
        }
        LdV<T, V>::st(h + row * W + c, v);
        if (rp.w) {
#pragma unroll
            for (int i = 0; i < V; ++i) urow[c + i] = (float)(T)v[i];
        }
    }
    if (rp.w) row_products<T, V == 4>(urow, urow + W, row, W, rp);
}

// The same for W % 4 == 0 up to 512 * 4 * NV: a thread keeps NV groups of four consecutive elements in registers, and everything the
// row needs is asked for in front of the first sum — a decode step is a few rows, so the launch is a chain of trips to memory.
template <typename T, int NV>
__global__ __launch_bounds__(512) void post_norm_held_kernel(const float* x, const int64_t* __restrict__ ids, const T* __restrict__ table,
                                                             float emb_scale, int64_t vocab, float alpha, float* x_out, SublayerResult r,
                                                             const float* __restrict__ w, const float* __restrict__ w2, T* __restrict__ h,
                                                             int64_t W, float eps, RowProducts rp) {
    extern __shared__ __attribute__((aligned(16))) float urow[];  // products: [W] + products and group ranks
    __shared__ float red[8];
    const int64_t row = blockIdx.x;
    const int64_t tok = ids ? min(max(ids[row], (int64_t)0), vocab - 1) : 0;
    f32x4 v[NV], g[NV], g2[NV];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int64_t c = ((int64_t)threadIdx.x + blockDim.x * i) * 4;
        v[i] = g[i] = g2[i] = f32x4{};
        if (c < W) {
            v[i] = ids ? Vec4<T>::ld(table + tok * W + c) * emb_scale : Vec4<float>::ld(x + row * W + c);
            if (w) g[i] = Vec4<float>::ld(w + c);
            if (w2) g2[i] = Vec4<float>::ld(w2 + c);
        }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int64_t c = ((int64_t)threadIdx.x + blockDim.x * i) * 4;
        if (r.kind && c < W) v[i] = v[i] * alpha + result_at<T, 4>(r, row, c);
        ss += dot4(v[i], v[i]);
    }
    if (w) {
        ss = group_sum(ss, red);
        const float rinv = 1.f / sqrtf(ss / (float)W + eps);
        ss = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            v[i] = v[i] * rinv * g[i];
            ss += dot4(v[i], v[i]);
        }
    }
    if (x_out) {
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int64_t c = ((int64_t)threadIdx.x + blockDim.x * i) * 4;
            if (c < W) Vec4<float>::st(x_out + row * W + c, v[i]);
        }
    }
    if (w2) {
        ss = group_sum(ss, red);
        const float rinv = 1.f / sqrtf(ss / (float)W + eps);
#pragma unroll
        for (int i = 0; i < NV; ++i) v[i] = v[i] * rinv * g2[i];
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int64_t c = ((int64_t)threadIdx.x + blockDim.x * i) * 4;
        if (c < W) {
            Vec4<T>::st(h + row * W + c, v[i]);
            if (rp.w) Vec4<float>::st(urow + c, f32x4{(float)(T)v[i][0], (float)(T)v[i][1], (float)(T)v[i][2], (float)(T)v[i][3]});
        }
    }
    if (rp.w) row_products<T, true>(urow, urow + W, row, W, rp);
}

template <typename T>
void launch_post_norm(bool vec, const float* x, const int64_t* ids, const void* table, float emb_scale, int64_t vocab, float alpha, float* x_out,
                      const SublayerResult& r, const float* w, const float* w2, void* h, int64_t rows, int64_t W, float eps, const RowProducts& rp,
                      hipStream_t st) {
    const int64_t lanes = vec ? W / 4 : W;
    const size_t products = rp.w ? ((size_t)rp.R + (rp.idx ? rp.groups : 0)) * 4 : 0;
    // products of the row keep eight waves busy whatever the width
    const int nt = rp.w ? 512 : (int)(lanes >= 512 ? 512 : (lanes + 63) / 64 * 64);
#define TGIS_POST_NORM(KERNEL, LDS)                                                                                                          \
    hipLaunchKernelGGL(KERNEL, dim3((unsigned)rows), dim3(nt), LDS, st, x, ids, (const T*)table, emb_scale, vocab, alpha, x_out, r, w, w2,   \
                       (T*)h, W, eps, rp)
    if (vec && W <= 512 * 4)
        TGIS_POST_NORM((post_norm_held_kernel<T, 1>), (rp.w ? (size_t)W * 4 : 0) + products);
    else if (vec && W <= 512 * 8)
        TGIS_POST_NORM((post_norm_held_kernel<T, 2>), (rp.w ? (size_t)W * 4 : 0) + products);
    else if (vec && W <= 512 * 16)
        TGIS_POST_NORM((post_norm_held_kernel<T, 4>), (rp.w ? (size_t)W * 4 : 0) + products);
    else if (vec)
        TGIS_POST_NORM((post_norm_kernel<T, 4>), (size_t)W * 4 + products);
    else
        TGIS_POST_NORM((post_norm_kernel<T, 1>), (size_t)W * 4 + products);
#undef TGIS_POST_NORM
}

// ---- out[t][n] = sum_c h[t][c] w[n][c] in fp32 for few outputs and many tokens (two-byte h and w, fp32 sums) --------------------
// Workgroup = four waves = 16 tokens x 64 outputs; the waves split the channels in interleaved steps of 32 and meet in LDS.
// Fragments come straight from memory: lane l holds token (or output) l % 16 and 8 channels at offset 8 (l / 16).
template <typename T>
__global__ __launch_bounds__(256) void narrow_product_kernel(const T* __restrict__ h, int64_t ld_h, const T* __restrict__ w, float* __restrict__ out,
                                                             int64_t rows, int R, int64_t W) {
    using V8 = typename VecT<T>::x8;
    __shared__ float part[4][16][68];
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int r = lane & 15, q = lane >> 4;
    const int64_t t0 = (int64_t)blockIdx.x * 16;
    const int n0 = blockIdx.y * 64;
    const T* hp = h + min(t0 + r, rows - 1) * ld_h + q * 8;
    const T* wp[4];
#pragma unroll
    for (int b = 0; b < 4; ++b) wp[b] = w + (int64_t)min(n0 + b * 16 + r, R - 1) * W + q * 8;
    f32x4 acc[4] = {};
    const int steps = (int)(W >> 5);
    int s = wave;
    for (; s + 4 < steps; s += 8) {  // two steps' fragments in flight
        const V8 a0 = *reinterpret_cast<const V8*>(hp + s * 32), a1 = *reinterpret_cast<const V8*>(hp + (s + 4) * 32);
        V8 b0[4], b1[4];
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            b0[b] = *reinterpret_cast<const V8*>(wp[b] + s * 32);
            b1[b] = *reinterpret_cast<const V8*>(wp[b] + (s + 4) * 32);
        }
#pragma unroll
        for (int b = 0; b < 4; ++b) {
            acc[b] = mfma16(a0, b0[b], acc[b]);
            acc[b] = mfma16(a1, b1[b], acc[b]);
        }
    }
    if (s < steps) {
        const V8 a = *reinterpret_cast<const V8*>(hp + s * 32);
#pragma unroll
        for (int b = 0; b < 4; ++b) acc[b] = mfma16(a, *reinterpret_cast<const V8*>(wp[b] + s * 32), acc[b]);
    }
    if ((W & 31) && wave == 0) {  // the last step is short: W is a multiple of 8, so a lane's fragment is whole or absent
        const bool in = steps * 32 + q * 8 + 8 <= W;
        const V8 a = in ? *reinterpret_cast<const V8*>(hp + steps * 32) : V8{};
#pragma unroll
        for (int b = 0; b < 4; ++b) acc[b] = mfma16(a, in ? *reinterpret_cast<const V8*>(wp[b] + steps * 32) : V8{}, acc[b]);
    }
    // accumulator i of lane l: token 4 (l / 16) + i, output l % 16
#pragma unroll
    for (int b = 0; b < 4; ++b)
#pragma unroll
        for (int i = 0; i < 4; ++i) part[wave][q * 4 + i][b * 16 + r] = acc[b][i];
    __syncthreads();
    for (int e = threadIdx.x; e < 16 * 64; e += 256) {
        const int m = e >> 6, n = e & 63;
        if (t0 + m < rows && n0 + n < R)
            out[(t0 + m) * R + n0 + n] = part[0][m][n] + part[1][m][n] + part[2][m][n] + part[3][m][n];
    }
}

}  // namespace

extern "C" int tgis_post_norm_update(const float* x, const int64_t* ids, const void* table, int64_t vocab, float emb_scale, float alpha,
                                     float* x_out, int kind, const void* y, int64_t ld_y, int slabs, const int32_t* pos,
                                     const float* pair_weight, int pairs, const float* w, const float* w2, void* h, int64_t rows, int64_t W,
                                     float eps, const void* dot_w, int R, float* dot_out, int32_t* idx, float* route_weight, int top,
                                     int groups, int keep, float route_scale, int dtype, void* stream) {
    TGIS_CHECK_ARG(dtype == TGIS_F16 || dtype == TGIS_BF16 || dtype == TGIS_F32, "tgis_post_norm_update: bad dtype");
    TGIS_CHECK_ARG((x != nullptr) != (ids != nullptr) && h && (!ids || (table && vocab >= 1)), "tgis_post_norm_update: a stream, or token ids and their table");
    TGIS_CHECK_ARG(kind >= 0 && kind <= 3 && (kind == 0 || (y && ld_y >= W)) && (kind != 2 || slabs >= 1) && (kind != 3 || (pos && pairs >= 1)),
                   "tgis_post_norm_update: bad sublayer result (kind %d)", kind);
    TGIS_CHECK_ARG(!dot_w || (R >= 1 && (idx ? (route_weight != nullptr) : (dot_out != nullptr))), "tgis_post_norm_update: products need a place");
    TGIS_CHECK_ARG(!dot_w || !idx || (top >= 1 && top <= 64 && groups >= 1 && R % groups == 0 && keep >= 1 && keep <= groups && (int64_t)keep * (R / groups) >= top),
                   "tgis_post_norm_update: cannot choose %d of %d experts in the best %d of %d groups", top, R, keep, groups);
    TGIS_CHECK_ARG(W >= 1 && (W + (dot_w ? R + (idx ? groups : 0) : 0)) * 4 <= 64 * 1024, "tgis_post_norm_update: up to 16384 channels and products (got %ld)", (long)W);
    if (rows == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_NORM, st);
    const RowProducts rp{dot_w, R, dot_out, idx, route_weight, top, groups, keep, route_scale};
    const SublayerResult r{kind, y, ld_y, slabs, pos, pair_weight, pairs, nullptr, 0, 0, nullptr};
    auto al = [](const void* p, size_t n) { return ((uintptr_t)p % n) == 0; };
    const size_t e4 = dtype == TGIS_F32 ? 16 : 8;
    const bool vec = W % 4 == 0 && al(x, 16) && al(x_out, 16) && al(table, e4) && al(h, e4) && al(w, 16) && al(w2, 16) && al(dot_w, 16) &&
                     (kind == 0 || (ld_y % 4 == 0 && al(y, kind == 2 ? 16 : e4)));
    if (dtype == TGIS_F16)
        launch_post_norm<f16>(vec, x, ids, table, emb_scale, vocab, alpha, x_out, r, w, w2, h, rows, W, eps, rp, st);
    else if (dtype == TGIS_BF16)
        launch_post_norm<bf16>(vec, x, ids, table, emb_scale, vocab, alpha, x_out, r, w, w2, h, rows, W, eps, rp, st);
    else
        launch_post_norm<float>(vec, x, ids, table, emb_scale, vocab, alpha, x_out, r, w, w2, h, rows, W, eps, rp, st);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}

extern "C" int tgis_narrow_product(const void* h, int64_t ld_h, const void* w, float* out, int64_t rows, int R, int64_t W, int dtype, void* stream) {
    TGIS_CHECK_ARG(h && w && out && R >= 1 && W >= 8 && W % 8 == 0 && ld_h >= W && ld_h % 8 == 0, "tgis_narrow_product: width and row stride are multiples of 8 (got %ld, %ld)", (long)W, (long)ld_h);
    TGIS_CHECK_ARG((dtype == TGIS_F16 || dtype == TGIS_BF16) && (((uintptr_t)h | (uintptr_t)w) & 15) == 0, "tgis_narrow_product: two-byte operands, 16-byte aligned");
    TGIS_CHECK_ARG(cdiv64(R, 64) <= 65535 && cdiv64(rows, 16) < (1ll << 31), "tgis_narrow_product: too large");
    if (rows == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_DENSE_GEMM, st);
    const dim3 grid((unsigned)cdiv64(rows, 16), (unsigned)cdiv64(R, 64));
    if (dtype == TGIS_F16)
        hipLaunchKernelGGL(narrow_product_kernel<f16>, grid, dim3(256), 0, st, (const f16*)h, ld_h, (const f16*)w, out, rows, R, W);
    else
        hipLaunchKernelGGL(narrow_product_kernel<bf16>, grid, dim3(256), 0, st, (const bf16*)h, ld_h, (const bf16*)w, out, rows, R, W);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}
