// One small matrix per head: out[t][h][n] = sum_k x[t][h][k] W[h][n][k] — what carries the queries of latent attention into
// latent space and its results out of it.  Heads of x and out lie at strides of their own inside a token's row, so nothing is
// copied or transposed on either side.
//
// A wave owns 32 tokens x NB * 32 outputs of one head: both operands are contiguous along k, fragments come straight from
// memory (mfma_frag.h).  A workgroup's four waves take neighbouring token tiles (long steps: they share W's fragments in L1)
// or neighbouring column blocks (decode).
#include "common.h"
#include "mfma_frag.h"

namespace {

template <typename T, int NB, bool WHOLE>
__global__ __launch_bounds__(256) void head_product_kernel(const T* __restrict__ x, int64_t ld_x, int64_t head_x, const T* __restrict__ w,
                                                           T* __restrict__ out, int64_t ld_out, int64_t head_out, int64_t Ttot, int N,
                                                           int K, int row_tiles, int col_blocks, int rows_first) {
    using F = Frag<T>;
    using V = typename F::V;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int unit = blockIdx.x * 4 + wave;
    if (unit >= row_tiles * col_blocks) return;
    const int rt = rows_first ? unit % row_tiles : unit / col_blocks, cb = rows_first ? unit / row_tiles : unit % col_blocks;
    const int h = blockIdx.y;
    const int r = lane & 31, half = lane >> 5;
    const int64_t t = (int64_t)rt * 32 + r;
    const T* ap = x + (t < Ttot ? t : Ttot - 1) * ld_x + h * head_x;  // clamped: rows past the end are computed and dropped
    const T* bp[NB];
    f32x16 acc[NB];
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
        const int n = (cb * NB + nb) * 32 + r;
        bp[nb] = w + ((int64_t)h * N + (n < N ? n : N - 1)) * K;
        acc[nb] = f32x16{};
    }
    auto frag = [&](const T* p, int k) {
        if (WHOLE) return k + F::PER <= K ? *reinterpret_cast<const V*>(p + k) : F::zero();  // K is a multiple of PER
        V v = F::zero();
#pragma unroll
        for (int i = 0; i < F::PER; ++i)
            if (k + i < K) v[i] = p[k + i];
        return v;
    };
#pragma unroll 2
    for (int k0 = 0; k0 < K; k0 += F::KSTEP) {
        const int k = k0 + half * F::PER;
        const V a = frag(ap, k);
#pragma unroll
        for (int nb = 0; nb < NB; ++nb) F::mma(a, frag(bp[nb], k), acc[nb]);
    }
#pragma unroll
    for (int nb = 0; nb < NB; ++nb) {
        const int n = (cb * NB + nb) * 32 + r;
        if (n >= N) continue;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int64_t row = (int64_t)rt * 32 + (i >> 2) * 8 + half * 4 + (i & 3);
            if (row < Ttot) out[row * ld_out + h * head_out + n] = (T)acc[nb][i];
        }
    }
}

template <typename T>
void launch(const void* x, int64_t ld_x, int64_t head_x, const void* w, void* out, int64_t ld_out, int64_t head_out, int64_t Ttot, int H,
            int N, int K, hipStream_t st) {
    const int64_t row_tiles = cdiv64(Ttot, 32);
    const bool many = row_tiles * H >= 1024;  // enough token tiles to fill the chip: two column blocks per wave
    const int nb = many ? 2 : 1;
    const int64_t col_blocks = cdiv64(N, 32 * nb);
    constexpr int PER = Frag<T>::PER;
    const bool whole = K % PER == 0 && ld_x % PER == 0 && head_x % PER == 0 && (((uintptr_t)x | (uintptr_t)w) & 15) == 0;
    dim3 grid((unsigned)cdiv64(row_tiles * col_blocks, 4), (unsigned)H);
#define TGIS_HEAD_PRODUCT(NB, WHOLE)                                                                                              \
    hipLaunchKernelGGL((head_product_kernel<T, NB, WHOLE>), grid, dim3(256), 0, st, (const T*)x, ld_x, head_x, (const T*)w, (T*)out, \
                       ld_out, head_out, Ttot, N, K, (int)row_tiles, (int)col_blocks, row_tiles >= 4 ? 1 : 0)
    if (many && whole)
        TGIS_HEAD_PRODUCT(2, true);
    else if (many)
        TGIS_HEAD_PRODUCT(2, false);
    else if (whole)
        TGIS_HEAD_PRODUCT(1, true);
    else
        TGIS_HEAD_PRODUCT(1, false);
#undef TGIS_HEAD_PRODUCT
}

}  // namespace

extern "C" int tgis_head_product(const void* x, int64_t ld_x, int64_t head_stride_x, const void* w, void* out, int64_t ld_out,
                                 int64_t head_stride_out, int64_t T, int H, int N, int K, int dtype, void* stream) {
    TGIS_CHECK_ARG(x && w && out, "tgis_head_product: null tensor");
    TGIS_CHECK_ARG(H >= 1 && H <= 65535 && N >= 1 && K >= 1 && head_stride_x >= K && head_stride_out >= N &&
                       ld_x >= (H - 1) * head_stride_x + K && ld_out >= (H - 1) * head_stride_out + N,
                   "tgis_head_product: bad geometry (H %d, N %d, K %d)", H, N, K);
    TGIS_CHECK_ARG(dtype == TGIS_F16 || dtype == TGIS_BF16 || dtype == TGIS_F32, "tgis_head_product: bad dtype");
    if (T == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_HEAD_PRODUCT, st);
    if (dtype == TGIS_F16)
        launch<f16>(x, ld_x, head_stride_x, w, out, ld_out, head_stride_out, T, H, N, K, st);
    else if (dtype == TGIS_BF16)
        launch<bf16>(x, ld_x, head_stride_x, w, out, ld_out, head_stride_out, T, H, N, K, st);
    else
        launch<float>(x, ld_x, head_stride_x, w, out, ld_out, head_stride_out, T, H, N, K, st);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}
