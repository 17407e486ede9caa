// minGRU: a gated recurrence whose gate and candidate read the current token only.  Per channel and sequence
//
//     z = sigmoid(z_t);   c = x_t + 1/2 if x_t >= 0 else sigmoid(x_t);   S <- (1 - z) S + z c;   out_t = S silu(g_t) * out_scale
//
// z, x, g are columns of one projection.  The recurrence is a first-order linear one, S_t = a_t S_(t-1) + b_t, and such steps
// compose: a run of tokens is (P, Q) = (product of the a, result from a zero state).  The waves of a workgroup own neighbouring
// runs of tokens of the same 64 (128) channels, walk them from zero, leave (P, Q) in LDS and take their start state from the
// runs before them: one barrier per NW * RT tokens.  Gates, composition and state are fp32.
#include "common.h"

namespace {

template <bool FAST> __device__ __forceinline__ float sigm(float z) {
    // two-byte serving: the hardware's base-two exponential and reciprocal (about one unit in the last fp32 place)
    if (FAST) return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
    return 1.f / (1.f + expf(-z));
}

template <typename T, int VEC> struct Raw;
template <typename T> struct Raw<T, 1> {
    T v[1];
    __device__ __forceinline__ void ld(const T* p) { v[0] = *p; }
};
template <> struct Raw<float, 2> {
    float v[2];
    __device__ __forceinline__ void ld(const float* p) { f32x2 t = *reinterpret_cast<const f32x2*>(p); v[0] = t[0]; v[1] = t[1]; }
};
template <typename T> struct Raw<T, 2> {
    T v[2];
    __device__ __forceinline__ void ld(const T* p) { typename VecT<T>::x2 t = *reinterpret_cast<const typename VecT<T>::x2*>(p); v[0] = t[0]; v[1] = t[1]; }
};

template <typename T, int VEC, int RT, int NW>
__global__ __launch_bounds__(64 * NW) void min_gru_kernel(const T* __restrict__ proj, int64_t ld, int64_t z_col, int64_t x_col, int64_t g_col,
                                                          float* __restrict__ state, const int32_t* __restrict__ state_slots,
                                                          const int32_t* __restrict__ cu_q, const int32_t* __restrict__ positions,
                                                          T* __restrict__ out, int64_t ld_out, float out_scale, int D) {
    constexpr bool FAST = sizeof(T) == 2;
    __shared__ float runs[NW > 1 ? 2 : 1][2][NW][64 * VEC];  // [round parity][P | Q][wave][channel]
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int b = blockIdx.y;
    const int t0 = cu_q[b], n = cu_q[b + 1] - t0;
    if (n <= 0) return;
    const int c = (blockIdx.x * 64 + lane) * VEC;
    const bool live = c < D;  // VEC 2: D is even
    float* srow = state + (int64_t)state_slots[b] * D + c;
    float carry[VEC];
#pragma unroll
    for (int v = 0; v < VEC; ++v) carry[v] = (live && positions[t0] > 0) ? srow[v] : 0.f;
    const T* base = proj + (int64_t)t0 * ld + (live ? c : 0);
    int parity = 0;
    for (int r0 = 0; r0 < n; r0 += NW * RT, parity ^= 1) {
        const int first = r0 + wave * RT;
        Raw<T, VEC> zr[RT], xr[RT], gr[RT];
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            const int64_t row = (int64_t)min(first + i, n - 1) * ld;  // rows past the end: loaded, not used
            zr[i].ld(base + row + z_col);
            xr[i].ld(base + row + x_col);
            gr[i].ld(base + row + g_col);
        }
        float P[RT][VEC], Q[RT][VEC], p[VEC], q[VEC];
#pragma unroll
        for (int v = 0; v < VEC; ++v) {
            p[v] = 1.f;
            q[v] = 0.f;
        }
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            const bool in = first + i < n;
#pragma unroll
            for (int v = 0; v < VEC; ++v) {
                const float z = in ? sigm<FAST>((float)zr[i].v[v]) : 0.f;  // z = 0: the state stays
                const float u = (float)xr[i].v[v];
                const float cand = u >= 0.f ? u + 0.5f : sigm<FAST>(u);
                const float a = 1.f - z;
                q[v] = a * q[v] + z * cand;
                p[v] *= a;
                P[i][v] = p[v];
                Q[i][v] = q[v];
            }
        }
        float S[VEC];
        if (NW > 1) {
#pragma unroll
            for (int v = 0; v < VEC; ++v) {
                runs[parity][0][wave][lane * VEC + v] = p[v];
                runs[parity][1][wave][lane * VEC + v] = q[v];
            }
            __syncthreads();  // the other parity's buffer is free again: every wave has passed this barrier of the round before
#pragma unroll
            for (int v = 0; v < VEC; ++v) {
                float s = carry[v];
                S[v] = s;
#pragma unroll
                for (int w = 0; w < NW; ++w) {
                    if (w == wave) S[v] = s;
                    s = runs[parity][0][w][lane * VEC + v] * s + runs[parity][1][w][lane * VEC + v];
                }
                carry[v] = s;
            }
        } else {
#pragma unroll
            for (int v = 0; v < VEC; ++v) {
                S[v] = carry[v];
                carry[v] = p[v] * carry[v] + q[v];
            }
        }
#pragma unroll
        for (int i = 0; i < RT; ++i) {
            if (live && first + i < n) {
                T* orow = out + (int64_t)(t0 + first + i) * ld_out + c;
#pragma unroll
                for (int v = 0; v < VEC; ++v) {
                    const float g = (float)gr[i].v[v];
                    orow[v] = (T)((P[i][v] * S[v] + Q[i][v]) * (g * sigm<FAST>(g)) * out_scale);
                }
            }
        }
    }
    if (live && wave == 0) {
#pragma unroll
        for (int v = 0; v < VEC; ++v) srow[v] = carry[v];
    }
}

template <typename T>
void launch(const void* proj, int64_t ld, int64_t z_col, int64_t x_col, int64_t g_col, float* state, const int32_t* state_slots,
            const int32_t* cu_q, const int32_t* positions, void* out, int64_t ld_out, float out_scale, int64_t B, int64_t max_q, int64_t D,
            hipStream_t st) {
    const size_t pair = 2 * sizeof(T);
    const bool pairs = D % 2 == 0 && ld % 2 == 0 && z_col % 2 == 0 && x_col % 2 == 0 && g_col % 2 == 0 && ((uintptr_t)proj % pair) == 0;
#define TGIS_MIN_GRU(VEC, RT, NW)                                                                                                 \
    hipLaunchKernelGGL((min_gru_kernel<T, VEC, RT, NW>), dim3((unsigned)cdiv64(D, 64 * VEC), (unsigned)B), dim3(64 * NW), 0, st, \
                       (const T*)proj, ld, z_col, x_col, g_col, state, state_slots, cu_q, positions, (T*)out, ld_out, out_scale, (int)D)
    // two channels per lane halve the memory instructions; they are taken where the workgroups still cover the chip
    if (max_q <= 2) {
        TGIS_MIN_GRU(1, 1, 1);
    } else if (max_q <= 32) {
        TGIS_MIN_GRU(1, 8, 4);
    } else if (pairs && B * cdiv64(D, 128) >= 512) {
        TGIS_MIN_GRU(2, 8, 8);
    } else {
        TGIS_MIN_GRU(1, 8, 16);
    }
#undef TGIS_MIN_GRU
}

}  // namespace

extern "C" int tgis_min_gru_scan(const void* proj, int64_t ld, int64_t z_col0, int64_t x_col0, int64_t g_col0, float* state,
                                 const int32_t* state_slots, const int32_t* cu_seqlens_q, const int32_t* positions, void* out,
                                 int64_t ld_out, float out_scale, int64_t B, int64_t T, int64_t max_q_len, int64_t D, int dtype,
                                 void* stream) {
    TGIS_CHECK_ARG(proj && state && state_slots && cu_seqlens_q && positions && out, "tgis_min_gru_scan: null tensor");
    TGIS_CHECK_ARG(D >= 1 && z_col0 >= 0 && x_col0 >= 0 && g_col0 >= 0 && ld >= z_col0 + D && ld >= x_col0 + D && ld >= g_col0 + D &&
                       ld_out >= D && B >= 1 && B <= 65535 && max_q_len >= 1,
                   "tgis_min_gru_scan: bad geometry (D %ld, ld %ld)", (long)D, (long)ld);
    TGIS_CHECK_ARG(dtype == TGIS_F16 || dtype == TGIS_BF16 || dtype == TGIS_F32, "tgis_min_gru_scan: bad dtype");
    if (T == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_SCAN, st);
    if (dtype == TGIS_F16)
        launch<f16>(proj, ld, z_col0, x_col0, g_col0, state, state_slots, cu_seqlens_q, positions, out, ld_out, out_scale, B, max_q_len, D, st);
    else if (dtype == TGIS_BF16)
        launch<bf16>(proj, ld, z_col0, x_col0, g_col0, state, state_slots, cu_seqlens_q, positions, out, ld_out, out_scale, B, max_q_len, D, st);
    else
        launch<float>(proj, ld, z_col0, x_col0, g_col0, state, state_slots, cu_seqlens_q, positions, out, ld_out, out_scale, B, max_q_len, D, st);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}
