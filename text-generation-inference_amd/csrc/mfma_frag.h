// Operand fragments of the 32x32 matrix products for products whose operands are both contiguous along the inner dimension:
// lane l holds row (l % 32) and PER consecutive inner elements at offset (l / 32) * PER — a 16-byte load for A and for B.
#pragma once
#include "common.h"

namespace {

template <typename T> struct Frag;
template <> struct Frag<bf16> {
    static constexpr int KSTEP = 16, PER = 8;
    using V = bf16x8;
    static __device__ __forceinline__ V zero() { return V{}; }
    static __device__ __forceinline__ V scaled(V a, float s) {
        V r;
#pragma unroll
        for (int i = 0; i < 8; ++i) r[i] = (bf16)((float)a[i] * s);
        return r;
    }
    static __device__ __forceinline__ void mma(V a, V b, f32x16& c) { c = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0); }
};
template <> struct Frag<f16> {
    static constexpr int KSTEP = 16, PER = 8;
    using V = f16x8;
    static __device__ __forceinline__ V zero() { return V{}; }
    static __device__ __forceinline__ V scaled(V a, float s) {
        V r;
#pragma unroll
        for (int i = 0; i < 8; ++i) r[i] = (f16)((float)a[i] * s);
        return r;
    }
    static __device__ __forceinline__ void mma(V a, V b, f32x16& c) { c = __builtin_amdgcn_mfma_f32_32x32x16_f16(a, b, c, 0, 0, 0); }
};
template <> struct Frag<float> {
    static constexpr int KSTEP = 8, PER = 4;
    using V = f32x4;
    static __device__ __forceinline__ V zero() { return V{}; }
    static __device__ __forceinline__ V scaled(V a, float s) { return a * s; }
    // four 32x32x2 fp32 products: the k index a lane contributes to product i is (l / 32) * 4 + i, for A and B alike
    static __device__ __forceinline__ void mma(V a, V b, f32x16& c) {
#pragma unroll
        for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_32x32x2f32(a[i], b[i], c, 0, 0, 0);
    }
};

}  // namespace
