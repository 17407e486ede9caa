// Loads and stores of row elements in the activation dtypes (fp32 in registers), and the sum over a workgroup: what the row
// kernels around an fp32 residual stream share.
#pragma once
#include "common.h"

namespace {

template <typename T> struct Elem;
template <> struct Elem<f16> { static __device__ __forceinline__ float ld(const f16* p) { return (float)*p; } };
template <> struct Elem<bf16> { static __device__ __forceinline__ float ld(const bf16* p) { return (float)*p; } };
template <> struct Elem<float> { static __device__ __forceinline__ float ld(const float* p) { return *p; } };
template <typename T> __device__ __forceinline__ T cvt_out(float v) { return (T)v; }

__device__ __forceinline__ float block_sum(float v, float* red) {
    // every thread of the block calls this; red holds one float per wave (<= 16)
    v = wave_sum(v);
    const int wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();  // red may still be read from a previous call
    if ((threadIdx.x & 63) == 0) red[wave] = v;
    __syncthreads();
    float s = 0.f;
    for (int i = 0; i < nw; ++i) s += red[i];
    return s;
}

template <typename T> struct Vec4;
template <> struct Vec4<float> {
    static __device__ __forceinline__ f32x4 ld(const float* p) { return *reinterpret_cast<const f32x4*>(p); }
    static __device__ __forceinline__ void st(float* p, f32x4 v) { *reinterpret_cast<f32x4*>(p) = v; }
};
template <> struct Vec4<bf16> {
    static __device__ __forceinline__ f32x4 ld(const bf16* p) {
        bf16x4 v = *reinterpret_cast<const bf16x4*>(p);
        return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
    }
    static __device__ __forceinline__ void st(bf16* p, f32x4 v) {
        *reinterpret_cast<bf16x4*>(p) = bf16x4{(bf16)v[0], (bf16)v[1], (bf16)v[2], (bf16)v[3]};
    }
};
template <> struct Vec4<f16> {
    static __device__ __forceinline__ f32x4 ld(const f16* p) {
        f16x4 v = *reinterpret_cast<const f16x4*>(p);
        return f32x4{(float)v[0], (float)v[1], (float)v[2], (float)v[3]};
    }
    static __device__ __forceinline__ void st(f16* p, f32x4 v) {
        *reinterpret_cast<f16x4*>(p) = f16x4{(f16)v[0], (f16)v[1], (f16)v[2], (f16)v[3]};
    }
};

// one element (in component 0) or four
template <typename T, int V> struct LdV;
template <typename T> struct LdV<T, 1> {
    static __device__ __forceinline__ f32x4 ld(const T* p) { return f32x4{Elem<T>::ld(p), 0.f, 0.f, 0.f}; }
    static __device__ __forceinline__ void st(T* p, f32x4 v) { *p = cvt_out<T>(v[0]); }
};
template <typename T> struct LdV<T, 4> {
    static __device__ __forceinline__ f32x4 ld(const T* p) { return Vec4<T>::ld(p); }
    static __device__ __forceinline__ void st(T* p, f32x4 v) { Vec4<T>::st(p, v); }
};

}  // namespace
