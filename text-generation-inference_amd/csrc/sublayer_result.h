// What a sublayer leaves for the residual update behind it — rows of the activation dtype, the split-K slabs of its last
// projection, or the unsummed expert rows of a mixture with their weights and a gated shared row — and how an update reads it.
#pragma once
#include "row_io.h"

namespace {

// What the sublayer left (kind 0: nothing — the residual only feeds the next norm).
struct SublayerResult {
    int kind;               // 1: T rows, 2: fp32 slabs, 3: mixture
    const void* p;          // T rows / slabs / expert rows
    int64_t ld;
    int slabs;
    const int32_t* pos;     // mixture: [tokens][k] row of each (token, choice)
    const float* weight;    // [tokens][k] or null (ones)
    int k;
    const void* shared;     // T rows, or slabs if shared_slabs > 0; null: none
    int64_t ld_shared;
    int shared_slabs;
    const float* shared_gate;  // [tokens] or null (ones)
};

// sum of the split-K slabs [row / 32][S][32][ld] at (row, c), four loads in flight
template <int V> __device__ __forceinline__ f32x4 slab_sum(const void* p, int64_t ld, int slabs, int64_t row, int64_t c) {
    const float* sp = reinterpret_cast<const float*>(p) + ((row >> 5) * slabs * 32 + (row & 31)) * ld + c;
    const int64_t step = 32 * ld;
    f32x4 v = {};
    int s = 0;
    for (; s + 4 <= slabs; s += 4) {
        f32x4 t[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) t[i] = LdV<float, V>::ld(sp + (int64_t)(s + i) * step);
#pragma unroll
        for (int i = 0; i < 4; ++i) v += t[i];
    }
    for (; s < slabs; ++s) v += LdV<float, V>::ld(sp + (int64_t)s * step);
    return v;
}

template <typename T, int V> __device__ __forceinline__ f32x4 result_at(const SublayerResult& r, int64_t row, int64_t c) {
    if (r.kind == 1) return LdV<T, V>::ld(reinterpret_cast<const T*>(r.p) + row * r.ld + c);
    if (r.kind == 2) return slab_sum<V>(r.p, r.ld, r.slabs, row, c);
    const T* rows = reinterpret_cast<const T*>(r.p);
    f32x4 v = {};
    int j = 0;
    for (; j + 2 <= r.k; j += 2) {
        const int64_t p0 = r.pos[row * r.k + j], p1 = r.pos[row * r.k + j + 1];
        const f32x4 a = LdV<T, V>::ld(rows + p0 * r.ld + c), b = LdV<T, V>::ld(rows + p1 * r.ld + c);
        v += a * (r.weight ? r.weight[row * r.k + j] : 1.f);
        v += b * (r.weight ? r.weight[row * r.k + j + 1] : 1.f);
    }
    if (j < r.k) v += LdV<T, V>::ld(rows + (int64_t)r.pos[row * r.k + j] * r.ld + c) * (r.weight ? r.weight[row * r.k + j] : 1.f);
    if (r.shared) {
        const f32x4 s = r.shared_slabs > 0 ? slab_sum<V>(r.shared, r.ld_shared, r.shared_slabs, row, c)
                                           : LdV<T, V>::ld(reinterpret_cast<const T*>(r.shared) + row * r.ld_shared + c);
        v += s * (r.shared_gate ? r.shared_gate[row] : 1.f);
    }
    return v;
}

}  // namespace
