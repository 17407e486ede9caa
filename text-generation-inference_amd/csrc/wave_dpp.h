// Sums and scans over neighbouring lanes by data-parallel-primitive moves (no trip through LDS).
#pragma once
#include "common.h"

namespace {

// lanes without a source get `old`
template <int CTRL, int ROWS = 0xF> __device__ __forceinline__ float moved(float old, float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, old), __builtin_bit_cast(int, v), CTRL, ROWS, 0xF, false));
}
__device__ __forceinline__ float lane_value(float v, int lane) {
    return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), lane));
}
// sums over 2, 4, 8 or 16 neighbouring lanes, in every one of them
template <int N> __device__ __forceinline__ float sum_neighbours(float v) {
    if (N >= 2) v += moved<0xB1>(0.f, v);    // lane ^ 1
    if (N >= 4) v += moved<0x4E>(0.f, v);    // lane ^ 2
    if (N >= 8) v += moved<0x141>(0.f, v);   // lane 7 - i of the half row: the other quad's total
    if (N >= 16) v += moved<0x140>(0.f, v);  // lane 15 - i of the row: the other half's
    return v;
}
// inclusive scans over the wave: within rows of 16, then row 0 into row 1 and row 2 into row 3, then lane 31 into the upper half
__device__ __forceinline__ float scan_sum(float v) {
    v += moved<0x111>(0.f, v);
    v += moved<0x112>(0.f, v);
    v += moved<0x114>(0.f, v);
    v += moved<0x118>(0.f, v);
    v += moved<0x142, 0xA>(0.f, v);
    v += moved<0x143, 0xC>(0.f, v);
    return v;
}
__device__ __forceinline__ float scan_max(float v) {
    v = fmaxf(v, moved<0x111>(-INFINITY, v));
    v = fmaxf(v, moved<0x112>(-INFINITY, v));
    v = fmaxf(v, moved<0x114>(-INFINITY, v));
    v = fmaxf(v, moved<0x118>(-INFINITY, v));
    v = fmaxf(v, moved<0x142, 0xA>(-INFINITY, v));
    v = fmaxf(v, moved<0x143, 0xC>(-INFINITY, v));
    return v;
}
// the wave's sum, in every lane
__device__ __forceinline__ float wave_total(float v) {
    v = sum_neighbours<16>(v);
    v += moved<0x142, 0xA>(0.f, v);
    v += moved<0x143, 0xC>(0.f, v);
    return lane_value(v, 63);
}

}  // namespace
