// The choice of a router for one token, by one wave: k passes over E logits in LDS (consumed), ties go to the lower index.
// softmax_top: the weights are the softmax over the chosen logits, else the sigmoid of each.  k <= 64.
#pragma once
#include "common.h"

namespace {

__device__ __forceinline__ void route_top_wave(float* logit, int E, int k, int softmax_top, int32_t* __restrict__ idx,
                                               float* __restrict__ weight) {
    const int lane = threadIdx.x & 63;
    float mine = -INFINITY;  // lane j: the logit of choice j
    float top = 0.f;
    for (int j = 0; j < k; ++j) {
        float bv = -INFINITY;
        int best = 0x7fffffff;
        for (int e = lane; e < E; e += 64) {
            const float v = logit[e];
            if (v > bv) {
                bv = v;
                best = e;
            }
        }
        const float m = wave_max(bv);
        int cand = (bv == m && best != 0x7fffffff) ? best : 0x7fffffff;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) cand = min(cand, __shfl_xor(cand, o, 64));
        const int chosen = cand == 0x7fffffff ? 0 : cand;  // NaN logits: still a valid index
        if (j == 0) top = m;
        if (lane == j) {
            mine = m;
            idx[j] = chosen;
        }
        if ((chosen & 63) == lane) logit[chosen] = -INFINITY;
    }
    float w;
    if (softmax_top) {
        const float e = lane < k ? expf(mine - top) : 0.f;
        w = e / wave_sum(e);
    } else {
        w = 1.f / (1.f + expf(-mine));
    }
    if (lane < k) weight[lane] = w;
}

}  // namespace
