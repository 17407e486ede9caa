// The choice of a router for one token, by one wave.  k passes over E numbers in LDS (consumed), ties go to the lower index; k <= 64.
#pragma once
#include "common.h"
#include "wave_dpp.h"

namespace {

// the k largest of score[0 .. E): idx[j], and in lane j the j-th of them (`mine`); `top` the largest
__device__ __forceinline__ void take_top_wave(float* score, int E, int k, int32_t* __restrict__ idx, float& mine, float& top) {
    const int lane = threadIdx.x & 63;
    mine = -INFINITY;
    top = 0.f;
    for (int j = 0; j < k; ++j) {
        float bv = -INFINITY;
        int best = 0x7fffffff;
        for (int e = lane; e < E; e += 64) {
            const float v = score[e];
            if (v > bv) {
                bv = v;
                best = e;
            }
        }
        const float m = lane_value(scan_max(bv), 63);
        const uint64_t hit = __ballot(bv == m && best != 0x7fffffff);
        int cand = 0x7fffffff;
        if (E <= 64) {  // a lane has one number: the lowest lane that holds the maximum
            if (hit) cand = __ffsll((unsigned long long)hit) - 1;
        } else {
            cand = (hit >> lane & 1) ? best : 0x7fffffff;
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) cand = min(cand, __shfl_xor(cand, o, 64));
        }
        const int chosen = cand == 0x7fffffff ? 0 : cand;  // NaN: still a valid index
        if (j == 0) top = m;
        if (lane == j) {
            mine = m;
            idx[j] = chosen;
        }
        if ((chosen & 63) == lane) score[chosen] = -INFINITY;
    }
}

// softmax_top: the weights are the softmax over the chosen logits, else the sigmoid of each.
__device__ __forceinline__ void route_top_wave(float* logit, int E, int k, int softmax_top, int32_t* __restrict__ idx,
                                               float* __restrict__ weight) {
    const int lane = threadIdx.x & 63;
    float mine, top;
    take_top_wave(logit, E, k, idx, mine, top);
    float w;
    if (softmax_top) {
        const float e = lane < k ? expf(mine - top) : 0.f;
        w = e / wave_sum(e);
    } else {
        w = 1.f / (1.f + expf(-mine));
    }
    if (lane < k) weight[lane] = w;
}

// Scores are the sigmoids of the logits.  The experts form `groups` equal groups of neighbours; a group counts by the sum of its two
// largest scores and only the `keep` best groups may be chosen from (keep * (E / groups) >= k).  Weights are the chosen scores times
// `scale`.  rank [groups] is LDS scratch.
__device__ __forceinline__ void route_grouped_sigmoid_wave(float* logit, float* rank, int E, int k, int groups, int keep, float scale,
                                                           int32_t* __restrict__ idx, float* __restrict__ weight) {
    const int lane = threadIdx.x & 63;
    for (int e = lane; e < E; e += 64) logit[e] = 1.f / (1.f + expf(-logit[e]));
    if (keep < groups) {
        const int per = E / groups;
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        for (int g = lane; g < groups; g += 64) {
            float a = -INFINITY, b = -INFINITY;  // the largest and the second
            for (int e = g * per; e < (g + 1) * per; ++e) {
                const float v = logit[e];
                b = fmaxf(b, fminf(a, v));
                a = fmaxf(a, v);
            }
            rank[g] = per > 1 ? a + b : a;
        }
        __threadfence_block();
        __builtin_amdgcn_wave_barrier();
        for (int e = lane; e < E; e += 64) {
            const int g = e / per;
            const float mine = rank[g];
            int ahead = 0;
            for (int o = 0; o < groups; ++o) ahead += (rank[o] > mine || (rank[o] == mine && o < g)) ? 1 : 0;
            if (ahead >= keep) logit[e] = -INFINITY;
        }
    }
    float mine, top;
    take_top_wave(logit, E, k, idx, mine, top);
    if (lane < k) weight[lane] = mine * scale;
}

}  // namespace
