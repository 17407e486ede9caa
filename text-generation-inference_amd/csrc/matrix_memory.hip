// Matrix memory with exponential gates (mLSTM), per sequence and head, S [dk, dv], n [dk] and m in fp32:
//
//     m_t = max(f_t + m_(t-1), i_t)          i = soft(z_i + b_i),  f = ln sigmoid(soft(z_f + b_f)),  soft(z) = cap tanh(z / cap)
//     S_t = e^(f_t + m_(t-1) - m_t) S_(t-1) + e^(i_t - m_t) k_t v_t^T;      n_t likewise with k_t alone
//     o_t = c S_t^T q_t / (max(|c n_t . q_t|, e^(-m_t)) + read_eps)
//     out_t = o_t / sqrt(mean(o_t^2) + eps) * gain[h] * sigmoid(g_t)       (norm per head over dv, gains of all heads side by side)
//
// Every sequence starts from S = 0, n = 0, m = 0.  q, k, v and the output gate's logits g are columns of one projection (activation
// dtype T); z_i, z_f are fp32 [T][2 H].  A slot of the state cache holds S [H][dk][dv] and (n, m) [H][dk + 1]; a step that starts at
// position 0 starts from zeros whatever the slot holds.
//
// matrix_memory_scan_kernel: token by token, any dtype and size up to 256 x 256 (decode, short runs, fp32 serving).  Workgroup =
// (sequence, head) = LPC dv_pad / CPL threads: LPC neighbouring lanes share column j of S (with CPL = 2 also j + dv_pad / 2), each
// keeps RPL rows of it in registers.  Tokens go through LDS in stages of `ts`, two buffers deep, the next stage on its way to
// registers while the current one is worked on; the stage's decays and write weights (one pair per token and head) are made by one
// wave, which carries m from stage to stage token by token; rows of n belong to the first dk threads.
//
// matrix_memory_chunk_kernel: long runs of bf16 models, heads of up to 128 x 128, 64 tokens at a time on the matrix cores.  With
// F_t = sum_(s <= t) f_s counted from the chunk's start and a_s = i_s - F_s, the maximum is m_t = F_t + M_t with M_t = max(m_0, max_(s <= t) a_s)
// and the recurrence becomes
//     S_t^T q_t = e^(m_0 - M_t) S_0^T q_t + sum_(s <= t) e^(a_s - M_t) (q_t . k_s) v_s        n_t . q_t the same with 1 for v_s
//     S_C = e^(m_0 - M_C) S_0 + sum_s e^(a_s - M_C) k_s v_s^T                                  (every exponent <= 0)
// q, k and v are bf16 already, so the products q . k are exact in fp32; the weighted scores, the state as an operand and the weighted
// values are fp32 numbers, each taken as the sum of two bf16 (16 bits of mantissa) with fp32 accumulation; the state itself stays in
// fp32 accumulators from the first chunk to the last.  Workgroup = (sequence, head) = eight waves; wave w owns value columns
// 32 (w % 4) .. with half of their rows of S, and leaves its share of the read-outs in LDS, where the two halves meet; the score tiles
// are shared through LDS too.
#include <algorithm>
#include "common.h"
#include "wave_dpp.h"

namespace {

constexpr int SEG_PAD = 4;  // floats between the row groups' segments
constexpr int PFQ = 4;      // (q, k) pairs and
constexpr int PFV = 4;      // values of the next stage that a thread holds in registers: ts dk <= PFQ threads, ts dv_pad <= PFV threads
constexpr int MAX_TS = 32;  // a stage's gates are made by one wave, half of it idle

struct MemoryArgs {
    const void* proj;
    int64_t ld, q_col0, k_col0, v_col0, g_col0;  // g_col0 < 0: no output gate
    const float* gates;                          // [T][ld_gates]: z_i of head h at h, z_f at H + h
    int64_t ld_gates;
    const float* i_bias;
    const float* f_bias;
    float cap;
    const float* gain;  // [H dv]
    float* state;
    float* memory;
    const int32_t* state_slots;
    const int32_t* cu_q;
    const int32_t* positions;
    void* out;
    int64_t ld_out;
    int H, dk, dv;
    float q_scale, eps, read_eps;
    int dv_pad, ts;
};

__device__ __forceinline__ float soft_capped(float z, float cap) { return cap * tanhf(z / cap); }
// ln(sigmoid(z)) without cancellation at either end
__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
// (i, f) of head h at token t
__device__ __forceinline__ void log_gates(const MemoryArgs& a, int64_t t, int h, float& li, float& lf) {
    const float* z = a.gates + t * a.ld_gates;
    li = soft_capped(z[h] + (a.i_bias ? a.i_bias[h] : 0.f), a.cap);
    lf = log_sigmoid(soft_capped(z[a.H + h] + (a.f_bias ? a.f_bias[h] : 0.f), a.cap));
}
template <typename T> __device__ __forceinline__ float output_gate(const MemoryArgs& a, int64_t t, int col) {
    if (a.g_col0 < 0) return 1.f;
    const float g = (float)reinterpret_cast<const T*>(a.proj)[t * a.ld + a.g_col0 + col];
    return 1.f / (1.f + expf(-g));
}

template <typename T, int RPL, int CPL, int LPC, int MAXT>
__global__ __launch_bounds__(MAXT) void matrix_memory_scan_kernel(MemoryArgs a) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    constexpr int SEG = RPL + SEG_PAD, ROW = LPC * SEG;
    const int ts = a.ts, dk = a.dk, dv = a.dv, dv_pad = a.dv_pad;
    float* qs = smem;                    // [2][ts][ROW]
    float* ks = qs + 2 * ts * ROW;       // [2][ts][ROW]
    float* vs = ks + 2 * ts * ROW;       // [2][ts][dv_pad]
    float* os = vs + 2 * ts * dv_pad;    // [ts][dv_pad]
    float* nq = os + ts * dv_pad;        // [ts][dk]: products of n and q
    f32x2* gs = reinterpret_cast<f32x2*>(nq + ((ts * dk + 1) & ~1));  // [2][ts]: (decay, write weight)
    float* fl = reinterpret_cast<float*>(gs + 2 * ts);                 // [2][ts]: e^-m
    const int b = blockIdx.x, h = blockIdx.y;
    const int tid = threadIdx.x, j = tid / LPC, qd = tid % LPC;
    const int t0 = a.cu_q[b], qlen = a.cu_q[b + 1] - t0;
    if (qlen <= 0) return;
    const int nthreads = blockDim.x;
    const int wave = tid >> 6, lane = tid & 63, nw = nthreads >> 6;
    const bool fresh = a.positions[t0] == 0;
    const T* proj = reinterpret_cast<const T*>(a.proj);
    const int64_t slot = a.state_slots[b];
    float* S = a.state + (slot * a.H + h) * (int64_t)dk * dv;
    float* N = a.memory + (slot * a.H + h) * (int64_t)(dk + 1);
    const int jstep = dv_pad / CPL;
    float s[CPL][RPL];
#pragma unroll
    for (int c = 0; c < CPL; ++c)
#pragma unroll
        for (int r = 0; r < RPL; ++r) {
            const int i = qd * RPL + r, jc = j + c * jstep;
            s[c][r] = (!fresh && i < dk && jc < dv) ? S[(int64_t)i * dv + jc] : 0.f;
        }
    float nrow[4];  // rows tid, tid + nthreads, ... of n: dk <= 256, at least 64 threads
#pragma unroll
    for (int u = 0; u < 4; ++u) nrow[u] = (!fresh && tid + u * nthreads < dk) ? N[tid + u * nthreads] : 0.f;
    float m_run = fresh ? 0.f : N[dk];  // carried by wave 0
    // rows past dk and columns past dv of both buffers stay zero
    for (int e = tid; e < 2 * ts * ROW; e += nthreads) {
        qs[e] = 0.f;
        ks[e] = 0.f;
    }
    for (int e = tid; e < 2 * ts * dv_pad; e += nthreads) vs[e] = 0.f;
    // a thread's share of a stage is the same in every stage: where it comes from and goes to is worked out once
    T qr[PFQ], kr[PFQ], vr[PFV];
    int q_tt[PFQ], q_src[PFQ], q_dst[PFQ], v_tt[PFV], v_src[PFV];
#pragma unroll
    for (int u = 0; u < PFQ; ++u) {
        const int e = tid + u * nthreads;
        const int tt = e / dk, i = e - tt * dk;
        q_tt[u] = tt;
        q_src[u] = tt * (int)a.ld + h * dk + i;
        q_dst[u] = tt * ROW + (i / RPL) * SEG + (i % RPL);
    }
#pragma unroll
    for (int u = 0; u < PFV; ++u) {
        const int e = tid + u * nthreads;
        const int tt = e / dv_pad, c = e - tt * dv_pad;
        v_tt[u] = c < dv ? tt : 1 << 30;  // a column past the head's width is never fetched
        v_src[u] = tt * (int)a.ld + h * dv + c;
    }
    auto fetch = [&](int first, int n) {
        const T* base = proj + (int64_t)(t0 + first) * a.ld;
#pragma unroll
        for (int u = 0; u < PFQ; ++u)
            if (q_tt[u] < n) {
                qr[u] = base[a.q_col0 + q_src[u]];
                kr[u] = base[a.k_col0 + q_src[u]];
            }
#pragma unroll
        for (int u = 0; u < PFV; ++u)
            if (v_tt[u] < n) vr[u] = base[a.v_col0 + v_src[u]];
    };
    // ... into stage buffer `buf`, and the gates of those tokens by wave 0
    auto commit = [&](int first, int n, int buf) {
#pragma unroll
        for (int u = 0; u < PFQ; ++u)
            if (q_tt[u] < n) {
                qs[buf * ts * ROW + q_dst[u]] = (float)qr[u] * a.q_scale;
                ks[buf * ts * ROW + q_dst[u]] = (float)kr[u];
            }
#pragma unroll
        for (int u = 0; u < PFV; ++u)
            if (v_tt[u] < n) vs[buf * ts * dv_pad + tid + u * nthreads] = (float)vr[u];
        if (wave != 0) return;
        float li = 0.f, lf = 0.f, before = 0.f, after = 0.f;
        if (lane < n) log_gates(a, t0 + first + lane, h, li, lf);
        for (int tt = 0; tt < n; ++tt) {
            const float top = fmaxf(lane_value(lf, tt) + m_run, lane_value(li, tt));
            if (lane == tt) {
                before = m_run;
                after = top;
            }
            m_run = top;
        }
        if (lane < n) {
            gs[buf * ts + lane] = f32x2{expf(lf + before - after), expf(li - after)};
            fl[buf * ts + lane] = expf(-after);
        }
    };
    fetch(0, min(ts, qlen));
    __syncthreads();  // the buffers are cleared
    commit(0, min(ts, qlen), 0);
    __syncthreads();
    T* out = reinterpret_cast<T*>(a.out);
    int buf = 0;
    for (int base = 0; base < qlen; base += ts, buf ^= 1) {
        const int n = min(ts, qlen - base);
        const int n_next = min(ts, qlen - base - ts);
        if (n_next > 0) fetch(base + ts, n_next);
        const float* qb = qs + buf * ts * ROW + qd * SEG;
        const float* kb = ks + buf * ts * ROW + qd * SEG;
        const float* vb = vs + buf * ts * dv_pad + j;
        const f32x2* gb = gs + buf * ts;
#pragma unroll 1
        for (int tt = 0; tt < n; ++tt) {
            const f32x2 g = gb[tt];
            float vj[CPL], acc[CPL];
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
                vj[c] = vb[tt * dv_pad + c * jstep] * g[1];
                acc[c] = 0.f;
            }
#pragma unroll
            for (int r4 = 0; r4 < RPL; r4 += 4) {
                const f32x4 q4 = *reinterpret_cast<const f32x4*>(qb + tt * ROW + r4);
                const f32x4 k4 = *reinterpret_cast<const f32x4*>(kb + tt * ROW + r4);
#pragma unroll
                for (int u = 0; u < 4; ++u)
#pragma unroll
                    for (int c = 0; c < CPL; ++c) {
                        s[c][r4 + u] = fmaf(g[0], s[c][r4 + u], k4[u] * vj[c]);
                        acc[c] = fmaf(s[c][r4 + u], q4[u], acc[c]);
                    }
            }
#pragma unroll
            for (int c = 0; c < CPL; ++c) {
                const float t = sum_neighbours<LPC>(acc[c]);
                if (qd == 0) os[tt * dv_pad + j + c * jstep] = t;
            }
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int i = tid + u * nthreads;
            if (i < dk) {
                const int at = buf * ts * ROW + (i / RPL) * SEG + (i % RPL);
                for (int tt = 0; tt < n; ++tt) {
                    const f32x2 g = gb[tt];
                    nrow[u] = fmaf(g[0], nrow[u], g[1] * ks[at + tt * ROW]);
                    nq[tt * dk + i] = nrow[u] * qs[at + tt * ROW];
                }
            }
        }
        __syncthreads();
        for (int tt = wave; tt < n; tt += nw) {
            float d = 0.f, ss = 0.f;
            for (int i = lane; i < dk; i += 64) d += nq[tt * dk + i];
            for (int c = lane; c < dv; c += 64) ss += os[tt * dv_pad + c] * os[tt * dv_pad + c];
            d = wave_total(d);
            ss = wave_total(ss);
            const float den = fmaxf(fabsf(d), fl[buf * ts + tt]) + a.read_eps;
            const float rinv = 1.f / sqrtf(ss / (float)dv + a.eps * den * den);  // o / den, normed
            const int64_t t = t0 + base + tt;
            T* orow = out + t * a.ld_out + (int64_t)h * dv;
            for (int c = lane; c < dv; c += 64)
                orow[c] = (T)(os[tt * dv_pad + c] * rinv * a.gain[h * dv + c] * output_gate<T>(a, t, h * dv + c));
        }
        if (n_next > 0) commit(base + ts, n_next, buf ^ 1);
        __syncthreads();  // the outputs are out, the next stage is in
    }
#pragma unroll
    for (int c = 0; c < CPL; ++c)
#pragma unroll
        for (int r = 0; r < RPL; ++r) {
            const int i = qd * RPL + r, jc = j + c * jstep;
            if (i < dk && jc < dv) S[(int64_t)i * dv + jc] = s[c][r];
        }
#pragma unroll
    for (int u = 0; u < 4; ++u)
        if (tid + u * nthreads < dk) N[tid + u * nthreads] = nrow[u];
    if (tid == 0) N[dk] = m_run;
}

template <typename T, int RPL, int CPL, int LPC, int MAXT>
void launch_memory_as(MemoryArgs a, int64_t B, int64_t max_q_len, int cols, hipStream_t st) {
    a.dv_pad = cols;
    const int threads = LPC * cols / CPL;
    auto bytes = [&](int ts) {
        return ((size_t)4 * ts * LPC * (RPL + SEG_PAD) + (size_t)3 * ts * cols + ((size_t)ts * a.dk + 1) / 2 * 2 + (size_t)6 * ts) * sizeof(float);
    };
    int ts = MAX_TS;
    while (ts > 1 && (bytes(ts) > 140 * 1024 || ts >= 2 * max_q_len || ts * a.dk > PFQ * threads || ts * cols > PFV * threads)) ts >>= 1;
    a.ts = ts;
    const size_t lds = bytes(ts);
    if (lds > 48 * 1024)
        (void)hipFuncSetAttribute((const void*)matrix_memory_scan_kernel<T, RPL, CPL, LPC, MAXT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((matrix_memory_scan_kernel<T, RPL, CPL, LPC, MAXT>), dim3((unsigned)B, (unsigned)a.H), dim3(threads), lds, st, a);
}

// R4: rows per lane with four lanes per column.  Steps of one or two tokens are mostly the state's trip from and to memory: two
// columns per lane from 64 value channels on; longer runs spread a column over eight lanes where 1024 threads allow it.
template <typename T, int R4>
void launch_memory(const MemoryArgs& a, int64_t B, int64_t max_q_len, hipStream_t st) {
    const int pad16 = (a.dv + 15) / 16 * 16;
    if constexpr (R4 <= 32) {
        if (a.dv >= 64 && max_q_len <= 2) return launch_memory_as<T, R4, 2, 4, 512>(a, B, max_q_len, (a.dv + 31) / 32 * 32, st);
    }
    if constexpr (R4 >= 8) {
        if (max_q_len > 2 && 8 * pad16 <= 1024) return launch_memory_as<T, R4 / 2, 1, 8, 1024>(a, B, max_q_len, pad16, st);
    }
    launch_memory_as<T, R4, 1, 4, 1024>(a, B, max_q_len, pad16, st);
}

template <typename T>
void launch_memory_rows(const MemoryArgs& a, int64_t B, int64_t max_q_len, hipStream_t st) {
    if (a.dk <= 16) launch_memory<T, 4>(a, B, max_q_len, st);
    else if (a.dk <= 32) launch_memory<T, 8>(a, B, max_q_len, st);
    else if (a.dk <= 64) launch_memory<T, 16>(a, B, max_q_len, st);
    else if (a.dk <= 128) launch_memory<T, 32>(a, B, max_q_len, st);
    else launch_memory<T, 64>(a, B, max_q_len, st);
}

// ---- chunks on the matrix cores -----------------------------------------------------------------------------------------
constexpr int CT = 64;        // tokens per chunk
constexpr int TROW = CT + 8;  // LDS row of a channel-major operand: the chunk's tokens + 16 bytes

template <int KT, int VT> struct ChunkLds {
    static constexpr int DKP = KT * 32, DVP = VT * 32;
    static constexpr int QROW = DKP + 8;
    static constexpr int OROW = DVP + 4;
    bf16 qs[CT * QROW];      // [token][channel]
    bf16 ks[CT * QROW];
    bf16 kt[DKP * TROW];     // [channel][token], groups of 8 tokens swizzled (token_group)
    bf16 vt[DVP * TROW];
    bf16 ph[CT * TROW];      // weighted scores [t][s], high and low parts
    bf16 pl[CT * TROW];
    float o[2][CT * OROW];   // read-outs [t][value channel], a part from either half of the waves
    float gain[DVP];
    float n[DKP];
    struct Gates {
        float a[CT];         // a_s
        float top[CT];       // M_t
        float d0[CT];        // e^(m_0 - M_t)
        float fl[CT];        // e^(-m_t)
        float w[CT];         // e^(a_s - M_C)
        float keep;          // e^(m_0 - M_C)
        float pad[3];
    } gates[2];
    float part[2][CT];       // sums of the weighted scores over the chunk's first and second 32 tokens
    float nq[CT];            // n_0 . q_t
};

// where group g of 8 tokens of a channel lies in its row: the transposing stores of 8 neighbouring channel pieces then hit
// different banks, and so do the 16-byte reads of 8 neighbouring channels
__device__ __forceinline__ int token_group(int channel, int g) { return (g ^ (channel >> 3 & 7)) * 8; }

__device__ __forceinline__ void split_bf16(float x, bf16& hi, bf16& lo) {
    hi = (bf16)x;
    lo = (bf16)(x - (float)hi);
}

template <int KT, int VT>
__global__ __launch_bounds__(512) void matrix_memory_chunk_kernel(MemoryArgs a) {
    extern __shared__ __attribute__((aligned(16))) unsigned char raw[];
    using L = ChunkLds<KT, VT>;
    L& sm = *reinterpret_cast<L*>(raw);
    constexpr int QROW = L::QROW, OROW = L::OROW;
    const int b = blockIdx.x, h = blockIdx.y;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, c = lane & 31, half = lane >> 5;
    const int t0 = a.cu_q[b], qlen = a.cu_q[b + 1] - t0;
    if (qlen <= 0) return;
    const int dk = a.dk, dv = a.dv;
    const bool fresh = a.positions[t0] == 0;
    const bf16* proj = reinterpret_cast<const bf16*>(a.proj);
    const int64_t slot = a.state_slots[b];
    float* Sg = a.state + (slot * a.H + h) * (int64_t)dk * dv;
    float* Ng = a.memory + (slot * a.H + h) * (int64_t)(dk + 1);
    constexpr int KH = KT / 2, VH = VT / 2;  // KT, VT: 2 or 4
    const bool owner = (wave & 3) < VT;      // has value columns
    const int col = (wave & 3) * 32 + c, hw = wave >> 2;
    f32x16 S[KH];  // this wave's tiles of S, rows 32 KH hw and on; accumulator i of lane (c, half): row 8 (i / 4) + 4 half + i % 4 of the 32-row tile, column c
#pragma unroll
    for (int kt = 0; kt < KH; ++kt)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int r = (hw * KH + kt) * 32 + (i >> 2) * 8 + half * 4 + (i & 3);
            S[kt][i] = (owner && !fresh && r < dk && col < dv) ? Sg[(int64_t)r * dv + col] : 0.f;
        }
    if (tid < L::DKP) sm.n[tid] = (!fresh && tid < dk) ? Ng[tid] : 0.f;
    // tokens of the first half never see keys of the second: that corner of the weighted scores stays zero
    if (tid < 256) {
        const int at = (tid >> 3) * TROW + 32 + (tid & 7) * 4;
        *reinterpret_cast<bf16x4*>(sm.ph + at) = bf16x4{};
        *reinterpret_cast<bf16x4*>(sm.pl + at) = bf16x4{};
    }
    if (tid < L::DVP) sm.gain[tid] = tid < dv ? a.gain[h * dv + tid] : 0.f;
    // A thread's share of a chunk: 8 of every 64 channels of one token, eight neighbouring lanes fetch a line
    bf16x8 qr[KH], kr[KH], vr[VH], gr[VH];
    const int st_t = tid >> 3, st_p = tid & 7;
    auto fetch = [&](int base, int n) {
        const bf16* row = proj + (int64_t)(t0 + base + st_t) * a.ld + st_p * 8;
#pragma unroll
        for (int u = 0; u < KH; ++u) {
            const bool in = st_t < n && u * 64 + st_p * 8 < dk;
            qr[u] = in ? *reinterpret_cast<const bf16x8*>(row + a.q_col0 + h * dk + u * 64) : bf16x8{};
            kr[u] = in ? *reinterpret_cast<const bf16x8*>(row + a.k_col0 + h * dk + u * 64) : bf16x8{};
        }
#pragma unroll
        for (int u = 0; u < VH; ++u) {
            const bool in = st_t < n && u * 64 + st_p * 8 < dv;
            vr[u] = in ? *reinterpret_cast<const bf16x8*>(row + a.v_col0 + h * dv + u * 64) : bf16x8{};
        }
    };
    // one wave without score tiles makes the gates, one chunk ahead, and carries m
    float zi = 0.f, zf = 0.f, m_run = fresh ? 0.f : Ng[dk];
    auto fetch_gates = [&](int base, int n) {
        if (lane < n) {
            const float* z = a.gates + (int64_t)(t0 + base + lane) * a.ld_gates;
            zi = z[h];
            zf = z[a.H + h];
        }
    };
    const float inv_dv = 1.f / (float)dv;
    const float ib = a.i_bias ? a.i_bias[h] : 0.f, fb = a.f_bias ? a.f_bias[h] : 0.f;
    auto make_gates = [&](int n, typename L::Gates& g) {
        float li = -INFINITY, F = 0.f;  // tokens past the end keep everything and write nothing
        if (lane < n) {
            li = soft_capped(zi + ib, a.cap);
            F = log_sigmoid(soft_capped(zf + fb, a.cap));
        }
        F = scan_sum(F);
        const float as = li - F;
        const float top = fmaxf(scan_max(as), m_run);
        const float end = lane_value(top, 63);
        g.a[lane] = as;
        g.top[lane] = top;
        g.d0[lane] = expf(m_run - top);
        g.fl[lane] = expf(-(F + top));
        g.w[lane] = expf(as - end);
        if (lane == 0) g.keep = expf(m_run - end);
        m_run = lane_value(F, 63) + end;
    };
    fetch(0, min(CT, qlen));
    if (wave == 3) {
        fetch_gates(0, min(CT, qlen));
        make_gates(min(CT, qlen), sm.gates[0]);
    }
    int buf = 0;
    for (int base = 0; base < qlen; base += CT, buf ^= 1) {
        const int n = min(CT, qlen - base), n_next = min(CT, qlen - base - CT);
        const typename L::Gates& G = sm.gates[buf];
        // ---- the chunk into LDS
#pragma unroll
        for (int u = 0; u < KH; ++u) {
            const int ch = u * 64 + st_p * 8;
            *reinterpret_cast<bf16x8*>(sm.qs + st_t * QROW + ch) = qr[u];
            *reinterpret_cast<bf16x8*>(sm.ks + st_t * QROW + ch) = kr[u];
            bf16* dst = sm.kt + ch * TROW + token_group(ch, st_t >> 3) + (st_t & 7);
#pragma unroll
            for (int j = 0; j < 8; ++j) dst[j * TROW] = kr[u][j];
        }
#pragma unroll
        for (int u = 0; u < VH; ++u) {
            const int ch = u * 64 + st_p * 8;
            bf16* dst = sm.vt + ch * TROW + token_group(ch, st_t >> 3) + (st_t & 7);
#pragma unroll
            for (int j = 0; j < 8; ++j) dst[j * TROW] = vr[u][j];
        }
        if (wave == 3 && n_next > 0) fetch_gates(base + CT, n_next);
        __syncthreads();
        if (n_next > 0) fetch(base + CT, n_next);
        if (a.g_col0 >= 0 && st_t < n) {
            const bf16* g = proj + (int64_t)(t0 + base + st_t) * a.ld + a.g_col0 + h * dv + st_p * 8;
#pragma unroll
            for (int u = 0; u < VH; ++u) gr[u] = u * 64 + st_p * 8 < dv ? *reinterpret_cast<const bf16x8*>(g + u * 64) : bf16x8{};
        }
        // ---- weighted scores: waves 4, 5, 6 take the (s, t) tiles (0, 0), (0, 1), (1, 1), transposed (a lane has one t)
        if (wave >= 4 && wave < 7) {
            const int ts = (wave - 4) >> 1, tt = (wave - 3) >> 1;
            f32x16 P = {};
#pragma unroll
            for (int s = 0; s < KT * 2; ++s) {
                const bf16x8 x = *reinterpret_cast<const bf16x8*>(sm.ks + (ts * 32 + c) * QROW + s * 16 + half * 8);
                const bf16x8 y = *reinterpret_cast<const bf16x8*>(sm.qs + (tt * 32 + c) * QROW + s * 16 + half * 8);
                P = mfma32(x, y, P);
            }
            const int t = tt * 32 + c;
            const float top = G.top[t];
            float sum = 0.f;
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const int s0 = ts * 32 + g * 8 + half * 4;
                const f32x4 as = *reinterpret_cast<const f32x4*>(G.a + s0);
                bf16x4 hi, lo;
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const float p = s0 + i <= t ? P[g * 4 + i] * __expf(as[i] - top) : 0.f;
                    sum += p;
                    bf16 x, y;
                    split_bf16(p, x, y);
                    hi[i] = x;
                    lo[i] = y;
                }
                *reinterpret_cast<bf16x4*>(sm.ph + t * TROW + s0) = hi;
                *reinterpret_cast<bf16x4*>(sm.pl + t * TROW + s0) = lo;
            }
            sum += __shfl_xor(sum, 32, 64);
            if (half == 0) {
                sm.part[ts][t] = sum;
                if (wave == 4) sm.part[1][t] = 0.f;  // no later keys for the first 32 tokens
            }
        }
        // ---- what the state of the chunk's start gives: S_0^T q and n_0 . q
        f32x16 O[2] = {};
        if (owner) {
#pragma unroll
            for (int kt = 0; kt < KH; ++kt)
#pragma unroll
                for (int x = 0; x < 2; ++x) {
                    bf16x8 hi, lo;  // rows 16 x + 8 (j / 4) + 4 half + j % 4 of the tile: the A operand follows that order
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        bf16 u, v;
                        split_bf16(S[kt][x * 8 + j], u, v);
                        hi[j] = u;
                        lo[j] = v;
                    }
                    bf16x8 qa[2];
#pragma unroll
                    for (int tt = 0; tt < 2; ++tt) {
                        const bf16* q = sm.qs + (tt * 32 + c) * QROW + (hw * KH + kt) * 32 + x * 16 + half * 4;
                        const bf16x4 q0 = *reinterpret_cast<const bf16x4*>(q), q1 = *reinterpret_cast<const bf16x4*>(q + 8);
                        qa[tt] = __builtin_shufflevector(q0, q1, 0, 1, 2, 3, 4, 5, 6, 7);
                    }
                    O[0] = mfma32(qa[0], hi, O[0]);
                    O[1] = mfma32(qa[1], hi, O[1]);
                    O[0] = mfma32(qa[0], lo, O[0]);
                    O[1] = mfma32(qa[1], lo, O[1]);
                }
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int g = 0; g < 4; ++g) {
                    const f32x4 d = *reinterpret_cast<const f32x4*>(G.d0 + tt * 32 + g * 8 + half * 4);
#pragma unroll
                    for (int i = 0; i < 4; ++i) O[tt][g * 4 + i] *= d[i];
                }
        }
        {
            float d = 0.f;
#pragma unroll
            for (int u = 0; u < KH; ++u) {
                const int ch = u * 64 + st_p * 8;
                const bf16x8 q = *reinterpret_cast<const bf16x8*>(sm.qs + st_t * QROW + ch);
                const f32x4 n0 = *reinterpret_cast<const f32x4*>(sm.n + ch), n1 = *reinterpret_cast<const f32x4*>(sm.n + ch + 4);
#pragma unroll
                for (int i = 0; i < 4; ++i) d += (float)q[i] * n0[i] + (float)q[4 + i] * n1[i];
            }
            d = sum_neighbours<8>(d);
            if (st_p == 0) sm.nq[st_t] = d;
        }
        if (wave == 3 && n_next > 0) make_gates(n_next, sm.gates[buf ^ 1]);
        __syncthreads();
        // ---- the chunk's own keys and values; the state of its end
        const float keep = G.keep;
        if (owner) {
#pragma unroll
            for (int kt = 0; kt < KH; ++kt) S[kt] *= keep;
            // the state takes all keys; the read-outs of either half of the waves those of one half of the chunk
#pragma unroll
            for (int kk = 0; kk < 4; ++kk) {
                const int g8 = kk * 2 + half;
                const bf16x8 v = *reinterpret_cast<const bf16x8*>(sm.vt + col * TROW + token_group(col, g8));
                bf16x8 k[KH];
#pragma unroll
                for (int kt = 0; kt < KH; ++kt) {
                    const int row = (hw * KH + kt) * 32 + c;
                    k[kt] = *reinterpret_cast<const bf16x8*>(sm.kt + row * TROW + token_group(row, g8));
                }
                // values times their write weights
                const f32x4 w0 = *reinterpret_cast<const f32x4*>(G.w + kk * 16 + half * 8), w1 = *reinterpret_cast<const f32x4*>(G.w + kk * 16 + half * 8 + 4);
                bf16x8 hl[2];
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    bf16 x, y;
                    split_bf16((float)v[j] * (j < 4 ? w0[j & 3] : w1[j & 3]), x, y);
                    hl[0][j] = x;
                    hl[1][j] = y;
                }
#pragma unroll
                for (int part = 0; part < 2; ++part)
#pragma unroll
                    for (int kt = 0; kt < KH; ++kt) S[kt] = mfma32(k[kt], hl[part], S[kt]);
            }
#pragma unroll
            for (int x = 0; x < 2; ++x) {
                const int kk = hw * 2 + x;
                const bf16x8 v = *reinterpret_cast<const bf16x8*>(sm.vt + col * TROW + token_group(col, kk * 2 + half));
                bf16x8 p[2][2];
#pragma unroll
                for (int tt = 0; tt < 2; ++tt) {
                    const int at = (tt * 32 + c) * TROW + kk * 16 + half * 8;
                    p[tt][0] = *reinterpret_cast<const bf16x8*>(sm.ph + at);
                    p[tt][1] = *reinterpret_cast<const bf16x8*>(sm.pl + at);
                }
#pragma unroll
                for (int part = 0; part < 2; ++part) {
                    O[0] = mfma32(p[0][part], v, O[0]);
                    O[1] = mfma32(p[1][part], v, O[1]);
                }
            }
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int i = 0; i < 16; ++i) sm.o[hw][(tt * 32 + (i >> 2) * 8 + half * 4 + (i & 3)) * OROW + col] = O[tt][i];
        }
        {
            // rows of n: 16 / KT neighbouring lanes share one, each takes its tokens
            constexpr int SHARE = 16 / KT;
            const int i = tid / SHARE, part = tid % SHARE;
            float s = 0.f;
#pragma unroll
            for (int p = 0; p < KH; ++p) {
                const int g8 = part * KH + p;
                const bf16x8 k = *reinterpret_cast<const bf16x8*>(sm.kt + i * TROW + token_group(i, g8));
                const f32x4 w0 = *reinterpret_cast<const f32x4*>(G.w + g8 * 8), w1 = *reinterpret_cast<const f32x4*>(G.w + g8 * 8 + 4);
#pragma unroll
                for (int j = 0; j < 4; ++j) s += (float)k[j] * w0[j] + (float)k[4 + j] * w1[j];
            }
            s = sum_neighbours<SHARE>(s);
            if (part == 0) sm.n[i] = fmaf(sm.n[i], keep, s);
        }
        __syncthreads();
        // ---- normaliser, norm and gate: eight neighbouring lanes per token
        {
            const float nq = (sm.nq[st_t] * G.d0[st_t] + sm.part[0][st_t] + sm.part[1][st_t]) * a.q_scale;
            const float den = fmaxf(fabsf(nq), G.fl[st_t]) + a.read_eps;
            f32x4 v[VH * 2];
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < VH * 2; ++j) {
                const int at = st_t * OROW + (j >> 1) * 64 + st_p * 8 + (j & 1) * 4;
                v[j] = (*reinterpret_cast<const f32x4*>(sm.o[0] + at) + *reinterpret_cast<const f32x4*>(sm.o[1] + at)) * a.q_scale;
#pragma unroll
                for (int i = 0; i < 4; ++i) ss += v[j][i] * v[j][i];  // columns past dv are zero
            }
            ss = sum_neighbours<8>(ss);
            const float rinv = __builtin_amdgcn_rsqf(ss * inv_dv + a.eps * den * den);  // o / den, normed
            bf16* orow = reinterpret_cast<bf16*>(a.out) + (int64_t)(t0 + base + st_t) * a.ld_out + (int64_t)h * dv + st_p * 8;
#pragma unroll
            for (int u = 0; u < VH; ++u) {
                bf16x8 y;
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const float g = a.g_col0 >= 0 ? __builtin_amdgcn_rcpf(1.f + __expf(-(float)gr[u][i])) : 1.f;
                    y[i] = (bf16)(v[u * 2 + (i >> 2)][i & 3] * rinv * sm.gain[u * 64 + st_p * 8 + i] * g);
                }
                if (st_t < n && u * 64 + st_p * 8 < dv) *reinterpret_cast<bf16x8*>(orow + u * 64) = y;
            }
        }
        // no barrier here: what this part reads (o, nq, part, n, this buffer's gates) is written again only behind the barrier after the
        // next chunk's staging, and that staging touches only what the part before this one read (in front of the last barrier)
    }
    if (owner) {
#pragma unroll
        for (int kt = 0; kt < KH; ++kt)
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const int r = (hw * KH + kt) * 32 + (i >> 2) * 8 + half * 4 + (i & 3);
                if (r < dk && col < dv) Sg[(int64_t)r * dv + col] = S[kt][i];
            }
    }
    if (tid < dk) Ng[tid] = sm.n[tid];
    if (tid == 192) Ng[dk] = m_run;  // the gates' wave
}

template <int KT, int VT> void launch_chunks(const MemoryArgs& a, int64_t B, hipStream_t st) {
    constexpr size_t lds = sizeof(ChunkLds<KT, VT>);
    static_assert(lds <= 160 * 1024, "a chunk's operands fit the LDS of a compute unit");
    (void)hipFuncSetAttribute((const void*)matrix_memory_chunk_kernel<KT, VT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((matrix_memory_chunk_kernel<KT, VT>), dim3((unsigned)B, (unsigned)a.H), dim3(512), lds, st, a);
}

// runs from this length on are worth a chunk of 64 (a single token costs a whole one)
constexpr int64_t CHUNKS_FROM = 12;

bool chunks_ok(const MemoryArgs& a, int dtype) {
    auto al = [](const void* p, size_t n) { return ((uintptr_t)p % n) == 0; };
    return dtype == TGIS_BF16 && a.dk <= 128 && a.dv <= 128 && a.dk % 8 == 0 && a.dv % 8 == 0 && a.ld % 8 == 0 && a.q_col0 % 8 == 0 && a.k_col0 % 8 == 0 &&
           a.v_col0 % 8 == 0 && (a.g_col0 < 0 || a.g_col0 % 8 == 0) && a.ld_out % 8 == 0 && al(a.proj, 16) && al(a.out, 16);
}

}  // namespace

extern "C" int tgis_matrix_memory(const void* proj, int64_t ld, int64_t q_col0, int64_t k_col0, int64_t v_col0, int64_t g_col0,
                                  const float* gates, int64_t ld_gates, const float* i_bias, const float* f_bias, float cap, const float* gain,
                                  float* state, float* memory, const int32_t* state_slots, const int32_t* cu_seqlens_q,
                                  const int32_t* positions, void* out, int64_t ld_out, int64_t B, int64_t T, int64_t max_q_len, int H, int dk,
                                  int dv, float q_scale, float eps, float read_eps, int impl, int dtype, void* stream) {
    TGIS_CHECK_ARG(proj && gates && gain && state && memory && state_slots && cu_seqlens_q && positions && out, "tgis_matrix_memory: null tensor");
    TGIS_CHECK_ARG(H >= 1 && H <= 65535 && dk >= 1 && dk <= 256 && dv >= 1 && dv <= 256, "tgis_matrix_memory: heads of up to 256 x 256 (got %d x %d)", dk, dv);
    TGIS_CHECK_ARG(q_col0 >= 0 && k_col0 >= 0 && v_col0 >= 0 && ld >= q_col0 + (int64_t)H * dk && ld >= k_col0 + (int64_t)H * dk &&
                       ld >= v_col0 + (int64_t)H * dv && (g_col0 < 0 || ld >= g_col0 + (int64_t)H * dv) && ld_gates >= 2 * (int64_t)H &&
                       ld_out >= (int64_t)H * dv && max_q_len >= 1 && T >= 0 && ld <= (1 << 24),
                   "tgis_matrix_memory: bad strides");
    TGIS_CHECK_ARG(cap > 0.f && impl >= 0 && impl <= 2, "tgis_matrix_memory: cap > 0; impl 0 (auto), 1 (token by token), 2 (chunks)");
    TGIS_CHECK_ARG(dtype == TGIS_F16 || dtype == TGIS_BF16 || dtype == TGIS_F32, "tgis_matrix_memory: bad dtype");
    if (B == 0 || T == 0) return TGIS_OK;
    hipStream_t st = (hipStream_t)stream;
    TgisTimedScope timed(TGIS_OP_SCAN, st);
    const MemoryArgs a{proj, ld, q_col0, k_col0, v_col0, g_col0, gates, ld_gates, i_bias, f_bias, cap, gain, state, memory, state_slots,
                       cu_seqlens_q, positions, out, ld_out, H, dk, dv, q_scale, eps, read_eps, 0, 0};
    const bool can = chunks_ok(a, dtype);
    TGIS_CHECK_ARG(impl != 2 || can, "tgis_matrix_memory: chunks take bf16, dk and dv multiples of 8 up to 128, aligned operands");
    if (impl == 2 || (impl == 0 && can && max_q_len >= CHUNKS_FROM)) {
        if (dk <= 64 && dv <= 64) launch_chunks<2, 2>(a, B, st);
        else if (dk <= 64) launch_chunks<2, 4>(a, B, st);
        else if (dv <= 64) launch_chunks<4, 2>(a, B, st);
        else launch_chunks<4, 4>(a, B, st);
        TGIS_CHECK_LAUNCH();
        return TGIS_OK;
    }
    if (dtype == TGIS_F16) launch_memory_rows<f16>(a, B, max_q_len, st);
    else if (dtype == TGIS_BF16) launch_memory_rows<bf16>(a, B, max_q_len, st);
    else launch_memory_rows<float>(a, B, max_q_len, st);
    TGIS_CHECK_LAUNCH();
    return TGIS_OK;
}
