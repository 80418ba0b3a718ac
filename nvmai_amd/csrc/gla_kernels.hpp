// Gated linear attention with a decay per key channel.  gfx950, wave64.
//
//   z_t = W_a2 a1_t + b,  alpha_t = sigmoid(z_t)^(1/tau)               (per key channel)
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T (scale q_t)
//   out_t = rmsnorm(o_t) * w * silu(g_t)                               (per head, over the value channels)
//
// Two forms of the same recurrence, both in fp32 throughout, from projections kept in 32 bits (the norm of a first token's
// output leaves little but the sign of q . k, which a rounding of q and k may turn):
//   * row by row, a block per (head, sequence), the state in registers: decoding and short portions;
//   * in chunks, for prompts.  With b_t = sum of log2 alpha from the start of a sub-chunk of 16 rows to t,
//         o_t  = (q_t 2^b_t)^T S_0 + sum_{s<=t} A_ts v_s,    A_ts = sum_d q_td k_sd 2^(b_td - b_sd)
//         S_16 = diag(2^b_16) S_0 + sum_s (k_s 2^(b_16 - b_s)) v_s^T
//     every exponent is <= 0, so nothing overflows however strong the decay is.  Spans of a few sub-chunks
//     first compute what they add to a zero state (all spans at once), a scan over the spans turns that into the
//     state each span starts from, and the spans then compute their outputs at once.  The products run on
//     v_mfma_f32_16x16x4_f32; the state of a span lives in the accumulators: register r of a tile in lane
//     (i, g) is S[16 tile + 4 g + r][i], which is a B operand of the next product as it stands when its four
//     k indices are read as the rows 4 g + r, g = 0 .. 3.
#pragma once

#include "common.hpp"

namespace nvmai {

typedef float gla_f4 __attribute__((ext_vector_type(4)));

constexpr uint32_t GLA_SUB = 16;         // rows of a sub-chunk
constexpr uint32_t GLA_MAX_DIM = 256;    // of the chunked form

struct GlaParams {
    const float *q, *k, *v, *g, *a1;     // projected rows in 32 bits, row stride proj_stride
    const uint16_t *a2, *a2_bias, *norm_weight;
    float* state;                        // [slots, heads, dk, dv]
    const uint32_t* slots;               // slot of a sequence, nullptr = slot0 + sequence
    void* out;
    uint32_t proj_stride, out_stride, slot0;
    uint32_t heads, dk, dv, dv_count, rank, rows;
    uint32_t span;                       // sub-chunks of a span (chunked form)
    float inv_tau, q_scale, eps;
    // scratch of the chunked form
    float *qd, *kd;                      // [sub, head, 16, dk]
    float* edge;                         // [sub, head, dk]        2^b_16
    float* att;                          // [sub, head, 16, 16]    A
    float* spans;                        // [span, head, dk, dv]
    float* span_decay;                   // [span, head, dk]
};

// log2(sigmoid(z)) / tau = -log2(1 + e^-z) / tau.  ln(1 + e) for 0 < e <= 1 is 2 atanh(u), u = e / (2 + e) <= 1/3, by its
// power series to u^13 (the next term is below 2e-8 of the sum).
__device__ __forceinline__ float gla_log2_decay(float z, float inv_tau) {
    const float e = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z));
    const float u = e * __builtin_amdgcn_rcpf(2.0f + e), w = u * u;
    float s = fmaf(w, 1.0f / 13.0f, 1.0f / 11.0f);
    s = fmaf(w, s, 1.0f / 9.0f);
    s = fmaf(w, s, 1.0f / 7.0f);
    s = fmaf(w, s, 1.0f / 5.0f);
    s = fmaf(w, s, 1.0f / 3.0f);
    const float l = 2.0f * fmaf(w * s, u, u);
    return -1.4426950408889634f * inv_tau * (z >= 0.0f ? l : l - z);
}

__device__ __forceinline__ float gla_silu(float x) { return x / (1.0f + expf(-x)); }

__device__ __forceinline__ void gla_unpack8(const uint4& q, float* w) {
    act2_to_f32<ACT_BF16>(q.x, w[0], w[1]);
    act2_to_f32<ACT_BF16>(q.y, w[2], w[3]);
    act2_to_f32<ACT_BF16>(q.z, w[4], w[5]);
    act2_to_f32<ACT_BF16>(q.w, w[6], w[7]);
}

// ---- row by row -------------------------------------------------------------------------------------
// NTH threads: thread (column j, group c) owns the state rows c PER .. c PER + PER - 1 of column j, in registers for the
// rows of the call (PER = 0: any number of them, in memory, where only this thread touches them).  Key channels past
// the last one have zero decay, key and query in LDS, so that no load or product stands under a condition; a row's
// operands are requested before the row ahead of it is finished, the first row's before the state.
template <int ACT, int PER, uint32_t NTH>
__global__ __launch_bounds__(NTH) void gla_recurrent_kernel(GlaParams p) {
    extern __shared__ __attribute__((aligned(16))) float gla_lds[];
    const uint32_t tid = threadIdx.x, head = blockIdx.x, seq = blockIdx.y;
    const uint32_t dk = p.dk, dv = p.dv, groups = NTH / dv, j = tid % dv, c = tid / dv;
    const uint32_t chans = PER > 0 ? groups * PER : dk;          // a multiple of 4
    const bool owner = c < groups;
    float* qs = gla_lds;
    float* ks = qs + chans;
    float* al = ks + chans;
    float* red = al + chans;             // [16]
    float* part = red + 16;              // [groups, dv]
    float* a1s = part + groups * dv;     // [rank]
    const uint32_t slot = p.slots ? p.slots[seq] : p.slot0 + seq;
    float* S = p.state + ((size_t)slot * p.heads + head) * dk * dv + j;
    const float *qp = p.q + head * dk, *kp = p.k + head * dk, *vp = p.v + head * dv, *gp = p.g + head * dv;
    const uint32_t dc = min(tid, dk - 1u), jc = min(tid, dv - 1u), rc = min(tid, p.rank - 1u), ch = head * dk + dc;
    float a1v, q0, k0, vj, gj;
    auto fetch = [&](uint32_t t) {
        const size_t at = ((size_t)seq * p.rows + t) * p.proj_stride;
        a1v = p.a1[at + rc];
        q0 = qp[at + dc];
        k0 = kp[at + dc];
        vj = vp[at + j];
        gj = gp[at + jc];
    };
    fetch(0);
    const uint16_t* a2 = p.a2 + (size_t)ch * p.rank;
    const uint4 w0 = *reinterpret_cast<const uint4*>(a2), w1 = *reinterpret_cast<const uint4*>(a2 + (p.rank > 8u ? 8u : 0u));
    const float b0 = bf16_to_f32(p.a2_bias[ch]), nw = bf16_to_f32(p.norm_weight[jc]);
    float st[PER > 0 ? PER : 1];
    if (PER > 0) {
#pragma unroll
        for (int e = 0; e < PER; ++e) st[e] = S[(size_t)min(c * PER + e, dk - 1u) * dv];
    }
    for (uint32_t t = 0; t < p.rows; ++t) {
        const size_t row = (size_t)seq * p.rows + t;
        if (tid < p.rank) a1s[tid] = a1v;
        __syncthreads();
        float z = b0, w[8];
        gla_unpack8(w0, w);
        {
            const gla_f4 x0 = *reinterpret_cast<const gla_f4*>(a1s), x1 = *reinterpret_cast<const gla_f4*>(a1s + 4);
#pragma unroll
            for (int u = 0; u < 4; ++u) z = fmaf(w[u], x0[u], z);
#pragma unroll
            for (int u = 0; u < 4; ++u) z = fmaf(w[4 + u], x1[u], z);
        }
        if (p.rank > 8u) {                           // uniform
            gla_unpack8(w1, w);
#pragma unroll
            for (int u = 0; u < 8; ++u) z = fmaf(w[u], a1s[8 + u], z);
            for (uint32_t r = 16u; r < p.rank; r += 8u) {
                gla_unpack8(*reinterpret_cast<const uint4*>(a2 + r), w);
#pragma unroll
                for (int u = 0; u < 8; ++u) z = fmaf(w[u], a1s[r + u], z);
            }
        }
        if (tid < chans) {
            const bool real = tid < dk;
            qs[tid] = real ? q0 * p.q_scale : 0.0f;
            ks[tid] = real ? k0 : 0.0f;
            al[tid] = real ? __builtin_amdgcn_exp2f(gla_log2_decay(z, p.inv_tau)) : 0.0f;
        }
        const float v = vj, gate = gj;
        fetch(min(t + 1u, p.rows - 1u));
        __syncthreads();
        float o = 0.0f;
        if (PER > 0) {
            const uint32_t c0 = min(c, groups - 1u) * PER;
#pragma unroll
            for (int e = 0; e < PER; e += 4) {
                const gla_f4 a = *reinterpret_cast<const gla_f4*>(al + c0 + e), k = *reinterpret_cast<const gla_f4*>(ks + c0 + e);
                const gla_f4 q = *reinterpret_cast<const gla_f4*>(qs + c0 + e);
#pragma unroll
                for (int u = 0; u < 4; ++u) {
                    st[e + u] = fmaf(a[u], st[e + u], k[u] * v);
                    o = fmaf(st[e + u], q[u], o);
                }
            }
        } else if (owner) {
            for (uint32_t i = c; i < dk; i += groups) {
                const float s = fmaf(al[i], S[(size_t)i * dv], ks[i] * v);
                S[(size_t)i * dv] = s;
                o = fmaf(s, qs[i], o);
            }
        }
        if (owner) part[c * dv + j] = o;
        __syncthreads();
        o = 0.0f;
        for (uint32_t e0 = 0; e0 < groups; e0 += 8u) {
            float x[8];
#pragma unroll
            for (int e = 0; e < 8; ++e) x[e] = part[min(e0 + e, groups - 1u) * dv + jc];
#pragma unroll
            for (int e = 0; e < 8; ++e) o += e0 + e < groups ? x[e] : 0.0f;
        }
        const float ss = wave_sum_bcast(tid < dv ? o * o : 0.0f);
        if ((tid & 63u) == 0) red[tid >> 6] = ss;
        __syncthreads();
        gla_f4 sum = *reinterpret_cast<const gla_f4*>(red);
#pragma unroll
        for (uint32_t x = 4; x < NTH / 64; x += 4) sum += *reinterpret_cast<const gla_f4*>(red + x);
        if (tid < dv) {
            const float inv = 1.0f / sqrtf(((sum[0] + sum[1]) + (sum[2] + sum[3])) / (float)p.dv_count + p.eps);
            static_cast<act_t<ACT>*>(p.out)[row * p.out_stride + head * dv + tid] = f32_to_act<ACT>(o * inv * nw * gla_silu(gate));
        }
    }
    if (PER > 0 && owner) {
#pragma unroll
        for (int e = 0; e < PER; ++e)
            if (c * PER + e < dk) S[(size_t)(c * PER + e) * dv] = st[e];
    }
}

// ---- chunked: gates, decayed operands and A of one (sub-chunk, head) ------------------------------------
// Two threads per key channel, eight rows each.  A = (q 2^b) (k 2^-b)^T on the matrix cores where no channel decays by
// more than 2^-GLA_SAFE within the sub-chunk (every factor then is far from overflow); pair by pair with the
// exponent of the difference otherwise.
constexpr float GLA_SAFE = 60.0f;

__global__ __launch_bounds__(256) void gla_prep_kernel(GlaParams p) {
    extern __shared__ __attribute__((aligned(16))) float gla_lds[];
    const uint32_t tid = threadIdx.x, sub = blockIdx.x, head = blockIdx.y, dk = p.dk, ld = dk + 4u;
    float* qs = gla_lds;                 // [16][ld]
    float* ks = qs + 16u * ld;
    float* bs = ks + 16u * ld;
    float* tot = bs + 16u * ld;          // [2][dk]: the decay of each half
    float* red = tot + 2u * dk;          // [4][256]
    float* a1s = red + 1024u;            // [16][rank]
    const uint32_t t0 = sub * GLA_SUB, live = min(GLA_SUB, p.rows > t0 ? p.rows - t0 : 0u);
    for (uint32_t e = tid; e < 16u * p.rank; e += 256u) {
        const uint32_t t = e / p.rank, r = e % p.rank;
        a1s[e] = t < live ? p.a1[(size_t)(t0 + t) * p.proj_stride + r] : 0.0f;
    }
    const size_t cell = (size_t)sub * p.heads + head;
    __syncthreads();
    bool strong = false;
    for (uint32_t u = tid; u < 2u * dk; u += 256u) {
        const uint32_t half = u >= dk ? 1u : 0u, d = u - half * dk, ch = head * dk + d;
        float z[8], qv[8], kv[8];
        const float bias = bf16_to_f32(p.a2_bias[ch]);
#pragma unroll
        for (int t = 0; t < 8; ++t) {
            const size_t at = (size_t)min(t0 + 8u * half + t, p.rows - 1u) * p.proj_stride + ch;
            qv[t] = p.q[at];
            kv[t] = p.k[at];
            z[t] = bias;
        }
        for (uint32_t r = 0; r < p.rank; r += 8u) {
            float w[8];
            gla_unpack8(*reinterpret_cast<const uint4*>(p.a2 + (size_t)ch * p.rank + r), w);
#pragma unroll
            for (int t = 0; t < 8; ++t)
#pragma unroll
                for (int e = 0; e < 8; ++e) z[t] = fmaf(w[e], a1s[(8u * half + t) * p.rank + r + e], z[t]);
        }
        float b = 0.0f;
#pragma unroll
        for (int t = 0; t < 8; ++t) {
            const uint32_t row = 8u * half + t;
            const bool on = row < live;              // dead rows neither decay nor add
            b += on ? gla_log2_decay(z[t], p.inv_tau) : 0.0f;
            qs[row * ld + d] = on ? qv[t] * p.q_scale : 0.0f;
            ks[row * ld + d] = on ? kv[t] : 0.0f;
            bs[row * ld + d] = b;
        }
        tot[half * dk + d] = b;
        strong = strong || b < -0.5f * GLA_SAFE;
    }
    const bool pairs = __syncthreads_or(strong);
    for (uint32_t u = tid; u < 2u * dk; u += 256u) {
        const uint32_t half = u >= dk ? 1u : 0u, d = u - half * dk;
        const float off = half ? tot[d] : 0.0f, last = tot[d] + tot[dk + d];
#pragma unroll
        for (int t = 0; t < 8; ++t) {
            const uint32_t row = 8u * half + t, at = row * ld + d;
            const float b = off + bs[at], q = qs[at], k = ks[at], qd = q * __builtin_amdgcn_exp2f(b);
            p.qd[(cell * 16u + row) * dk + d] = qd;
            p.kd[(cell * 16u + row) * dk + d] = k * __builtin_amdgcn_exp2f(last - b);
            if (pairs) {
                bs[at] = b;
            } else {
                qs[at] = qd;
                ks[at] = k * __builtin_amdgcn_exp2f(-b);
            }
        }
        if (half == 0u) p.edge[cell * dk + d] = __builtin_amdgcn_exp2f(last);
    }
    __syncthreads();
    const uint32_t t = tid >> 4, s = tid & 15u;
    if (!pairs) {
        const uint32_t lane = tid & 63u, wave = tid >> 6, i = lane & 15u, g = lane >> 4;
        gla_f4 acc = gla_f4{0.0f, 0.0f, 0.0f, 0.0f};
        for (uint32_t st = wave; st < dk / 4u; st += 4u)
            acc = __builtin_amdgcn_mfma_f32_16x16x4f32(qs[i * ld + 4u * st + g], ks[i * ld + 4u * st + g], acc, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) red[wave * 256u + (4u * g + r) * 16u + i] = acc[r];
        __syncthreads();
        p.att[cell * 256u + tid] = s <= t ? (red[tid] + red[256u + tid]) + (red[512u + tid] + red[768u + tid]) : 0.0f;
        return;
    }
    float a = 0.0f;
    if (s <= t) {
        for (uint32_t d = 0; d < dk; d += 4u) {
            const gla_f4 q = *reinterpret_cast<const gla_f4*>(qs + t * ld + d), k = *reinterpret_cast<const gla_f4*>(ks + s * ld + d);
            const gla_f4 x = *reinterpret_cast<const gla_f4*>(bs + t * ld + d) - *reinterpret_cast<const gla_f4*>(bs + s * ld + d);
#pragma unroll
            for (int e = 0; e < 4; ++e) a = fmaf(q[e] * k[e], __builtin_amdgcn_exp2f(x[e]), a);
        }
    }
    p.att[cell * 256u + tid] = a;
}

// ---- chunked: a span's sub-chunks in order ---------------------------------------------------------------
// Wave w owns the value columns 16 w .. 16 w + 15.  OUT = false: from a zero state, the span's own contribution
// goes to spans / span_decay.  OUT = true: from the state in spans, the outputs.
template <int ACT, int KT, bool OUT>
__global__ __launch_bounds__(1024) void gla_span_kernel(GlaParams p) {
    constexpr uint32_t KR = 16u * KT, KLD = KR + 16u, QLD = KR + 4u;
    __shared__ __attribute__((aligned(16))) float kds[16 * KLD];
    __shared__ __attribute__((aligned(16))) float qds[OUT ? 16 * QLD : 4];
    __shared__ __attribute__((aligned(16))) float es[KR];
    __shared__ float as[OUT ? 16 * 17 : 1];
    __shared__ float ssq[OUT ? 16 * 16 : 1];
    const uint32_t tid = threadIdx.x, nthr = blockDim.x, lane = tid & 63u, wave = tid >> 6, i = lane & 15u, g = lane >> 4;
    const uint32_t span = blockIdx.x, head = blockIdx.y, dk = p.dk, dv = p.dv, waves = nthr >> 6;
    const uint32_t col = 16u * wave + i;
    const size_t cell_s = (size_t)span * p.heads + head;
    float* S = p.spans + cell_s * dk * dv;
    gla_f4 acc[KT];
#pragma unroll
    for (int t = 0; t < KT; ++t) {
        acc[t] = gla_f4{0.0f, 0.0f, 0.0f, 0.0f};
        if (OUT) {
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const uint32_t row = 16u * t + 4u * g + r;
                if (row < dk) acc[t][r] = S[(size_t)row * dv + col];
            }
        }
    }
    for (uint32_t c = 0; c < p.span; ++c) {
        const uint32_t sub = span * p.span + c, t0 = sub * GLA_SUB;
        if (t0 >= p.rows) break;                     // uniform
        const size_t cell = (size_t)sub * p.heads + head;
        __syncthreads();
        for (uint32_t e = tid; e < 16u * KR / 4u; e += nthr) {
            const uint32_t t = e / (KR / 4u), d = (e % (KR / 4u)) * 4u;
            const gla_f4 zero = gla_f4{0.0f, 0.0f, 0.0f, 0.0f};
            const size_t at = (cell * 16u + t) * dk + d;
            *reinterpret_cast<gla_f4*>(kds + t * KLD + d) = d < dk ? *reinterpret_cast<const gla_f4*>(p.kd + at) : zero;
            if (OUT) *reinterpret_cast<gla_f4*>(qds + t * QLD + d) = d < dk ? *reinterpret_cast<const gla_f4*>(p.qd + at) : zero;
        }
        for (uint32_t d = tid; d < KR; d += nthr) es[d] = d < dk ? p.edge[cell * dk + d] : 0.0f;
        if (OUT)
            for (uint32_t e = tid; e < 256u; e += nthr) as[(e >> 4) * 17u + (e & 15u)] = p.att[cell * 256u + e];
        float vb[4];                                 // B operand: row 4 ks + g, this lane's column
#pragma unroll
        for (int ks = 0; ks < 4; ++ks) {
            const uint32_t t = t0 + 4u * ks + g;
            const float v = p.v[(size_t)min(t, p.rows - 1u) * p.proj_stride + head * dv + col];
            vb[ks] = t < p.rows ? v : 0.0f;
        }
        float gate[4];
        if (OUT) {
#pragma unroll
            for (int r = 0; r < 4; ++r)
                gate[r] = p.g[(size_t)min(t0 + 4u * g + r, p.rows - 1u) * p.proj_stride + head * dv + col];
        }
        __syncthreads();
        if (OUT) {
            gla_f4 o0 = gla_f4{0.0f, 0.0f, 0.0f, 0.0f}, o1 = o0;
#pragma unroll
            for (int t = 0; t < KT; ++t) {
                const gla_f4 q = *reinterpret_cast<const gla_f4*>(qds + i * QLD + 16 * t + 4u * g);
                o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(q[0], acc[t][0], o0, 0, 0, 0);
                o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(q[1], acc[t][1], o1, 0, 0, 0);
                o0 = __builtin_amdgcn_mfma_f32_16x16x4f32(q[2], acc[t][2], o0, 0, 0, 0);
                o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(q[3], acc[t][3], o1, 0, 0, 0);
            }
#pragma unroll
            for (int ks = 0; ks < 4; ++ks) o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(as[i * 17u + 4u * ks + g], vb[ks], o1, 0, 0, 0);
            o0 += o1;                                // o0[r]: row 4 g + r, this lane's column
            float sq[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) sq[r] = seg_reduce_sum<16>(o0[r] * o0[r]);
            if (i == 0) {
#pragma unroll
                for (int r = 0; r < 4; ++r) ssq[wave * 16u + 4u * g + r] = sq[r];
            }
            __syncthreads();
            const float nw = bf16_to_f32(p.norm_weight[col]);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                float sum = 0.0f;
                for (uint32_t w = 0; w < waves; ++w) sum += ssq[w * 16u + 4u * g + r];
                const float inv = 1.0f / sqrtf(sum / (float)p.dv_count + p.eps);
                const uint32_t t = t0 + 4u * g + r;
                if (t < p.rows)
                    static_cast<act_t<ACT>*>(p.out)[(size_t)t * p.out_stride + head * dv + col] = f32_to_act<ACT>(o0[r] * inv * nw * gla_silu(gate[r]));
            }
            if (c + 1u == p.span) break;           // the state after the span came from the scan
        }
#pragma unroll
        for (int t = 0; t < KT; ++t) {
            const gla_f4 e = *reinterpret_cast<const gla_f4*>(es + 16 * t + 4u * g);
            acc[t] *= e;
#pragma unroll
            for (int ks = 0; ks < 4; ++ks)
                acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(kds[(4u * ks + g) * KLD + 16 * t + i], vb[ks], acc[t], 0, 0, 0);
        }
    }
    if (OUT) return;
#pragma unroll
    for (int t = 0; t < KT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t row = 16u * t + 4u * g + r;
            if (row < dk) S[(size_t)row * dv + col] = acc[t][r];
        }
}

// spans: each span's own contribution -> the state it starts from; the sequence's state ends after the last span.
__global__ __launch_bounds__(256) void gla_scan_kernel(GlaParams p, uint32_t n_spans) {
    constexpr int AHEAD = 8;
    const uint32_t per_head = p.dk * p.dv / 4u, at = blockIdx.x * 256u + threadIdx.x, head = blockIdx.y;
    if (at >= per_head) return;
    const uint32_t row = at * 4u / p.dv;
    gla_f4* state = reinterpret_cast<gla_f4*>(p.state + ((size_t)p.slot0 * p.heads + head) * p.dk * p.dv) + at;
    gla_f4* own = reinterpret_cast<gla_f4*>(p.spans + (size_t)head * p.dk * p.dv) + at;
    const size_t step = (size_t)p.heads * per_head;
    const float* dec = p.span_decay + (size_t)head * p.dk + row;
    const size_t dstep = (size_t)p.heads * p.dk;
    gla_f4 S = *state;
    for (uint32_t n0 = 0; n0 < n_spans; n0 += AHEAD) {
        gla_f4 add[AHEAD];
        float d[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; ++u) {
            const uint32_t n = min(n0 + u, n_spans - 1u);
            add[u] = own[n * step];
            d[u] = dec[n * dstep];
        }
#pragma unroll
        for (int u = 0; u < AHEAD; ++u)
            if (n0 + u < n_spans) {
                own[(n0 + u) * step] = S;
                S = S * d[u] + add[u];
            }
    }
    *state = S;
}

// the decay of a whole span: the product of its sub-chunks'
__global__ __launch_bounds__(256) void gla_span_decay_kernel(GlaParams p, uint32_t n_subs) {
    const uint32_t at = blockIdx.x * 256u + threadIdx.x, span = blockIdx.y;
    if (at >= p.heads * p.dk) return;
    float d = 1.0f;
    for (uint32_t c = 0; c < p.span; ++c)
        if (span * p.span + c < n_subs) d *= p.edge[(size_t)(span * p.span + c) * p.heads * p.dk + at];
    p.span_decay[(size_t)span * p.heads * p.dk + at] = d;
}

}  // namespace nvmai
