// Gated linear attention with a decay per key channel.  gfx950, wave64.
//
//   z_t = W_a2 a1_t + b,  alpha_t = sigmoid(z_t)^(1/tau)               (per key channel)
//   S_t = diag(alpha_t) S_(t-1) + k_t v_t^T,   o_t = S_t^T (scale q_t)
//   out_t = rmsnorm(o_t) * w * silu(g_t)                               (per head, over the value channels)
//
// Two forms of the same recurrence, both in fp32 throughout:
//   * row by row, a block per (head, sequence), the state in registers: decoding and short portions;
//   * in chunks, for prompts.  With b_t = sum of log2 alpha from the start of a sub-chunk of 16 rows to t,
//         o_t  = (q_t 2^b_t)^T S_0 + sum_{s<=t} A_ts v_s,    A_ts = sum_d q_td k_sd 2^(b_td - b_sd)
//         S_16 = diag(2^b_16) S_0 + sum_s (k_s 2^(b_16 - b_s)) v_s^T
//     every exponent is <= 0, so nothing overflows however strong the decay is.  Spans of GLA_SPAN sub-chunks
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
constexpr uint32_t GLA_SPAN = 4;         // sub-chunks of a span
constexpr uint32_t GLA_MAX_DIM = 256;    // of the chunked form

struct GlaParams {
    const void *q, *k, *v, *g, *a1;      // activations, row stride proj_stride
    const uint16_t *a2, *a2_bias, *norm_weight;
    float* state;                        // [slots, heads, dk, dv]
    const uint32_t* slots;               // slot of a sequence, nullptr = slot0 + sequence
    void* out;
    uint32_t proj_stride, out_stride, slot0;
    uint32_t heads, dk, dv, dv_count, rank, rows;
    float inv_tau, q_scale, eps;
    // scratch of the chunked form
    float *qd, *kd;                      // [sub, head, 16, dk]
    float* edge;                         // [sub, head, dk]        2^b_16
    float* att;                          // [sub, head, 16, 16]    A
    float* spans;                        // [span, head, dk, dv]
    float* span_decay;                   // [span, head, dk]
};

// log2(sigmoid(z)) / tau
__device__ __forceinline__ float gla_log2_decay(float z, float inv_tau) {
    const float l = log1pf(expf(-fabsf(z)));
    return -1.4426950408889634f * inv_tau * (z >= 0.0f ? l : l - z);
}

__device__ __forceinline__ float gla_silu(float x) { return x / (1.0f + expf(-x)); }

__device__ __forceinline__ void gla_bf8(const uint16_t* p, float* w) {
    const uint4 q = *reinterpret_cast<const uint4*>(p);
    act2_to_f32<ACT_BF16>(q.x, w[0], w[1]);
    act2_to_f32<ACT_BF16>(q.y, w[2], w[3]);
    act2_to_f32<ACT_BF16>(q.z, w[4], w[5]);
    act2_to_f32<ACT_BF16>(q.w, w[6], w[7]);
}

// ---- row by row -------------------------------------------------------------------------------------
// 512 threads: thread (column j, group c) owns the state rows c, c + groups, ... of column j; in registers when
// they are at most PER, else (PER = 0) in memory, where only this thread touches them.
template <int ACT, int PER>
__global__ __launch_bounds__(512) void gla_recurrent_kernel(GlaParams p) {
    extern __shared__ __attribute__((aligned(16))) float gla_lds[];
    const uint32_t tid = threadIdx.x, head = blockIdx.x, seq = blockIdx.y;
    const uint32_t dk = p.dk, dv = p.dv, groups = 512u / dv, j = tid % dv, c = tid / dv;
    const bool owner = c < groups;
    float* qs = gla_lds;
    float* ks = qs + dk;
    float* al = ks + dk;
    float* part = al + dk;               // [groups, dv]
    float* red = part + groups * dv;     // [8]
    float* a1s = red + 8;                // [rank]
    const uint32_t slot = p.slots ? p.slots[seq] : p.slot0 + seq;
    float* S = p.state + ((size_t)slot * p.heads + head) * dk * dv;
    float st[PER > 0 ? PER : 1];
    if (PER > 0 && owner) {
#pragma unroll
        for (int e = 0; e < PER; ++e) st[e] = S[(size_t)min(c + groups * e, dk - 1u) * dv + j];
    }
    const act_t<ACT>* a1p = static_cast<const act_t<ACT>*>(p.a1);
    for (uint32_t t = 0; t < p.rows; ++t) {
        const size_t row = (size_t)seq * p.rows + t;
        const size_t at = row * p.proj_stride;
        for (uint32_t r = tid; r < p.rank; r += 512u) a1s[r] = act_to_f32<ACT>(a1p[at + r]);
        const uint32_t jc = min(tid, dv - 1u);       // requested early, used at the end of the row
        const float gate = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.g)[at + head * dv + jc]);
        const float vj = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.v)[at + head * dv + j]);
        const float nw = bf16_to_f32(p.norm_weight[jc]);
        __syncthreads();
        for (uint32_t d = tid; d < dk; d += 512u) {
            const uint32_t ch = head * dk + d;
            float z = bf16_to_f32(p.a2_bias[ch]);
            for (uint32_t r = 0; r < p.rank; r += 8u) {
                float w[8];
                gla_bf8(p.a2 + (size_t)ch * p.rank + r, w);
#pragma unroll
                for (int u = 0; u < 8; ++u) z = fmaf(w[u], a1s[r + u], z);
            }
            qs[d] = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.q)[at + ch]) * p.q_scale;
            ks[d] = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.k)[at + ch]);
            al[d] = __builtin_amdgcn_exp2f(gla_log2_decay(z, p.inv_tau));
        }
        __syncthreads();
        if (owner) {
            float o = 0.0f;
            if (PER > 0) {
#pragma unroll
                for (int e = 0; e < PER; ++e) {
                    const uint32_t i = c + groups * e;
                    if (i < dk) {
                        st[e] = fmaf(al[i], st[e], ks[i] * vj);
                        o = fmaf(st[e], qs[i], o);
                    }
                }
            } else {
                for (uint32_t i = c; i < dk; i += groups) {
                    const float s = fmaf(al[i], S[(size_t)i * dv + j], ks[i] * vj);
                    S[(size_t)i * dv + j] = s;
                    o = fmaf(s, qs[i], o);
                }
            }
            part[c * dv + j] = o;
        }
        __syncthreads();
        float o = 0.0f;
        if (tid < dv)
            for (uint32_t e = 0; e < groups; ++e) o += part[e * dv + tid];
        const float ss = wave_sum_bcast(tid < dv ? o * o : 0.0f);
        if ((tid & 63u) == 0) red[tid >> 6] = ss;
        __syncthreads();
        float sum = 0.0f;
#pragma unroll
        for (int w = 0; w < 8; ++w) sum += red[w];
        if (tid < dv) {
            const float inv = 1.0f / sqrtf(sum / (float)p.dv_count + p.eps);
            static_cast<act_t<ACT>*>(p.out)[row * p.out_stride + head * dv + tid] = f32_to_act<ACT>(o * inv * nw * gla_silu(gate));
        }
    }
    if (PER > 0 && owner) {
#pragma unroll
        for (int e = 0; e < PER; ++e)
            if (c + groups * e < dk) S[(size_t)(c + groups * e) * dv + j] = st[e];
    }
}

// ---- chunked: gates, decayed operands and A of one (sub-chunk, head) ------------------------------------
template <int ACT>
__global__ __launch_bounds__(256) void gla_prep_kernel(GlaParams p) {
    extern __shared__ __attribute__((aligned(16))) float gla_lds[];
    const uint32_t tid = threadIdx.x, sub = blockIdx.x, head = blockIdx.y, dk = p.dk, ld = dk + 4u;
    float* qs = gla_lds;                 // [16][ld]
    float* ks = qs + 16u * ld;
    float* bs = ks + 16u * ld;
    float* a1s = bs + 16u * ld;          // [16][rank]
    const uint32_t t0 = sub * GLA_SUB, live = min(GLA_SUB, p.rows > t0 ? p.rows - t0 : 0u);
    for (uint32_t e = tid; e < 16u * p.rank; e += 256u) {
        const uint32_t t = e / p.rank, r = e % p.rank;
        a1s[e] = t < live ? act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.a1)[(size_t)(t0 + t) * p.proj_stride + r]) : 0.0f;
    }
    __syncthreads();
    const size_t cell = (size_t)sub * p.heads + head;
    for (uint32_t d = tid; d < dk; d += 256u) {
        const uint32_t ch = head * dk + d;
        float z[16], qv[16], kv[16];
        const float bias = bf16_to_f32(p.a2_bias[ch]);
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            const size_t at = (size_t)min(t0 + t, p.rows - 1u) * p.proj_stride + ch;
            qv[t] = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.q)[at]);
            kv[t] = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.k)[at]);
            z[t] = bias;
        }
        for (uint32_t r = 0; r < p.rank; r += 8u) {
            float w[8];
            gla_bf8(p.a2 + (size_t)ch * p.rank + r, w);
#pragma unroll
            for (int t = 0; t < 16; ++t)
#pragma unroll
                for (int u = 0; u < 8; ++u) z[t] = fmaf(w[u], a1s[t * p.rank + r + u], z[t]);
        }
        float b = 0.0f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            const bool on = (uint32_t)t < live;      // dead rows neither decay nor add
            b += on ? gla_log2_decay(z[t], p.inv_tau) : 0.0f;
            z[t] = b;
            qv[t] = on ? qv[t] * p.q_scale : 0.0f;
            kv[t] = on ? kv[t] : 0.0f;
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            qs[t * ld + d] = qv[t];
            ks[t * ld + d] = kv[t];
            bs[t * ld + d] = z[t];
            p.qd[(cell * 16u + t) * dk + d] = qv[t] * __builtin_amdgcn_exp2f(z[t]);
            p.kd[(cell * 16u + t) * dk + d] = kv[t] * __builtin_amdgcn_exp2f(b - z[t]);
        }
        p.edge[cell * dk + d] = __builtin_amdgcn_exp2f(b);
    }
    __syncthreads();
    const uint32_t t = tid >> 4, s = tid & 15u;
    float a = 0.0f;
    if (s <= t) {
        for (uint32_t d = 0; d < dk; d += 4u) {
            const gla_f4 q = *reinterpret_cast<const gla_f4*>(qs + t * ld + d), k = *reinterpret_cast<const gla_f4*>(ks + s * ld + d);
            const gla_f4 x = *reinterpret_cast<const gla_f4*>(bs + t * ld + d) - *reinterpret_cast<const gla_f4*>(bs + s * ld + d);
#pragma unroll
            for (int u = 0; u < 4; ++u) a = fmaf(q[u] * k[u], __builtin_amdgcn_exp2f(x[u]), a);
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
    for (uint32_t c = 0; c < GLA_SPAN; ++c) {
        const uint32_t sub = span * GLA_SPAN + c, t0 = sub * GLA_SUB;
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
            const float v = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.v)[(size_t)min(t, p.rows - 1u) * p.proj_stride + head * dv + col]);
            vb[ks] = t < p.rows ? v : 0.0f;
        }
        float gate[4];
        if (OUT) {
#pragma unroll
            for (int r = 0; r < 4; ++r)
                gate[r] = act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.g)[(size_t)min(t0 + 4u * g + r, p.rows - 1u) * p.proj_stride + head * dv + col]);
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
            if (c + 1u == GLA_SPAN) break;           // the state after the span came from the scan
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
    for (uint32_t c = 0; c < GLA_SPAN; ++c)
        if (span * GLA_SPAN + c < n_subs) d *= p.edge[(size_t)(span * GLA_SPAN + c) * p.heads * p.dk + at];
    p.span_decay[(size_t)span * p.heads * p.dk + at] = d;
}

}  // namespace nvmai
