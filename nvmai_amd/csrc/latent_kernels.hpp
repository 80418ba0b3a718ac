// Latent attention: keys and values are linear images of one cached latent per position, plus one rotated key part
// that all heads share.  gfx950, wave64.
//
//   score(h, i, j) = scale * (q_n(h, i) . W_uk(h) c_j + q_r(h, i) . k_r(j)),   window: 0 <= i - j < window
//   out(h, i)      = sigmoid(gate(h, i)) * W_uv(h) sum_j softmax_j(score) c_j
//
// A cache row holds [c | rotated key part | zeros], row stride `row_stride`, in the activation type or (CT) in BF16 beside
// 32-bit activations.  Two forms of the same sum:
//   * absorbed, for decoding and short portions: q_n is taken through W_uk(h)^T once, every head then reads the
//     latents themselves (each cache row is fetched once per sixteen heads), W_uv(h) is applied to the sum;
//   * expanded, for prompts: keys and values of the range are formed by two matrix products, then flash attention.
#pragma once

#include "rows.hpp"

namespace nvmai {

typedef __bf16 la_b8 __attribute__((ext_vector_type(8)));
typedef float la_f4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ la_f4 la_mfma(const uint4& a, const uint4& b, la_f4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(la_b8, a), __builtin_bit_cast(la_b8, b), c, 0, 0, 0);
}

// Two floats rounded to BF16 (nearest even) in one dword: one hardware conversion.
typedef float la_f2 __attribute__((ext_vector_type(2)));
typedef __bf16 la_b2 __attribute__((ext_vector_type(2)));
__device__ __forceinline__ uint32_t la_pack2(float lo, float hi) {
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(la_f2{lo, hi}, la_b2));
}

constexpr float LA_LOG2E = 1.4426950408889634f;
constexpr float LA_NONE = -1e30f;        // maximum of no scores

struct LatentCache {
    void* base;
    uint64_t slot_stride;    // elements
    uint32_t row_stride, capacity;
};

__device__ __forceinline__ float la_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// ---- after the down projections: both latents normed, the key part rotated, the cache row written ---------
struct LatentEpilogueParams {
    const void* proj;                    // [rows, proj_stride]: [W_dq h | W_dkv h: latent, rotated part]
    const uint16_t *q_norm, *kv_norm;    // readable up to the counts rounded up to 8
    const double* inv_freq;              // [rot_dims / 2]
    void* cq;                            // [rows, cq_stride]
    SeqRows rows;
    LatentCache cache;
    uint32_t proj_stride, q_at, kv_at, rot_at, cq_stride, q_count, rank_count, rank, rot_dim, rot_dims;
    float eps;
};

// Eight activations.
template <int ACT>
__device__ __forceinline__ void la_load8(const act_t<ACT>* p, float* v) {
    if constexpr (ACT == ACT_FP32) {
        const la_f4 a = reinterpret_cast<const la_f4*>(p)[0], b = reinterpret_cast<const la_f4*>(p)[1];
#pragma unroll
        for (int e = 0; e < 4; ++e) { v[e] = a[e]; v[4 + e] = b[e]; }
    } else {
        const uint4 q = *reinterpret_cast<const uint4*>(p);
        act2_to_f32<ACT>(q.x, v[0], v[1]);
        act2_to_f32<ACT>(q.y, v[2], v[3]);
        act2_to_f32<ACT>(q.z, v[4], v[5]);
        act2_to_f32<ACT>(q.w, v[6], v[7]);
    }
}

template <int ACT>
__device__ __forceinline__ void la_store8(act_t<ACT>* p, const float* v) {
    if constexpr (ACT == ACT_FP32) {
        reinterpret_cast<la_f4*>(p)[0] = la_f4{v[0], v[1], v[2], v[3]};
        reinterpret_cast<la_f4*>(p)[1] = la_f4{v[4], v[5], v[6], v[7]};
    } else {
        uint4 q;
        q.x = f32_to_act<ACT>(v[0]) | ((uint32_t)f32_to_act<ACT>(v[1]) << 16);
        q.y = f32_to_act<ACT>(v[2]) | ((uint32_t)f32_to_act<ACT>(v[3]) << 16);
        q.z = f32_to_act<ACT>(v[4]) | ((uint32_t)f32_to_act<ACT>(v[5]) << 16);
        q.w = f32_to_act<ACT>(v[6]) | ((uint32_t)f32_to_act<ACT>(v[7]) << 16);
        *reinterpret_cast<uint4*>(p) = q;
    }
}

// Both latents in pieces of eight elements, NP per thread, in registers between the sums and the stores; every load
// (norm weights and rotation included) is issued before the first sum.  Elements past a latent's count are zero in proj.
template <int ACT, int CT, int NP>
__global__ __launch_bounds__(256) void latent_epilogue_kernel(LatentEpilogueParams p) {
    __shared__ float lds[8];
    const uint32_t row = blockIdx.x, tid = threadIdx.x;
    const act_t<ACT>* proj = static_cast<const act_t<ACT>*>(p.proj) + (size_t)row * p.proj_stride;
    const uint32_t position = p.rows.position_of(row);
    act_t<CT>* out = static_cast<act_t<CT>*>(p.cache.base) + (size_t)p.rows.slot_of(row) * p.cache.slot_stride +
                      (size_t)(position % p.cache.capacity) * p.cache.row_stride;
    act_t<ACT>* cq = static_cast<act_t<ACT>*>(p.cq) + (size_t)row * p.cq_stride;
    const uint32_t qp = (p.q_count + 7u) / 8u, kp = (p.rank_count + 7u) / 8u, pieces = qp + kp;
    float v[NP][8];
    uint4 w[NP];
#pragma unroll
    for (int n = 0; n < NP; ++n) {
        const uint32_t u = min(tid + 256u * n, pieces - 1u);
        la_load8<ACT>(proj + (u < qp ? p.q_at + 8u * u : p.kv_at + 8u * (u - qp)), v[n]);
        w[n] = *reinterpret_cast<const uint4*>(u < qp ? p.q_norm + 8u * u : p.kv_norm + 8u * (u - qp));
    }
    // the rope part, by the last threads (the first have the longest lists of pieces)
    const uint32_t half = p.rot_dims / 2u;
    for (uint32_t j = 255u - tid; j < p.rot_dim; j += 256u) {
        if (j < half) {
            float c, s;
            position_angle(position, p.inv_freq[j], c, s);
            const float a = act_to_f32<ACT>(proj[p.rot_at + j]), b = act_to_f32<ACT>(proj[p.rot_at + half + j]);
            out[p.rank + j] = f32_to_act<CT>(a * c - b * s);
            out[p.rank + half + j] = f32_to_act<CT>(b * c + a * s);
        } else if (j >= p.rot_dims) {
            out[p.rank + j] = f32_to_act<CT>(act_to_f32<ACT>(proj[p.rot_at + j]));
        }
    }
    float qs = 0.0f, ks = 0.0f;
#pragma unroll
    for (int n = 0; n < NP; ++n) {
        const uint32_t u = tid + 256u * n;
        float s = 0.0f;
#pragma unroll
        for (int e = 0; e < 8; ++e) s = fmaf(v[n][e], v[n][e], s);
        qs += u < qp ? s : 0.0f;
        ks += u >= qp && u < pieces ? s : 0.0f;
    }
    qs = wave_sum_bcast(qs);
    ks = wave_sum_bcast(ks);
    if ((tid & 63u) == 0) { lds[tid >> 6] = qs; lds[4 + (tid >> 6)] = ks; }
    __syncthreads();
    const float qi = 1.0f / sqrtf(((lds[0] + lds[1]) + (lds[2] + lds[3])) / (float)p.q_count + p.eps);
    const float ki = 1.0f / sqrtf(((lds[4] + lds[5]) + (lds[6] + lds[7])) / (float)p.rank_count + p.eps);
#pragma unroll
    for (int n = 0; n < NP; ++n) {
        const uint32_t u = tid + 256u * n;
        if (u >= pieces) break;
        const float inv = u < qp ? qi : ki;
        float f[8];
        act2_to_f32<ACT_BF16>(w[n].x, f[0], f[1]);
        act2_to_f32<ACT_BF16>(w[n].y, f[2], f[3]);
        act2_to_f32<ACT_BF16>(w[n].z, f[4], f[5]);
        act2_to_f32<ACT_BF16>(w[n].w, f[6], f[7]);
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] *= v[n][e] * inv;
        if (u < qp) la_store8<ACT>(cq + 8u * u, f);
        else la_store8<CT>(out + 8u * (u - qp), f);
    }
}

struct LatentAttnParams {
    const void* q;                       // [rows, q_stride]: head by head [nope | rot], not yet rotated
    const void* gate;                    // [rows, gate_stride]: one logit per head, nullptr = no gate
    const uint16_t *uk, *uv;             // [heads * nope, rank], [heads * vdim, rank] BF16
    const double* inv_freq;
    SeqRows rows;
    LatentCache cache;
    void* out;                           // [rows, out_stride]: head by head [vdim]
    uint32_t q_stride, gate_stride, out_stride, n_rows, heads, nope, rot, vdim, rank, rot_dims, window;
    float scale_log2;                    // scale * log2(e)
    // absorbed form
    void* qa;                            // [rows, heads, row_stride]
    float *part_o, *part_m, *part_l;     // [rows, heads, splits, rank], [rows, heads, splits] x 2
    uint32_t splits, split_keys;
    // expanded form
    void *lat, *kn, *v;                  // [nk_pad, row_stride], [nk_pad, kn_stride], V (or V^T) rows of v_stride
    uint32_t nk, nk_pad, key0;           // keys of the call, the position of the first
    uint32_t kn_stride, v_stride;
};

// ---- absorbed: q_n -> W_uk(h)^T q_n, q_r rotated ----------------------------------------------------
// A block per (head, row, 128 latent dims): sixteen lanes cover the latents in pieces of eight, sixteen groups of
// lanes split the rows of W_uk(h).
template <int ACT, int CT>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentAttnParams p) {
    extern __shared__ __attribute__((aligned(16))) float la_lds[];
    __shared__ __attribute__((aligned(16))) float part[16][132];
    const uint32_t head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, piece = tid & 15u, group = tid >> 4;
    float* qs = la_lds;                  // [nope]
    const act_t<ACT>* q = static_cast<const act_t<ACT>*>(p.q) + (size_t)row * p.q_stride + head * (p.nope + p.rot);
    act_t<CT>* out = static_cast<act_t<CT>*>(p.qa) + ((size_t)row * p.heads + head) * p.cache.row_stride;
    if (blockIdx.z == gridDim.z - 1u) {              // the rotated part has a block of its own
        const uint32_t position = p.rows.position_of(row), half = p.rot_dims / 2u;
        for (uint32_t j = tid; j < p.cache.row_stride - p.rank; j += 256u) {
            if (j < half) {
                float c, s;
                position_angle(position, p.inv_freq[j], c, s);
                const float u = act_to_f32<ACT>(q[p.nope + j]), v = act_to_f32<ACT>(q[p.nope + half + j]);
                out[p.rank + j] = f32_to_act<CT>(u * c - v * s);
                out[p.rank + half + j] = f32_to_act<CT>(v * c + u * s);
            } else if (j >= p.rot_dims) {
                out[p.rank + j] = f32_to_act<CT>(j < p.rot ? act_to_f32<ACT>(q[p.nope + j]) : 0.0f);
            }
        }
        return;
    }
    const uint32_t r0 = blockIdx.z * 128u, r = min(r0 + piece * 8u, p.rank - 8u);
    const uint16_t* uk = p.uk + (size_t)head * p.nope * p.rank + r;
    float acc[8] = {};
    for (uint32_t d0 = 0; d0 < p.nope; d0 += 128u) {
        uint4 w[8];                                  // eight rows of W_uk in flight per lane
#pragma unroll
        for (int u = 0; u < 8; ++u) w[u] = *reinterpret_cast<const uint4*>(uk + (size_t)min(d0 + group + 16u * u, p.nope - 1u) * p.rank);
        if (d0 == 0) {
            for (uint32_t d = tid; d < p.nope; d += 256u) qs[d] = act_to_f32<ACT>(q[d]);
            __syncthreads();
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const uint32_t d = d0 + group + 16u * u;
            const float x = d < p.nope ? qs[min(d, p.nope - 1u)] : 0.0f;
            float f[8];
            act2_to_f32<ACT_BF16>(w[u].x, f[0], f[1]);
            act2_to_f32<ACT_BF16>(w[u].y, f[2], f[3]);
            act2_to_f32<ACT_BF16>(w[u].z, f[4], f[5]);
            act2_to_f32<ACT_BF16>(w[u].w, f[6], f[7]);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] = fmaf(f[e], x, acc[e]);
        }
    }
    *reinterpret_cast<la_f4*>(&part[group][piece * 8u]) = la_f4{acc[0], acc[1], acc[2], acc[3]};
    *reinterpret_cast<la_f4*>(&part[group][piece * 8u + 4u]) = la_f4{acc[4], acc[5], acc[6], acc[7]};
    __syncthreads();
    if (tid < 128u && r0 + tid < p.rank) {
        float a = 0.0f;
#pragma unroll
        for (int g = 0; g < 16; ++g) a += part[g][tid];
        out[r0 + tid] = f32_to_act<CT>(a);
    }
}

// ---- absorbed: scores and sums over one split of the window, sixteen heads per block --------------------
// Per 32 keys: S^T[key, head] = K Q^T with the waves splitting the row's elements (cache rows are the A operand as
// they lie in memory), the partial scores summed through LDS, the softmax in registers, and
// O^T[latent, head] += C^T P^T with the waves splitting the latent.  C^T comes from LDS: a thread transposes four
// keys x eight latents on the way in.  The score registers of a lane are the B operand of the second product when
// its eight keys are read as 4 g .. 4 g + 3 and 16 + 4 g .. 16 + 4 g + 3, so the columns of C^T lie in that order.
// P enters as two BF16 halves (hi + lo): fp32 weights.
template <int NT>
__global__ __launch_bounds__(256) void latent_partial_mfma_kernel(LatentAttnParams p) {
    constexpr int NQ = (2 * NT + 7) / 4;             // 32-element steps of a row per wave: rank <= 64 NT, rest <= 128
    constexpr int NV = (NT + 3) / 4;                 // transposed units per thread
    extern __shared__ __attribute__((aligned(16))) float la_lds[];
    uint16_t* ct = reinterpret_cast<uint16_t*>(la_lds);      // [rank][40]: 32 keys, rows 16 bytes off a power of two
    __shared__ __attribute__((aligned(16))) float sc[4][16][36];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, i = lane & 15u, g = lane >> 4;
    const uint32_t split = blockIdx.x, h0 = blockIdx.y * 16u, row = blockIdx.z;
    const uint32_t position = p.rows.position_of(row), first = first_key(position, p.window);
    const uint32_t lo = first + split * p.split_keys, hi = min(position + 1u, lo + p.split_keys);
    const uint32_t head = min(h0 + i, p.heads - 1u);
    const size_t cell = ((size_t)row * p.heads + head) * p.splits + split;
    if (lo >= hi) {                                  // uniform
        if (tid < 16u && h0 + tid < p.heads) { p.part_m[cell] = LA_NONE; p.part_l[cell] = 0.0f; }
        return;
    }
    const uint32_t rs = p.cache.row_stride, steps = rs / 32u, tiles = p.rank / 16u;
    const uint16_t* cache = static_cast<const uint16_t*>(p.cache.base) + (size_t)p.rows.slot_of(row) * p.cache.slot_stride;
    const uint16_t* q = static_cast<const uint16_t*>(p.qa) + ((size_t)row * p.heads + head) * rs;
    uint4 qf[NQ];
#pragma unroll
    for (int n = 0; n < NQ; ++n) qf[n] = *reinterpret_cast<const uint4*>(q + min(wave + 4u * n, steps - 1u) * 32u + 8u * g);
    la_f4 acc[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[n] = la_f4{0.0f, 0.0f, 0.0f, 0.0f};
    float m = LA_NONE, l = 0.0f;
    const uint32_t units = p.rank;                   // 8 groups of four keys x rank / 8 pieces
    for (uint32_t k0 = lo; k0 < hi; k0 += 32u) {
        const uint32_t ring0 = k0 % p.cache.capacity, most = hi - 1u - k0;
        auto row_of = [&](uint32_t key) {            // keys past the split repeat its last one
            uint32_t r = ring0 + min(key, most);
            r -= r >= p.cache.capacity ? p.cache.capacity : 0u;
            return cache + (size_t)r * rs;
        };
        uint4 vv[NV][4];
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const uint32_t u = min(tid + 256u * n, units - 1u), kg = u & 7u, piece = u >> 3;
#pragma unroll
            for (int e = 0; e < 4; ++e) vv[n][e] = *reinterpret_cast<const uint4*>(row_of(4u * kg + e) + piece * 8u);
        }
        const uint16_t *ka = row_of(i) + 8u * g, *kb = row_of(16u + i) + 8u * g;
        la_f4 s0 = la_f4{0.0f, 0.0f, 0.0f, 0.0f}, s1 = s0;
        uint4 fa[NQ], fb[NQ];
#pragma unroll
        for (int n = 0; n < NQ; ++n) {
            const uint32_t at = min(wave + 4u * n, steps - 1u) * 32u;
            fa[n] = *reinterpret_cast<const uint4*>(ka + at);
            fb[n] = *reinterpret_cast<const uint4*>(kb + at);
        }
#pragma unroll
        for (int n = 0; n < NQ; ++n)
            if (wave + 4u * n < steps) {             // uniform
                s0 = la_mfma(fa[n], qf[n], s0);
                s1 = la_mfma(fb[n], qf[n], s1);
            }
        *reinterpret_cast<la_f4*>(&sc[wave][i][4u * g]) = s0;
        *reinterpret_cast<la_f4*>(&sc[wave][i][16u + 4u * g]) = s1;
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const uint32_t u = tid + 256u * n, kg = u & 7u, piece = u >> 3;
            if (u < units) {
                const uint32_t at = kg < 4u ? 8u * kg : 8u * (kg - 4u) + 4u;
                const uint32_t a[4][4] = {{vv[n][0].x, vv[n][0].y, vv[n][0].z, vv[n][0].w}, {vv[n][1].x, vv[n][1].y, vv[n][1].z, vv[n][1].w},
                                          {vv[n][2].x, vv[n][2].y, vv[n][2].z, vv[n][2].w}, {vv[n][3].x, vv[n][3].y, vv[n][3].z, vv[n][3].w}};
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    const uint32_t sel = (e & 1) ? 0x07060302u : 0x05040100u;     // high or low halves of two dwords
                    uint2 w;
                    w.x = __builtin_amdgcn_perm(a[1][e >> 1], a[0][e >> 1], sel);
                    w.y = __builtin_amdgcn_perm(a[3][e >> 1], a[2][e >> 1], sel);
                    *reinterpret_cast<uint2*>(&ct[(piece * 8u + e) * 40u + at]) = w;
                }
            }
        }
        __syncthreads();
        float s[8];
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            la_f4 v = *reinterpret_cast<const la_f4*>(&sc[0][i][16 * h + 4u * g]);
#pragma unroll
            for (int w = 1; w < 4; ++w) v += *reinterpret_cast<const la_f4*>(&sc[w][i][16 * h + 4u * g]);
#pragma unroll
            for (int j = 0; j < 4; ++j) s[4 * h + j] = k0 + 16u * h + 4u * g + j < hi ? v[j] * p.scale_log2 : LA_NONE;
        }
        float tm = s[0];
#pragma unroll
        for (int j = 1; j < 8; ++j) tm = fmaxf(tm, s[j]);
        tm = fmaxf(tm, shfl_xor_f(tm, 16));
        tm = fmaxf(tm, shfl_xor_f(tm, 32));
        const float mn = fmaxf(m, tm), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        float ts = 0.0f;
        uint16_t ph[8], pl[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float e = s[j] > LA_NONE ? __builtin_amdgcn_exp2f(s[j] - mn) : 0.0f;
            ts += e;
            ph[j] = f32_to_bf16(e);
            pl[j] = f32_to_bf16(e - bf16_to_f32(ph[j]));
        }
        ts += shfl_xor_f(ts, 16);
        ts += shfl_xor_f(ts, 32);
        l = fmaf(l, alpha, ts);
        uint4 bh, bl;
        bh.x = ph[0] | ((uint32_t)ph[1] << 16); bh.y = ph[2] | ((uint32_t)ph[3] << 16);
        bh.z = ph[4] | ((uint32_t)ph[5] << 16); bh.w = ph[6] | ((uint32_t)ph[7] << 16);
        bl.x = pl[0] | ((uint32_t)pl[1] << 16); bl.y = pl[2] | ((uint32_t)pl[3] << 16);
        bl.z = pl[4] | ((uint32_t)pl[5] << 16); bl.w = pl[6] | ((uint32_t)pl[7] << 16);
#pragma unroll
        for (int n = 0; n < NT; ++n) {
            const uint32_t tile = wave + 4u * n;
            if (tile < tiles) {                      // uniform
                const uint4 a = *reinterpret_cast<const uint4*>(&ct[(16u * tile + i) * 40u + 8u * g]);
                acc[n] *= alpha;
                acc[n] = la_mfma(a, bh, acc[n]);
                acc[n] = la_mfma(a, bl, acc[n]);
            }
        }
        __syncthreads();
    }
    if (h0 + i >= p.heads) return;
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        const uint32_t tile = wave + 4u * n;
        if (tile < tiles) *reinterpret_cast<la_f4*>(p.part_o + cell * p.rank + 16u * tile + 4u * g) = acc[n];
    }
    if (wave == 0 && g == 0) { p.part_m[cell] = m; p.part_l[cell] = l; }
}

// One query row against keys [lo, hi) in blocks of 256, a thread per key, any sizes: the plain form behind both
// kernels below.  dot(key) is the score without scale, value(key, j) one value element; acc (LDS, [vd]) receives
// sum p v, and every thread the maximum and the sum.
template <typename Dot, typename Value>
__device__ __forceinline__ void la_plain_rows(uint32_t lo, uint32_t hi, uint32_t vd, float scale_log2, float* acc, float* ps,
                                              float* red, float& m, float& l, Dot dot, Value value) {
    const uint32_t tid = threadIdx.x;
    m = LA_NONE;
    l = 0.0f;
    for (uint32_t j = tid; j < vd; j += 256u) acc[j] = 0.0f;
    for (uint32_t k0 = lo; k0 < hi; k0 += 256u) {
        const uint32_t key = k0 + tid;
        const float s = key < hi ? dot(key) * scale_log2 : LA_NONE;
        const float wm = wave_max_f32(s);
        __syncthreads();                             // the previous block's ps and red have been read
        if ((tid & 63u) == 0) red[tid >> 6] = wm;
        __syncthreads();
        const float mn = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        const float e = key < hi ? __builtin_amdgcn_exp2f(s - mn) : 0.0f;
        ps[tid] = e;
        const float ws = wave_sum_bcast(e);
        if ((tid & 63u) == 0) red[4 + (tid >> 6)] = ws;
        __syncthreads();
        l = fmaf(l, alpha, (red[4] + red[5]) + (red[6] + red[7]));
        const uint32_t n = min(256u, hi - k0);
        for (uint32_t j = tid; j < vd; j += 256u) {
            float a = acc[j] * alpha;
            for (uint32_t k = 0; k < n; ++k) a = fmaf(ps[k], value(k0 + k, j), a);
            acc[j] = a;
        }
    }
    __syncthreads();
}

template <int ACT>
__global__ __launch_bounds__(256) void latent_partial_plain_kernel(LatentAttnParams p) {
    extern __shared__ __attribute__((aligned(16))) float la_lds[];
    const uint32_t tid = threadIdx.x, split = blockIdx.x, head = blockIdx.y, row = blockIdx.z, rs = p.cache.row_stride;
    float *qs = la_lds, *acc = qs + rs, *ps = acc + p.rank, *red = ps + 256;
    const uint32_t position = p.rows.position_of(row), first = first_key(position, p.window);
    const uint32_t lo = first + split * p.split_keys, hi = min(position + 1u, lo + p.split_keys);
    const size_t cell = ((size_t)row * p.heads + head) * p.splits + split;
    if (lo >= hi) {
        if (tid == 0) { p.part_m[cell] = LA_NONE; p.part_l[cell] = 0.0f; }
        return;
    }
    const act_t<ACT>* q = static_cast<const act_t<ACT>*>(p.qa) + ((size_t)row * p.heads + head) * rs;
    for (uint32_t j = tid; j < rs; j += 256u) qs[j] = act_to_f32<ACT>(q[j]);
    __syncthreads();
    const act_t<ACT>* cache = static_cast<const act_t<ACT>*>(p.cache.base) + (size_t)p.rows.slot_of(row) * p.cache.slot_stride;
    float m, l;
    la_plain_rows(lo, hi, p.rank, p.scale_log2, acc, ps, red, m, l,
        [&](uint32_t key) {
            const act_t<ACT>* k = cache + (size_t)(key % p.cache.capacity) * rs;
            float s = 0.0f;
            for (uint32_t j = 0; j < p.rank + p.rot; ++j) s = fmaf(act_to_f32<ACT>(k[j]), qs[j], s);
            return s;
        },
        [&](uint32_t key, uint32_t j) { return act_to_f32<ACT>(cache[(size_t)(key % p.cache.capacity) * rs + j]); });
    for (uint32_t j = tid; j < p.rank; j += 256u) p.part_o[cell * p.rank + j] = acc[j];
    if (tid == 0) { p.part_m[cell] = m; p.part_l[cell] = l; }
}

// ---- absorbed: splits combined, W_uv(h), the output gate ------------------------------------------------
// A block of 1024 per (head, row): eight groups of threads share the splits, the waves then the value rows.
template <int ACT>
__global__ __launch_bounds__(1024) void latent_combine_kernel(LatentAttnParams p) {
    extern __shared__ __attribute__((aligned(16))) float la_lds[];
    const uint32_t head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    float* o = la_lds;                   // [rank]
    float* sums = o + p.rank;            // [8][rank]
    float* wt = sums + 8u * p.rank;      // [splits]
    const size_t cell = ((size_t)row * p.heads + head) * p.splits;
    const float gate = p.gate ? la_sigmoid(act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.gate)[(size_t)row * p.gate_stride + head])) : 1.0f;
    // splits past the last key of this row wrote no sums and weigh nothing: the live ones are a prefix
    const uint32_t position = p.rows.position_of(row);
    const uint32_t live = min(p.splits, (position + 1u - first_key(position, p.window) + p.split_keys - 1u) / p.split_keys);
    const uint32_t group = tid >> 7, r0 = min((tid & 127u) * 4u, p.rank - 4u);
    const float* po = p.part_o + cell * p.rank;
    la_f4 ahead[8];                      // this group's first eight splits, requested before their weights are known
#pragma unroll
    for (int u = 0; u < 8; ++u) ahead[u] = *reinterpret_cast<const la_f4*>(po + (size_t)min(group + 8u * u, live - 1u) * p.rank + r0);
    float m = LA_NONE;
    for (uint32_t s = lane; s < p.splits; s += 64u) m = fmaxf(m, p.part_m[cell + s]);
    m = wave_max_f32(m);
    float l = 0.0f;
    for (uint32_t s = lane; s < p.splits; s += 64u) {
        const float ls = p.part_l[cell + s];
        const float w = ls > 0.0f ? __builtin_amdgcn_exp2f(p.part_m[cell + s] - m) : 0.0f;
        l = fmaf(ls, w, l);
        if (wave == 0) wt[s] = w;
    }
    l = wave_sum_bcast(l);
    const float inv = 1.0f / l;
    __syncthreads();
    for (uint32_t r = (tid & 127u) * 4u; r < p.rank; r += 512u) {
        la_f4 a = la_f4{0.0f, 0.0f, 0.0f, 0.0f};
        uint32_t s = group;
        if (r < 512u) {
#pragma unroll
            for (int u = 0; u < 8; ++u)
                if (group + 8u * u < live) a += ahead[u] * wt[group + 8u * u];
            s += 64u;
        }
#pragma unroll 8
        for (; s < live; s += 8u) a += *reinterpret_cast<const la_f4*>(po + (size_t)s * p.rank + r) * wt[s];
        *reinterpret_cast<la_f4*>(sums + group * p.rank + r) = a;
    }
    __syncthreads();
    for (uint32_t r = tid; r < p.rank; r += 1024u) {
        float a = 0.0f;
#pragma unroll
        for (int u = 0; u < 8; ++u) a += sums[u * p.rank + r];
        o[r] = a * inv;
    }
    __syncthreads();
    for (uint32_t j0 = wave * 4u; j0 < p.vdim; j0 += 64u) {      // four value rows of a wave in flight
        float a[4] = {};
        for (uint32_t r = lane * 8u; r < p.rank; r += 512u) {
            uint4 w[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) w[u] = *reinterpret_cast<const uint4*>(p.uv + (size_t)(head * p.vdim + min(j0 + u, p.vdim - 1u)) * p.rank + r);
            const la_f4 o0 = *reinterpret_cast<const la_f4*>(o + r), o1 = *reinterpret_cast<const la_f4*>(o + r + 4u);
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                float f[8];
                act2_to_f32<ACT_BF16>(w[u].x, f[0], f[1]);
                act2_to_f32<ACT_BF16>(w[u].y, f[2], f[3]);
                act2_to_f32<ACT_BF16>(w[u].z, f[4], f[5]);
                act2_to_f32<ACT_BF16>(w[u].w, f[6], f[7]);
#pragma unroll
                for (int e = 0; e < 4; ++e) a[u] = fmaf(f[4 + e], o1[e], fmaf(f[e], o0[e], a[u]));
            }
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const float v = wave_sum_bcast(a[u]);
            if (lane == (uint32_t)u && j0 + u < p.vdim)
                static_cast<act_t<ACT>*>(p.out)[(size_t)row * p.out_stride + head * p.vdim + j0 + u] = f32_to_act<ACT>(v * gate);
        }
    }
}

// ---- expanded: the range's cache rows gathered from the ring, queries rotated in place --------------------
template <int ACT>
__global__ __launch_bounds__(256) void latent_gather_kernel(LatentAttnParams p) {
    constexpr uint32_t PER = 16u / sizeof(act_t<ACT>);
    const uint32_t key = blockIdx.x, pieces = p.cache.row_stride / PER;
    const act_t<ACT>* src = static_cast<const act_t<ACT>*>(p.cache.base) + (size_t)p.rows.slot * p.cache.slot_stride +
                            (size_t)((p.key0 + min(key, p.nk - 1u)) % p.cache.capacity) * p.cache.row_stride;
    act_t<ACT>* dst = static_cast<act_t<ACT>*>(p.lat) + (size_t)key * p.cache.row_stride;
    for (uint32_t j = threadIdx.x; j < pieces; j += 256u) {
        const uint4 v = reinterpret_cast<const uint4*>(src)[j];
        reinterpret_cast<uint4*>(dst)[j] = key < p.nk ? v : make_uint4(0u, 0u, 0u, 0u);
    }
}

template <int ACT>
__global__ __launch_bounds__(256) void latent_rotate_q_kernel(LatentAttnParams p) {
    const uint32_t row = blockIdx.x, half = p.rot_dims / 2u, position = p.rows.position + row;
    extern __shared__ __attribute__((aligned(16))) float la_lds[];      // [half] cos, [half] sin
    for (uint32_t j = threadIdx.x; j < half; j += 256u) position_angle(position, p.inv_freq[j], la_lds[j], la_lds[half + j]);
    __syncthreads();
    act_t<ACT>* q = static_cast<act_t<ACT>*>(const_cast<void*>(p.q)) + (size_t)row * p.q_stride;
    for (uint32_t e = threadIdx.x; e < p.heads * half; e += 256u) {
        const uint32_t head = e / half, j = e % half;
        act_t<ACT>* r = q + head * (p.nope + p.rot) + p.nope + j;
        const float u = act_to_f32<ACT>(r[0]), v = act_to_f32<ACT>(r[half]), c = la_lds[j], s = la_lds[half + j];
        r[0] = f32_to_act<ACT>(u * c - v * s);
        r[half] = f32_to_act<ACT>(v * c + u * s);
    }
}

template <int ACT>
__global__ __launch_bounds__(256) void latent_expanded_plain_kernel(LatentAttnParams p) {
    extern __shared__ __attribute__((aligned(16))) float la_lds[];
    const uint32_t tid = threadIdx.x, head = blockIdx.x, row = blockIdx.y, dq = p.nope + p.rot;
    float *qs = la_lds, *acc = qs + dq, *ps = acc + p.vdim, *red = ps + 256;
    const act_t<ACT>* q = static_cast<const act_t<ACT>*>(p.q) + (size_t)row * p.q_stride + head * dq;
    for (uint32_t j = tid; j < dq; j += 256u) qs[j] = act_to_f32<ACT>(q[j]);
    __syncthreads();
    const uint32_t position = p.rows.position + row, lo = first_key(position, p.window) - p.key0, hi = position + 1u - p.key0;
    const act_t<ACT>*kn = static_cast<const act_t<ACT>*>(p.kn), *lat = static_cast<const act_t<ACT>*>(p.lat), *v = static_cast<const act_t<ACT>*>(p.v);
    float m, l;
    la_plain_rows(lo, hi, p.vdim, p.scale_log2, acc, ps, red, m, l,
        [&](uint32_t key) {
            const act_t<ACT>* a = kn + (size_t)key * p.kn_stride + head * p.nope;
            const act_t<ACT>* b = lat + (size_t)key * p.cache.row_stride + p.rank;
            float s = 0.0f;
            for (uint32_t j = 0; j < p.nope; ++j) s = fmaf(act_to_f32<ACT>(a[j]), qs[j], s);
            for (uint32_t j = 0; j < p.rot; ++j) s = fmaf(act_to_f32<ACT>(b[j]), qs[p.nope + j], s);
            return s;
        },
        [&](uint32_t key, uint32_t j) { return act_to_f32<ACT>(v[(size_t)key * p.v_stride + head * p.vdim + j]); });
    const float gate = p.gate ? la_sigmoid(act_to_f32<ACT>(static_cast<const act_t<ACT>*>(p.gate)[(size_t)row * p.gate_stride + head])) : 1.0f;
    for (uint32_t j = tid; j < p.vdim; j += 256u)
        static_cast<act_t<ACT>*>(p.out)[(size_t)row * p.out_stride + head * p.vdim + j] = f32_to_act<ACT>(acc[j] / l * gate);
}

// ---- expanded: flash attention over a window, BF16 -------------------------------------------------------
// 128 queries of one head per block, 32 per wave; K rows (in two regions, the head's own part and the shared rotated
// part) and V^T rows in tiles of 64 keys, loaded straight into LDS, the next tile under the current tile's products.
// S^T[key, query] = K Q^T and O^T[value, query] += V^T P^T.  Row m of score tile 2 h (2 h + 1) is key
// 32 h + 8 (m / 4) + m % 4 (+ 4): a lane's registers of the two tiles are then the keys 8 g .. 8 g + 7, in order, and
// stand as the B operand of the second product beside 16 contiguous bytes of V^T.
// LDS pieces of 16 bytes are exchanged within a row (la_swizzle) so that the eight lanes that a read serves at once
// fall into different banks.  NP, RP: the two parts of a key, DV: value dims, padded with zeros (a lane whose column
// does not exist loads from past the end of the buffer, which reads as zero).
template <int W>                         // row width in pieces
__device__ __forceinline__ uint32_t la_swizzle(uint32_t key) {
    return W >= 8 ? (key & 3u) | ((key >> 1) & 4u) : (key >> 3) & (W - 1u);
}

constexpr uint32_t LA_OUT_OF_BOUNDS = 0x80000000u;

template <int NP, int RP, int DV>
__global__ __launch_bounds__(256, NP + RP + DV <= 320 ? 2 : 1) void latent_flash_kernel(LatentAttnParams p) {
    constexpr int KN = NP / 32, KR = RP / 32, NV = DV / 16;
    constexpr int LN = NP / 32, LR = RP / 32, LV = DV / 32;      // 1 KB loads per wave and tile
    constexpr uint32_t AT_R = 64u * NP * 2u, AT_V = AT_R + 64u * RP * 2u, STAGE = AT_V + DV * 128u;
    extern __shared__ __attribute__((aligned(16))) float la_lds[];
    uint8_t* lds = reinterpret_cast<uint8_t*>(la_lds);
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i = lane & 15u, g = lane >> 4;
    // Blocks are dealt to the eight XCDs in turn: an XCD keeps to its own heads (their keys stay in its L2) where
    // the heads divide.  Even rounds take the query blocks with the most keys first, odd ones last: a compute unit's
    // two blocks then add up to the same work.
    const uint32_t nqb = (p.n_rows + 127u) / 128u, id = blockIdx.x;
    const uint32_t nth = p.heads % 8u == 0u ? id / 8u : id, round = nth / nqb, in_round = nth % nqb;
    const uint32_t head = p.heads % 8u == 0u ? round * 8u + id % 8u : round, qb = round & 1u ? in_round : nqb - 1u - in_round;
    const uint32_t q0 = qb * 128u, dq = p.nope + p.rot;
    const uint16_t* q = static_cast<const uint16_t*>(p.q) + head * dq;
    uint4 qf[2][KN + KR];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        const uint16_t* qr = q + (size_t)min(q0 + wave * 32u + 16u * b + i, p.n_rows - 1u) * p.q_stride;
#pragma unroll
        for (int s = 0; s < KN + KR; ++s) {
            const uint32_t d = s < KN ? 32u * s + 8u * g : 32u * (s - KN) + 8u * g, n = s < KN ? p.nope : p.rot;
            const uint4 v = *reinterpret_cast<const uint4*>(qr + (d < n ? (s < KN ? d : p.nope + d) : 0u));
            qf[b][s] = d < n ? v : make_uint4(0u, 0u, 0u, 0u);
        }
    }
    la_f4 acc[2][NV];
    float m[2] = {LA_NONE, LA_NONE}, l[2] = {0.0f, 0.0f};
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int n = 0; n < NV; ++n) acc[b][n] = la_f4{0.0f, 0.0f, 0.0f, 0.0f};
    // keys are numbered from key0
    const uint32_t last_t = min(q0 + 127u, p.n_rows - 1u);
    const uint32_t k_lo = (first_key(p.rows.position + q0, p.window) - p.key0) & ~63u;
    const uint32_t k_hi = p.rows.position + last_t + 1u - p.key0;
    const uint32_t kn_bytes = p.kn_stride * 2u, lat_bytes = p.cache.row_stride * 2u, v_bytes = p.v_stride * 2u;
    [[maybe_unused]] const __amdgpu_buffer_rsrc_t nrs = __builtin_amdgcn_make_buffer_rsrc(p.kn, 0, (int)(p.nk_pad * kn_bytes), 0x00020000);
    [[maybe_unused]] const __amdgpu_buffer_rsrc_t rrs = __builtin_amdgcn_make_buffer_rsrc(p.lat, 0, (int)(p.nk_pad * lat_bytes), 0x00020000);
    [[maybe_unused]] const __amdgpu_buffer_rsrc_t vrs = __builtin_amdgcn_make_buffer_rsrc(p.v, 0, (int)(p.heads * p.vdim * v_bytes), 0x00020000);
    uint32_t noff[LN], roff[LR], voff[LV];
#pragma unroll
    for (int j = 0; j < LN; ++j) {
        const uint32_t u = (wave * LN + j) * 64u + lane, key = u / (NP / 8), d = ((u % (NP / 8)) ^ la_swizzle<NP / 8>(key)) * 8u;
        noff[j] = d < p.nope ? key * kn_bytes + (head * p.nope + d) * 2u : LA_OUT_OF_BOUNDS;
    }
#pragma unroll
    for (int j = 0; j < LR; ++j) {
        const uint32_t u = (wave * LR + j) * 64u + lane, key = u / (RP / 8), d = ((u % (RP / 8)) ^ la_swizzle<RP / 8>(key)) * 8u;
        roff[j] = d < p.rot ? key * lat_bytes + (p.rank + d) * 2u : LA_OUT_OF_BOUNDS;
    }
#pragma unroll
    for (int j = 0; j < LV; ++j) {
        const uint32_t u = (wave * LV + j) * 64u + lane, d = u >> 3, piece = (u & 7u) ^ (d & 7u);
        voff[j] = d < p.vdim ? (head * p.vdim + d) * v_bytes + piece * 16u : LA_OUT_OF_BOUNDS;
    }
    auto issue = [&](uint32_t k0, uint8_t* dst) {
#if defined(__HIP_DEVICE_COMPILE__)     // the host pass rejects the 16-byte form of the load
#pragma unroll
        for (int j = 0; j < LN; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(nrs, (__attribute__((address_space(3))) void*)(dst + (wave * LN + j) * 1024u), 16, noff[j], k0 * kn_bytes, 0, 0);
#pragma unroll
        for (int j = 0; j < LR; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(rrs, (__attribute__((address_space(3))) void*)(dst + AT_R + (wave * LR + j) * 1024u), 16, roff[j], k0 * lat_bytes, 0, 0);
#pragma unroll
        for (int j = 0; j < LV; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(vrs, (__attribute__((address_space(3))) void*)(dst + AT_V + (wave * LV + j) * 1024u), 16, voff[j], k0 * 2u, 0, 0);
#endif
    };
    // this wave's own range of keys, and the part of it that every one of its queries sees
    const uint32_t wt0 = q0 + wave * 32u, wt1 = min(wt0 + 31u, p.n_rows - 1u);
    const bool wave_live = wt0 < p.n_rows;
    const uint32_t w_lo = first_key(p.rows.position + wt0, p.window) - p.key0, w_hi = p.rows.position + wt1 + 1u - p.key0;
    const uint32_t full_lo = first_key(p.rows.position + wt1, p.window) - p.key0, full_hi = p.rows.position + wt0 + 1u - p.key0;
    const uint32_t krow = 8u * (i >> 2) + (i & 3u);              // key of this lane's row in an even score tile
    issue(k_lo, lds);
    uint32_t stage = 0;
    for (uint32_t k0 = k_lo; k0 < k_hi; k0 += 64u, stage ^= 1u) {
        __syncthreads();                             // this tile has landed; everyone is done with the other stage
        if (k0 + 64u < k_hi) issue(k0 + 64u, lds + (stage ^ 1u) * STAGE);
        if (!wave_live || k0 >= w_hi || k0 + 64u <= w_lo) continue;             // wave-uniform
        const uint8_t* cur = lds + stage * STAGE;
        la_f4 s[2][4];
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int t = 0; t < 4; ++t) s[b][t] = la_f4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int st = 0; st < KN + KR; ++st) {
            uint4 a[4];
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const uint32_t key = 32u * (t >> 1) + 4u * (t & 1) + krow;
                a[t] = st < KN ? *reinterpret_cast<const uint4*>(cur + key * (NP * 2u) + ((4u * st + g) ^ la_swizzle<NP / 8>(key)) * 16u)
                               : *reinterpret_cast<const uint4*>(cur + AT_R + key * (RP * 2u) + ((4u * (st - KN) + g) ^ la_swizzle<RP / 8>(key)) * 16u);
            }
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int b = 0; b < 2; ++b) s[b][t] = la_mfma(a[t], qf[b][st], s[b][t]);
        }
        const bool masked = k0 < full_lo || k0 + 64u > full_hi;
        uint4 pf[2][2];
#pragma unroll
        for (int b = 0; b < 2; ++b) {
#pragma unroll
            for (int t = 0; t < 4; ++t) s[b][t] *= p.scale_log2;
            if (masked) {
                const uint32_t pos = p.rows.position + min(wt0 + 16u * b + i, p.n_rows - 1u);
                const uint32_t lo = first_key(pos, p.window) - p.key0, hi = pos + 1u - p.key0;
#pragma unroll
                for (int t = 0; t < 4; ++t)
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const uint32_t key = k0 + 32u * (t >> 1) + 8u * g + 4u * (t & 1) + j;
                        s[b][t][j] = key >= lo && key < hi ? s[b][t][j] : 2.0f * LA_NONE;
                    }
            }
            float tm = fmaxf(fmaxf(s[b][0][0], s[b][0][1]), fmaxf(s[b][0][2], s[b][0][3]));
#pragma unroll
            for (int t = 1; t < 4; ++t) tm = fmaxf(fmaxf(fmaxf(s[b][t][0], s[b][t][1]), fmaxf(s[b][t][2], s[b][t][3])), tm);
            tm = fmaxf(tm, shfl_xor_f(tm, 16));
            tm = fmaxf(tm, shfl_xor_f(tm, 32));
            if (__any(tm > m[b])) {
                const float mn = fmaxf(m[b], tm), alpha = __builtin_amdgcn_exp2f(m[b] - mn);
                m[b] = mn;
                l[b] *= alpha;
#pragma unroll
                for (int n = 0; n < NV; ++n) acc[b][n] *= alpha;
            }
            // a query without a key so far has m = LA_NONE, and exp2(2 LA_NONE - LA_NONE) = 0
            uint32_t w[8];
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                float e[4];
#pragma unroll
                for (int j = 0; j < 4; ++j) e[j] = __builtin_amdgcn_exp2f(s[b][t][j] - m[b]);
                l[b] += (e[0] + e[1]) + (e[2] + e[3]);
                w[2 * t] = la_pack2(e[0], e[1]);
                w[2 * t + 1] = la_pack2(e[2], e[3]);
            }
            pf[b][0] = make_uint4(w[0], w[1], w[2], w[3]);
            pf[b][1] = make_uint4(w[4], w[5], w[6], w[7]);
        }
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int n = 0; n < NV; ++n) {
                const uint4 a = *reinterpret_cast<const uint4*>(cur + AT_V + (16u * n + i) * 128u + ((4u * h + g) ^ (i & 7u)) * 16u);
#pragma unroll
                for (int b = 0; b < 2; ++b) acc[b][n] = la_mfma(a, pf[b][h], acc[b][n]);
            }
    }
    if (!wave_live) return;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        float sum = l[b];
        sum += shfl_xor_f(sum, 16);
        sum += shfl_xor_f(sum, 32);
        const uint32_t t = wt0 + 16u * b + i;
        if (t >= p.n_rows) continue;
        const float gate = p.gate ? la_sigmoid(bf16_to_f32(static_cast<const uint16_t*>(p.gate)[(size_t)t * p.gate_stride + head])) : 1.0f;
        const float f = gate / sum;
        uint16_t* out = static_cast<uint16_t*>(p.out) + (size_t)t * p.out_stride + head * p.vdim;
#pragma unroll
        for (int n = 0; n < NV; ++n) {
            const uint32_t d = 16u * n + 4u * g;
            if (d < p.vdim) *reinterpret_cast<uint2*>(out + d) = make_uint2(la_pack2(acc[b][n][0] * f, acc[b][n][1] * f), la_pack2(acc[b][n][2] * f, acc[b][n][3] * f));
        }
    }
}

}  // namespace nvmai
