// Windowed grouped-query attention over a cache of normed keys and transposed values.  gfx950, wave64.
//
// The token at t looks at s <= t where t - s < window, and at s < keep.  With z = scale q_t . k_s (k of the
// head's group), its score for s is cap(z) - slope (t - s): cap(z) = c tanh(z / c), or z where there is no cap; the slope of a
// head is a power of two of its index, or 0.  The softmax weights' sum over the values is multiplied by out_scale and, where
// there is a gate, by the sigmoid of one number per head and token.
//
// Keys and values of a slot lie in a ring (position p in row p % ring, ring a multiple of 64, so an aligned tile of
// positions is a run of rows) behind `pinned` rows that hold the first positions for good: position p < pinned is in
// row p as well and is read there (the ring may have passed over it while it is still seen).  What a token looks at is a
// range of kept tiles followed by the window's tiles, and one test per (query, key) decides what is seen in either.
// Values are stored transposed: 16 bytes of a row are eight positions of one channel, an A operand of the second product
// as they lie.
//   * split: decoding and short portions, sixteen heads of one kv head per block, waves and blocks share the tiles;
//   * flash: prompts, 128 queries of one head per block, tiles of 64 keys through LDS;
//   * plain: any sizes and types, a thread per key.
#pragma once

#include "rows.hpp"

namespace nvmai {

typedef __bf16 wa_b8 __attribute__((ext_vector_type(8)));
typedef float wa_f4 __attribute__((ext_vector_type(4)));
typedef float wa_f2 __attribute__((ext_vector_type(2)));
typedef __bf16 wa_b2 __attribute__((ext_vector_type(2)));

__device__ __forceinline__ wa_f4 wa_mfma(const uint4& a, const uint4& b, wa_f4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(wa_b8, a), __builtin_bit_cast(wa_b8, b), c, 0, 0, 0);
}
__device__ __forceinline__ uint32_t wa_pack2(float lo, float hi) {
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(wa_f2{lo, hi}, wa_b2));
}

constexpr float WA_LOG2E = 1.4426950408889634f;
constexpr float WA_NONE = -1e30f;        // maximum of no scores

struct KvRing {
    void *k, *v;
    uint32_t kv_heads, dk, dv, pinned, ring;
    __device__ __forceinline__ uint32_t rows() const { return pinned + ring; }
    // where a position, or an aligned tile of positions, is read
    __device__ __forceinline__ uint32_t row_of(uint32_t position) const { return position < pinned ? position : pinned + position % ring; }
};

struct WindowParams {
    const void* q;                       // [rows, q_stride], the cache's type
    const float* gate;                   // [rows, gate_stride], nullptr = none
    void* out;                           // [rows, out_stride] activations
    KvRing cache;
    SeqRows rows;
    uint32_t q_stride, gate_stride, out_stride, n_rows, heads, window, keep;
    // score to exponent of two: cap == 0: s -> a s;  else s -> b tanh(a s)
    float a, b, out_scale;
    bool capped, alibi;
    // split form
    float *part_o, *part_m, *part_l;     // [rows, heads, splits, dv], [rows, heads, splits] x 2
    uint32_t splits, tiles_per_split;
};

__device__ __forceinline__ float wa_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// 2^(-8 (head + 1) / heads) log2(e)
__device__ __forceinline__ float wa_slope_log2(uint32_t head, uint32_t heads) {
    return WA_LOG2E * exp2f(-8.0f * (float)(head + 1u) / (float)heads);
}

// tanh by the hardware exponential and reciprocal: absolute error of a few 2^-24, which is what a score's sum has.
__device__ __forceinline__ float wa_tanh(float z) {
    return fmaf(-2.0f, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(2.0f * WA_LOG2E * z)), 1.0f);
}

__device__ __forceinline__ bool wa_visible(uint32_t i, uint32_t j, uint32_t window, uint32_t keep) {
    return j <= i && (window == 0u || i - j < window || j < keep);
}

// ---- per-head norms of q and k, cache entries -----------------------------------------------------------
struct WindowEpilogueParams {
    const float* proj;
    const uint16_t *q_norm, *k_norm;     // [dk]
    void* q;
    KvRing cache;
    SeqRows rows;
    uint32_t proj_stride, q_at, k_at, v_at, q_stride, n_rows, heads, key_count;
    bool values;                         // write the values too (else window_values_kernel does)
    float eps;
};

// A wave per (row, head of q | k | v); NV elements per lane.
template <int CT, int NV>
__global__ __launch_bounds__(256) void window_epilogue_kernel(WindowEpilogueParams p) {
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, row = blockIdx.x, unit = blockIdx.y * 4u + wave;
    const uint32_t G = p.cache.kv_heads, dk = p.cache.dk, dv = p.cache.dv;
    const uint32_t units = p.heads + (p.k_norm ? (p.values ? 2u * G : G) : 0u);
    if (unit >= units) return;
    const float* proj = p.proj + (size_t)row * p.proj_stride;
    const uint32_t slot = p.rows.slot_of(row), position = p.rows.position_of(row);
    const uint32_t place = p.cache.pinned + position % p.cache.ring;
    const bool pin = position < p.cache.pinned;
    if (unit >= p.heads + G) {
        const uint32_t g = unit - p.heads - G;
        act_t<CT>* v = static_cast<act_t<CT>*>(p.cache.v) + ((size_t)slot * G + g) * dv * p.cache.rows();
        for (uint32_t d = lane; d < dv; d += 64u) {
            const act_t<CT> x = f32_to_act<CT>(proj[p.v_at + g * dv + d]);
            v[(size_t)d * p.cache.rows() + place] = x;
            if (pin) v[(size_t)d * p.cache.rows() + position] = x;
        }
        return;
    }
    const bool is_q = unit < p.heads;
    const uint32_t head = is_q ? unit : unit - p.heads;
    const float* src = proj + (is_q ? p.q_at : p.k_at) + head * dk;
    const uint16_t* w = is_q ? p.q_norm : p.k_norm;
    float v[NV], ss = 0.0f;
#pragma unroll
    for (int e = 0; e < NV; ++e) {
        const uint32_t d = lane + 64u * e;
        v[e] = d < dk ? src[min(d, dk - 1u)] : 0.0f;
        ss = fmaf(v[e], v[e], ss);
    }
    const float inv = 1.0f / sqrtf(wave_sum_bcast(ss) / (float)p.key_count + p.eps);
    act_t<CT>* k = static_cast<act_t<CT>*>(p.cache.k) + ((size_t)slot * G + (is_q ? 0u : head)) * p.cache.rows() * dk;
    act_t<CT>* q = static_cast<act_t<CT>*>(p.q) + (size_t)row * p.q_stride + head * dk;
#pragma unroll
    for (int e = 0; e < NV; ++e) {
        const uint32_t d = lane + 64u * e;
        if (d >= dk) break;
        const act_t<CT> x = f32_to_act<CT>(v[e] * inv * bf16_to_f32(w[d]));
        if (is_q) {
            q[d] = x;
        } else {
            k[(size_t)place * dk + d] = x;
            if (pin) k[(size_t)position * dk + d] = x;
        }
    }
}

// The values of a prompt's portion, 64 positions of one aligned tile x 64 channels at a time, transposed through LDS.
template <int CT>
__global__ __launch_bounds__(256) void window_values_kernel(WindowEpilogueParams p) {
    __shared__ float t[64][65];
    const uint32_t tid = threadIdx.x, g = blockIdx.y, d0 = blockIdx.z * 64u, dv = p.cache.dv, total = p.cache.rows();
    const uint32_t tile0 = (p.rows.position / 64u + blockIdx.x) * 64u;           // position of the tile's first row
    const uint32_t c = tid & 63u;
    for (uint32_t r = tid >> 6; r < 64u; r += 4u) {
        const uint32_t position = tile0 + r;
        if (position >= p.rows.position && position < p.rows.position + p.n_rows && d0 + c < dv)
            t[r][c] = p.proj[(size_t)(position - p.rows.position) * p.proj_stride + p.v_at + g * dv + d0 + c];
    }
    __syncthreads();
    const uint32_t position = tile0 + c;
    if (position < p.rows.position || position >= p.rows.position + p.n_rows) return;
    act_t<CT>* v = static_cast<act_t<CT>*>(p.cache.v) + ((size_t)p.rows.slot * p.cache.kv_heads + g) * dv * total;
    const uint32_t place = p.cache.pinned + position % p.cache.ring;
    for (uint32_t d = tid >> 6; d < 64u && d0 + d < dv; d += 4u) {
        const act_t<CT> x = f32_to_act<CT>(t[c][d]);
        v[(size_t)(d0 + d) * total + place] = x;
        if (position < p.cache.pinned) v[(size_t)(d0 + d) * total + position] = x;
    }
}

// ---- split form ------------------------------------------------------------------------------------------
// Tiles of 32 positions that the token at `position` looks at: `kept` of them from the pinned rows, then those from
// the window's first one on.
struct WindowTiles {
    uint32_t kept, first, count;
    __device__ __forceinline__ WindowTiles(uint32_t position, uint32_t window, uint32_t keep) {
        first = first_key(position, window) / 32u;
        kept = min((keep + 31u) / 32u, first);
        count = kept + position / 32u - first + 1u;
    }
    __device__ __forceinline__ uint32_t at(uint32_t n) const { return n < kept ? n : first + n - kept; }
};

// Block: (split, sixteen heads of a kv head, row); the four waves take the split's tiles in turn, each with maximum,
// sum and outputs of its own, and add them up at the end.  Per tile S^T[key, head] = K Q^T and O^T[value, head] += V^T P^T;
// row m of score tile 0 (1) is key 8 (m / 4) + m % 4 (+ 4), so a lane's score registers are the keys 8 g .. 8 g + 7 in order
// and stand as the second product's B operand beside 16 contiguous bytes of V^T.  P enters as two BF16 halves.
template <int DK, int DV>
__global__ __launch_bounds__(256) void window_split_kernel(WindowParams p) {
    constexpr int KS = DK / 32, VS = DV / 16;
    __shared__ __attribute__((aligned(16))) float os[3][VS][64][4];
    __shared__ float ms[4][16], ls[4][16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i = lane & 15u, g = lane >> 4;
    const uint32_t per = p.heads / p.cache.kv_heads, blocks = (per + 15u) / 16u;
    const uint32_t kv = blockIdx.y / blocks, sub = (blockIdx.y % blocks) * 16u, row = blockIdx.z, split = blockIdx.x;
    const uint32_t head = kv * per + min(sub + i, per - 1u);
    const uint32_t position = p.rows.position_of(row), dk = p.cache.dk, dv = p.cache.dv, total = p.cache.rows();
    const WindowTiles tiles(position, p.window, p.keep);
    const uint32_t lo = split * p.tiles_per_split, hi = min(tiles.count, lo + p.tiles_per_split);
    const size_t cell = ((size_t)row * p.heads + head) * p.splits + split;
    if (lo >= hi) {                                  // uniform
        if (tid < 16u && sub + tid < per) { p.part_m[cell] = WA_NONE; p.part_l[cell] = 0.0f; }
        return;
    }
    const size_t own = (size_t)p.rows.slot_of(row) * p.cache.kv_heads + kv;
    const uint16_t* kc = static_cast<const uint16_t*>(p.cache.k) + own * total * dk;
    const uint16_t* vc = static_cast<const uint16_t*>(p.cache.v) + own * dv * total;
    const uint16_t* q = static_cast<const uint16_t*>(p.q) + (size_t)row * p.q_stride + head * dk;
    const uint4 zero = make_uint4(0u, 0u, 0u, 0u);
    uint4 qf[KS];
#pragma unroll
    for (int s = 0; s < KS; ++s) {
        const uint4 v = *reinterpret_cast<const uint4*>(q + min(32u * s, dk - 32u) + 8u * g);
        qf[s] = 32u * s < dk ? v : zero;
    }
    wa_f4 acc[VS];
#pragma unroll
    for (int n = 0; n < VS; ++n) acc[n] = wa_f4{0.0f, 0.0f, 0.0f, 0.0f};
    float m = WA_NONE, l = 0.0f;
    const float slope = p.alibi ? wa_slope_log2(head, p.heads) : 0.0f;
    const uint32_t krow = 8u * (i >> 2) + (i & 3u);
    for (uint32_t n = lo + wave; n < hi; n += 4u) {
        const uint32_t pos0 = tiles.at(n) * 32u, row0 = p.cache.row_of(pos0);
        uint4 ka[KS], kb[KS], vf[VS];
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const uint16_t* k = kc + (size_t)(row0 + krow) * dk + min(32u * s, dk - 32u) + 8u * g;
            ka[s] = *reinterpret_cast<const uint4*>(k);
            kb[s] = *reinterpret_cast<const uint4*>(k + 4u * dk);
        }
#pragma unroll
        for (int t = 0; t < VS; ++t) vf[t] = *reinterpret_cast<const uint4*>(vc + (size_t)min(16u * t + i, dv - 1u) * total + row0 + 8u * g);
        wa_f4 s0 = wa_f4{0.0f, 0.0f, 0.0f, 0.0f}, s1 = s0;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            s0 = wa_mfma(ka[s], qf[s], s0);
            s1 = wa_mfma(kb[s], qf[s], s1);
        }
        float s[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const uint32_t key = pos0 + 8u * g + e;
            float v = (e < 4 ? s0[e & 3] : s1[e & 3]) * p.a;
            if (p.capped) v = p.b * wa_tanh(v);
            v = fmaf(-slope, (float)(int32_t)(position - key), v);
            s[e] = wa_visible(position, key, p.window, p.keep) ? v : 2.0f * WA_NONE;
        }
        float tm = s[0];
#pragma unroll
        for (int e = 1; e < 8; ++e) tm = fmaxf(tm, s[e]);
        tm = fmaxf(tm, shfl_xor_f(tm, 16));
        tm = fmaxf(tm, shfl_xor_f(tm, 32));
        const float mn = fmaxf(m, tm), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        float ts = 0.0f, hi8[8], lo8[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float x = __builtin_amdgcn_exp2f(s[e] - mn);   // no key so far: mn = WA_NONE, and exp2(WA_NONE) = 0
            ts += x;
            hi8[e] = bf16_to_f32(f32_to_bf16(x));
            lo8[e] = x - hi8[e];
        }
        ts += shfl_xor_f(ts, 16);
        ts += shfl_xor_f(ts, 32);
        l = fmaf(l, alpha, ts);
        const uint4 bh = make_uint4(wa_pack2(hi8[0], hi8[1]), wa_pack2(hi8[2], hi8[3]), wa_pack2(hi8[4], hi8[5]), wa_pack2(hi8[6], hi8[7]));
        const uint4 bl = make_uint4(wa_pack2(lo8[0], lo8[1]), wa_pack2(lo8[2], lo8[3]), wa_pack2(lo8[4], lo8[5]), wa_pack2(lo8[6], lo8[7]));
#pragma unroll
        for (int t = 0; t < VS; ++t) {
            acc[t] *= alpha;
            acc[t] = wa_mfma(vf[t], bh, acc[t]);
            acc[t] = wa_mfma(vf[t], bl, acc[t]);
        }
    }
    if (g == 0) { ms[wave][i] = m; ls[wave][i] = l; }
    __syncthreads();
    const float top = fmaxf(fmaxf(ms[0][i], ms[1][i]), fmaxf(ms[2][i], ms[3][i])), f = __builtin_amdgcn_exp2f(m - top);
    if (wave != 0) {
#pragma unroll
        for (int t = 0; t < VS; ++t) *reinterpret_cast<wa_f4*>(&os[wave - 1][t][lane][0]) = acc[t] * f;
    }
    __syncthreads();
    if (wave != 0 || sub + i >= per) return;
    float sum = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) sum = fmaf(ls[w][i], __builtin_amdgcn_exp2f(ms[w][i] - top), sum);
#pragma unroll
    for (int t = 0; t < VS; ++t) {
        wa_f4 o = acc[t] * f;
#pragma unroll
        for (int w = 0; w < 3; ++w) o += *reinterpret_cast<const wa_f4*>(&os[w][t][lane][0]);
        if (16u * t < dv) *reinterpret_cast<wa_f4*>(p.part_o + cell * dv + 16u * t + 4u * g) = o;
    }
    if (g == 0) { p.part_m[cell] = top; p.part_l[cell] = sum; }
}

// The splits of one (head, row), the gate, the scale.  A quarter of dv per 64 threads' four columns: NG groups of
// dv / 4 threads share the splits.
template <int ACT>
__global__ __launch_bounds__(256) void window_combine_kernel(WindowParams p) {
    extern __shared__ __attribute__((aligned(16))) float wa_lds[];
    const uint32_t head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63u, dv = p.cache.dv;
    const uint32_t position = p.rows.position_of(row);
    const WindowTiles tiles(position, p.window, p.keep);
    const uint32_t live = (tiles.count + p.tiles_per_split - 1u) / p.tiles_per_split;
    float* wt = wa_lds;                              // [splits rounded up to 4]
    float* sums = wa_lds + (p.splits + 3u) / 4u * 4u;         // [groups, dv]
    const size_t cell = ((size_t)row * p.heads + head) * p.splits;
    const float gate = p.gate ? wa_sigmoid(p.gate[(size_t)row * p.gate_stride + head]) : 1.0f;
    const uint32_t cols = dv / 4u, groups = 256u / cols, group = tid / cols, d = (tid % cols) * 4u;
    const float* po = p.part_o + cell * dv;
    wa_f4 ahead[4];                                  // requested before their weights are known
#pragma unroll
    for (int u = 0; u < 4; ++u) ahead[u] = *reinterpret_cast<const wa_f4*>(po + (size_t)min(group + groups * u, live - 1u) * dv + d);
    float m = WA_NONE;
    for (uint32_t s = lane; s < live; s += 64u) m = fmaxf(m, p.part_m[cell + s]);
    m = wave_max_f32(m);
    float l = 0.0f;
    for (uint32_t s = lane; s < live; s += 64u) {
        const float ls = p.part_l[cell + s], w = ls > 0.0f ? __builtin_amdgcn_exp2f(p.part_m[cell + s] - m) : 0.0f;
        l = fmaf(ls, w, l);
        if (tid < 64u) wt[s] = w;
    }
    l = wave_sum_bcast(l);
    __syncthreads();
    wa_f4 a = wa_f4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int u = 0; u < 4; ++u)
        if (group + groups * u < live) a += ahead[u] * wt[group + groups * u];
    for (uint32_t s = group + 4u * groups; s < live; s += groups) a += *reinterpret_cast<const wa_f4*>(po + (size_t)s * dv + d) * wt[s];
    if (group < groups) *reinterpret_cast<wa_f4*>(sums + group * dv + d) = a;
    __syncthreads();
    for (uint32_t j = tid; j < dv; j += 256u) {
        float v = 0.0f;
        for (uint32_t u = 0; u < groups; ++u) v += sums[u * dv + j];
        static_cast<act_t<ACT>*>(p.out)[(size_t)row * p.out_stride + head * dv + j] = f32_to_act<ACT>(v / l * (gate * p.out_scale));
    }
}

// ---- plain form: a block per (head, row), a thread per key ------------------------------------------------
template <int ACT, int CT>
__global__ __launch_bounds__(256) void window_plain_kernel(WindowParams p) {
    extern __shared__ __attribute__((aligned(16))) float wa_lds[];
    const uint32_t head = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, dk = p.cache.dk, dv = p.cache.dv, total = p.cache.rows();
    float *qs = wa_lds, *acc = qs + dk, *ps = acc + dv, *red = ps + 256;
    const uint32_t position = p.rows.position_of(row), first = first_key(position, p.window), kept = min(p.keep, first);
    const size_t own = (size_t)p.rows.slot_of(row) * p.cache.kv_heads + head / (p.heads / p.cache.kv_heads);
    const act_t<CT>* kc = static_cast<const act_t<CT>*>(p.cache.k) + own * total * dk;
    const act_t<CT>* vc = static_cast<const act_t<CT>*>(p.cache.v) + own * dv * total;
    const act_t<CT>* q = static_cast<const act_t<CT>*>(p.q) + (size_t)row * p.q_stride + head * dk;
    for (uint32_t j = tid; j < dk; j += 256u) qs[j] = act_to_f32<CT>(q[j]);
    for (uint32_t j = tid; j < dv; j += 256u) acc[j] = 0.0f;
    __syncthreads();
    const float slope = p.alibi ? wa_slope_log2(head, p.heads) : 0.0f;
    const uint32_t keys = kept + position - first + 1u;
    auto key_at = [&](uint32_t n) { return n < kept ? n : first + n - kept; };
    auto row_at = [&](uint32_t n) { return p.cache.row_of(key_at(n)); };
    float m = WA_NONE, l = 0.0f;
    for (uint32_t n0 = 0; n0 < keys; n0 += 256u) {
        const uint32_t n = n0 + tid;
        float s = WA_NONE;
        if (n < keys) {
            const act_t<CT>* k = kc + (size_t)row_at(n) * dk;
            float dot = 0.0f;
            for (uint32_t j = 0; j < dk; ++j) dot = fmaf(act_to_f32<CT>(k[j]), qs[j], dot);
            s = dot * p.a;
            if (p.capped) s = p.b * tanhf(s);
            s = fmaf(-slope, (float)(position - key_at(n)), s);
        }
        const float wm = wave_max_f32(s);
        __syncthreads();                             // the previous block's ps and red have been read
        if ((tid & 63u) == 0) red[tid >> 6] = wm;
        __syncthreads();
        const float mn = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m), alpha = __builtin_amdgcn_exp2f(m - mn);
        m = mn;
        const float e = n < keys ? exp2f(s - mn) : 0.0f;
        ps[tid] = e;
        const float ws = wave_sum_bcast(e);
        if ((tid & 63u) == 0) red[4 + (tid >> 6)] = ws;
        __syncthreads();
        l = fmaf(l, alpha, (red[4] + red[5]) + (red[6] + red[7]));
        const uint32_t live = min(256u, keys - n0);
        for (uint32_t j = tid; j < dv; j += 256u) {
            float a = acc[j] * alpha;
            for (uint32_t e0 = 0; e0 < live; ++e0) a = fmaf(ps[e0], act_to_f32<CT>(vc[(size_t)j * total + row_at(n0 + e0)]), a);
            acc[j] = a;
        }
    }
    __syncthreads();
    const float gate = (p.gate ? wa_sigmoid(p.gate[(size_t)row * p.gate_stride + head]) : 1.0f) * p.out_scale;
    for (uint32_t j = tid; j < dv; j += 256u)
        static_cast<act_t<ACT>*>(p.out)[(size_t)row * p.out_stride + head * dv + j] = f32_to_act<ACT>(acc[j] / l * gate);
}

// ---- flash form ------------------------------------------------------------------------------------------
// 128 queries of one head per block, 32 per wave; K and V^T tiles of 64 keys, loaded straight into LDS, the next tile
// under the current tile's products.  S^T[key, query] = K Q^T, O^T[value, query] += V^T P^T, with the order of keys of the split
// form.  LDS pieces of 16 bytes are exchanged within a row so that the lanes a read serves at once fall into different
// banks.  DK, DV: sizes padded with zeros (a lane whose column does not exist loads from past the end of the
// buffer, which reads as zero).
// BOUND: the scores are capped and the cap b (in powers of two) is at most WA_BOUND, so weights relative to b / 2 instead of
// the running maximum stay between 2^(-3 b / 2) and 2^(b / 2): no maximum, and b tanh(z) - b / 2 = b / 2 - 2 b / (1 + e^(2 z)) is
// one exponential, one reciprocal and one multiply-add.
template <int W>                         // row width in pieces
__device__ __forceinline__ uint32_t wa_swizzle(uint32_t key) {
    return W >= 8 ? (key & 3u) | ((key >> 1) & 4u) : (key >> 3) & (W - 1u);
}

constexpr uint32_t WA_OUT_OF_BOUNDS = 0x80000000u;
constexpr float WA_BOUND = 80.0f;

template <int DK, int DV, bool BOUND>
__global__ __launch_bounds__(256, DK + DV <= 256 ? 2 : 1) void window_flash_kernel(WindowParams p) {
    constexpr int KS = DK / 32, VS = DV / 16;
    constexpr int LK = DK / 32, LV = DV / 32;        // 1 KB loads per wave and tile
    constexpr uint32_t AT_V = 64u * DK * 2u, STAGE = AT_V + DV * 128u;
    extern __shared__ __attribute__((aligned(16))) float wa_lds[];
    uint8_t* lds = reinterpret_cast<uint8_t*>(wa_lds);
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i = lane & 15u, g = lane >> 4;
    // Blocks are dealt to the eight XCDs in turn: an XCD keeps to its own heads (their keys stay in its L2) where
    // the heads divide.  Even rounds take the query blocks with the most keys first, odd ones last: a compute unit's
    // two blocks then add up to the same work.
    const uint32_t nqb = (p.n_rows + 127u) / 128u, id = blockIdx.x;
    const uint32_t nth = p.heads % 8u == 0u ? id / 8u : id, round = nth / nqb, in_round = nth % nqb;
    // neighbouring heads (which share a kv head) on one XCD
    const uint32_t head = p.heads % 8u == 0u ? (id % 8u) * (p.heads / 8u) + round : round, qb = round & 1u ? in_round : nqb - 1u - in_round;
    const uint32_t q0 = qb * 128u, dk = p.cache.dk, dv = p.cache.dv, total = p.cache.rows(), start = p.rows.position;
    const uint16_t* q = static_cast<const uint16_t*>(p.q) + head * dk;
    uint4 qf[2][KS];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        const uint16_t* qr = q + (size_t)min(q0 + wave * 32u + 16u * b + i, p.n_rows - 1u) * p.q_stride;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const uint32_t d = 32u * s + 8u * g;
            const uint4 v = *reinterpret_cast<const uint4*>(qr + (d < dk ? d : 0u));
            qf[b][s] = d < dk ? v : make_uint4(0u, 0u, 0u, 0u);
        }
    }
    wa_f4 acc[2][VS];
    float m[2] = {WA_NONE, WA_NONE}, l[2] = {0.0f, 0.0f};
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int n = 0; n < VS; ++n) acc[b][n] = wa_f4{0.0f, 0.0f, 0.0f, 0.0f};
    const uint32_t last = start + min(q0 + 127u, p.n_rows - 1u);
    // tiles of 64 positions: the kept ones, then from the window's first one to the last query's
    const uint32_t first_t = first_key(start + q0, p.window) / 64u, kept = min((p.keep + 63u) / 64u, first_t), count = kept + last / 64u - first_t + 1u;
    const size_t own = (size_t)p.rows.slot * p.cache.kv_heads + head / (p.heads / p.cache.kv_heads);
    [[maybe_unused]] const __amdgpu_buffer_rsrc_t krs = __builtin_amdgcn_make_buffer_rsrc(
        static_cast<uint16_t*>(p.cache.k) + own * total * dk, 0, (int)(total * dk * 2u), 0x00020000);
    [[maybe_unused]] const __amdgpu_buffer_rsrc_t vrs = __builtin_amdgcn_make_buffer_rsrc(
        static_cast<uint16_t*>(p.cache.v) + own * dv * total, 0, (int)(total * dv * 2u), 0x00020000);
    uint32_t koff[LK], voff[LV];
#pragma unroll
    for (int j = 0; j < LK; ++j) {
        const uint32_t u = (wave * LK + j) * 64u + lane, key = u / (DK / 8), d = ((u % (DK / 8)) ^ wa_swizzle<DK / 8>(key)) * 8u;
        koff[j] = d < dk ? (key * dk + d) * 2u : WA_OUT_OF_BOUNDS;
    }
#pragma unroll
    for (int j = 0; j < LV; ++j) {
        const uint32_t u = (wave * LV + j) * 64u + lane, d = u >> 3, piece = (u & 7u) ^ (d & 7u);
        voff[j] = d < dv ? d * total * 2u + piece * 16u : WA_OUT_OF_BOUNDS;
    }
    auto position_of = [&](uint32_t n) { return (n < kept ? n : first_t + n - kept) * 64u; };
    auto issue = [&](uint32_t n, uint8_t* dst) {
        [[maybe_unused]] const uint32_t pos0 = position_of(n), row0 = p.cache.row_of(pos0);
#if defined(__HIP_DEVICE_COMPILE__)     // the host pass rejects the 16-byte form of the load
#pragma unroll
        for (int j = 0; j < LK; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(krs, (__attribute__((address_space(3))) void*)(dst + (wave * LK + j) * 1024u), 16, koff[j], row0 * dk * 2u, 0, 0);
#pragma unroll
        for (int j = 0; j < LV; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(vrs, (__attribute__((address_space(3))) void*)(dst + AT_V + (wave * LV + j) * 1024u), 16, voff[j], row0 * 2u, 0, 0);
#endif
    };
    // this wave's queries, the keys some of them see beside the kept ones, and those that all of them see
    const uint32_t wt0 = q0 + wave * 32u, wt1 = min(wt0 + 31u, p.n_rows - 1u);
    const bool wave_live = wt0 < p.n_rows;
    const uint32_t w_lo = first_key(start + wt0, p.window), w_hi = start + wt1 + 1u;
    const uint32_t full_lo = first_key(start + wt1, p.window), full_hi = start + wt0 + 1u;
    const uint32_t krow = 8u * (i >> 2) + (i & 3u);              // key of this lane's row in an even score tile
    const float slope = p.alibi ? wa_slope_log2(head, p.heads) : 0.0f;
    issue(0, lds);
    uint32_t stage = 0;
    for (uint32_t n = 0; n < count; ++n, stage ^= 1u) {
        __syncthreads();                             // this tile has landed; everyone is done with the other stage
        if (n + 1u < count) issue(n + 1u, lds + (stage ^ 1u) * STAGE);
        const uint32_t k0 = position_of(n);
        if (!wave_live || k0 >= w_hi || (k0 + 64u <= w_lo && k0 >= p.keep)) continue;              // wave-uniform
        const uint8_t* cur = lds + stage * STAGE;
        wa_f4 s[2][4];
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int t = 0; t < 4; ++t) s[b][t] = wa_f4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int st = 0; st < KS; ++st) {
            uint4 a[4];
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                const uint32_t key = 32u * (t >> 1) + 4u * (t & 1) + krow;
                a[t] = *reinterpret_cast<const uint4*>(cur + key * (DK * 2u) + ((4u * st + g) ^ wa_swizzle<DK / 8>(key)) * 16u);
            }
#pragma unroll
            for (int t = 0; t < 4; ++t)
#pragma unroll
                for (int b = 0; b < 2; ++b) s[b][t] = wa_mfma(a[t], qf[b][st], s[b][t]);
        }
        const bool masked = k0 < full_lo || k0 + 64u > full_hi;
        uint4 pf[2][2];
#pragma unroll
        for (int b = 0; b < 2; ++b) {
            const uint32_t pos = start + min(wt0 + 16u * b + i, p.n_rows - 1u);
            uint32_t w[8];
            if (BOUND) {
                const float z2 = 2.0f * WA_LOG2E * p.a, half = 0.5f * p.b, slide = -2.0f * p.b;
#pragma unroll
                for (int t = 0; t < 4; ++t) {
                    float e[4];
#pragma unroll
                    for (int j = 0; j < 4; ++j)
                        e[j] = __builtin_amdgcn_exp2f(fmaf(slide, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z2 * s[b][t][j])), half));
                    if (masked) {
#pragma unroll
                        for (int j = 0; j < 4; ++j) {
                            const uint32_t key = k0 + 32u * (t >> 1) + 8u * g + 4u * (t & 1) + j;
                            e[j] = wa_visible(pos, key, p.window, p.keep) ? e[j] : 0.0f;
                        }
                    }
                    l[b] += (e[0] + e[1]) + (e[2] + e[3]);
                    w[2 * t] = wa_pack2(e[0], e[1]);
                    w[2 * t + 1] = wa_pack2(e[2], e[3]);
                }
                pf[b][0] = make_uint4(w[0], w[1], w[2], w[3]);
                pf[b][1] = make_uint4(w[4], w[5], w[6], w[7]);
                continue;
            }
#pragma unroll
            for (int t = 0; t < 4; ++t) s[b][t] *= p.a;
            if (p.capped) {
#pragma unroll
                for (int t = 0; t < 4; ++t)
#pragma unroll
                    for (int j = 0; j < 4; ++j) s[b][t][j] = p.b * wa_tanh(s[b][t][j]);
            }
            if (p.alibi) {
                const float far = (float)(int32_t)(pos - k0 - 8u * g);           // distance of this lane's first key
#pragma unroll
                for (int t = 0; t < 4; ++t)
#pragma unroll
                    for (int j = 0; j < 4; ++j) s[b][t][j] = fmaf(-slope, far - (float)(32 * (t >> 1) + 4 * (t & 1) + j), s[b][t][j]);
            }
            if (masked) {
#pragma unroll
                for (int t = 0; t < 4; ++t)
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const uint32_t key = k0 + 32u * (t >> 1) + 8u * g + 4u * (t & 1) + j;
                        s[b][t][j] = wa_visible(pos, key, p.window, p.keep) ? s[b][t][j] : 2.0f * WA_NONE;
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
                for (int t = 0; t < VS; ++t) acc[b][t] *= alpha;
            }
            // a query without a key so far has m = WA_NONE, and exp2(2 WA_NONE - WA_NONE) = 0
#pragma unroll
            for (int t = 0; t < 4; ++t) {
                float e[4];
#pragma unroll
                for (int j = 0; j < 4; ++j) e[j] = __builtin_amdgcn_exp2f(s[b][t][j] - m[b]);
                l[b] += (e[0] + e[1]) + (e[2] + e[3]);
                w[2 * t] = wa_pack2(e[0], e[1]);
                w[2 * t + 1] = wa_pack2(e[2], e[3]);
            }
            pf[b][0] = make_uint4(w[0], w[1], w[2], w[3]);
            pf[b][1] = make_uint4(w[4], w[5], w[6], w[7]);
        }
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int t = 0; t < VS; ++t) {
                const uint4 a = *reinterpret_cast<const uint4*>(cur + AT_V + (16u * t + i) * 128u + ((4u * h + g) ^ (i & 7u)) * 16u);
#pragma unroll
                for (int b = 0; b < 2; ++b) acc[b][t] = wa_mfma(a, pf[b][h], acc[b][t]);
            }
    }
    if (!wave_live) return;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        float sum = l[b];
        sum += shfl_xor_f(sum, 16);
        sum += shfl_xor_f(sum, 32);
        const uint32_t t0 = wt0 + 16u * b + i;
        if (t0 >= p.n_rows) continue;
        const float gate = p.gate ? wa_sigmoid(p.gate[(size_t)t0 * p.gate_stride + head]) : 1.0f;
        const float f = gate * p.out_scale / sum;
        uint16_t* out = static_cast<uint16_t*>(p.out) + (size_t)t0 * p.out_stride + head * dv;
#pragma unroll
        for (int t = 0; t < VS; ++t) {
            const uint32_t d = 16u * t + 4u * g;
            if (d < dv) *reinterpret_cast<uint2*>(out + d) = make_uint2(wa_pack2(acc[b][t][0] * f, acc[b][t][1] * f), wa_pack2(acc[b][t][2] * f, acc[b][t][3] * f));
        }
    }
}

}  // namespace nvmai
