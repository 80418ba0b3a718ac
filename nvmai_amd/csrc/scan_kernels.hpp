// Recurrences with one decay per head and a matrix state, all in fp32.  gfx950, wave64.
//
//   S_t = g_t S_(t-1) + k_t u_t^T,   o_t = S_t^T q_t,   g_t = e^(-x_t)
//   gated delta rule:   u_t = beta_t (v_t - g_t S_(t-1)^T k_t);  q, k unit vectors per head
//   state-space (SSD):  u_t = dt_t v_t;  o_t += skip v_t         (q = C, k = B, v = x)
//
// q, k and v are projected rows after a causal filter per channel and silu.  Two forms:
//   * recurrent, for decoding and short portions: one launch, filter included, sixteen state columns per block;
//   * chunked, for prompts, 64 rows at a time.  With X_i = x_0 + .. + x_i, G_i = e^(-X_i) and S the state a chunk finds:
//         (I + L) U = R,  L[i][m] = beta_i e^(X_m - X_i) (k_m . k_i)  (m < i),  R[i] = beta_i v_i - beta_i G_i S^T k_i
//         o_i   = G_i S^T q_i + sum_{m <= i} W[i][m] u_m,   W[i][m] = e^(X_m - X_i) (k_m . q_i)
//         S_end = G_63 S + sum_m e^(X_m - X_63) k_m u_m^T
//     scan_prep_kernel makes what needs no state for every (chunk, head) at once: W, the decays, and for the delta rule
//     U0 = (I + L)^-1 beta V and Kt = (I + L)^-1 beta G K by forward substitution, a thread per column; U = U0 - Kt S.
//     (SSD: U = dt V.)  scan_chain_kernel then walks the chunks, a block per (head, sixteen state columns).
//     The sums X are kept in double: e^(X_m - X_i) of two late rows stays exact behind a row that has forgotten everything.
// All products run on v_mfma_f32_16x16x4_f32.  Register r of an accumulator tile in lane (i, g) is row 4 g + r, column i, which
// is a B operand of the next product as it stands when its k indices are taken in the order 4 g + r.
#pragma once

#include "rows.hpp"

namespace nvmai {

typedef float sc_f4 __attribute__((ext_vector_type(4)));

constexpr uint32_t SCAN_CHUNK = 64;
constexpr uint32_t SCAN_AHEAD = 32;      // rows of one recurrent launch: history_rows >= taps - 1 + SCAN_AHEAD

struct ScanParams {
    const float* proj;                   // [rows, proj_stride]
    const uint16_t *conv, *conv_bias;    // [channels, taps], [channels] or nullptr
    const uint16_t *a_log, *dt_bias, *skip;
    float* history;                      // [slots, history_rows, channels]
    float* state;                        // [slots, heads, dk, dv]
    float* out;                          // row t, head h: out + t out_stride + h out_head
    uint64_t out_head;
    SeqRows rows;
    uint32_t proj_stride, out_stride, n_rows, heads, key_heads, dk, dv, taps, history_rows, conv_at, a_at, b_at, channels;
    float q_scale;
    // chunked form
    float* mixed;                        // q [key_heads, rows_p, dk] | k, the same | v [heads, rows_p, dv]: after filter, silu and norm
    float *in_a, *in_b;                  // [heads, rows_p]: the gates' inputs
    uint32_t rows_p;                     // rows up to a whole chunk
    float *w, *gates;                    // [chunk, head, 64, 64], [chunk, head, 3, 64]: G, e^(X_i - X_63), dt
    // operands of the chain as its waves hold them, a float4 per lane: Kt [chunk, head, 4 row tiles, dk / 16], U0 [chunk, head,
    // dv / 16, 4 row tiles], k^T [chunk, key head, dk / 16, 4 row tiles], each of 64 lanes
    float *kt, *u0, *k_t;

    // Rows of a head lie together: a chunk's operand is one run of memory, not 64 pieces at the stride of a whole row.
    __device__ __forceinline__ float* q_of(uint32_t key_head, uint32_t row) const { return mixed + ((size_t)key_head * rows_p + row) * dk; }
    __device__ __forceinline__ float* k_of(uint32_t key_head, uint32_t row) const { return q_of(key_heads + key_head, row); }
    __device__ __forceinline__ float* v_of(uint32_t head, uint32_t row) const {
        return mixed + (size_t)2u * key_heads * rows_p * dk + ((size_t)head * rows_p + row) * dv;
    }
};

__device__ __forceinline__ float scan_softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float scan_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// The filter's input at row t of a sequence's rows (t < 0: from the history, zeros before the sequence).
// first: position of row 0, base: index of row 0 in proj.
__device__ __forceinline__ float scan_input(const ScanParams& p, uint32_t slot, uint32_t base, uint32_t first, int32_t t, uint32_t ch) {
    if (t >= 0) return p.proj[(size_t)(base + (uint32_t)t) * p.proj_stride + p.conv_at + ch];
    const int64_t position = (int64_t)first + t;
    return position < 0 ? 0.0f : p.history[((size_t)slot * p.history_rows + (uint32_t)position % p.history_rows) * p.channels + ch];
}

__device__ __forceinline__ float scan_filter(const ScanParams& p, uint32_t slot, uint32_t base, uint32_t first, uint32_t t, uint32_t ch) {
    float z = p.conv_bias ? bf16_to_f32(p.conv_bias[ch]) : 0.0f;
    const uint16_t* w = p.conv + (size_t)ch * p.taps;
    for (uint32_t j = 0; j < p.taps; ++j) z = fmaf(bf16_to_f32(w[j]), scan_input(p, slot, base, first, (int32_t)(t + j) - (int32_t)(p.taps - 1u), ch), z);
    return silu(z);
}

// A barrier of the block's waves that leaves loads from memory in flight.
__device__ __forceinline__ void scan_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// ---- recurrent form --------------------------------------------------------------------------------------
// Block (head, 16 CP columns, sequence): thread (j = tid % 16, group c = tid / 16) owns the state rows c PER .. c PER + PER - 1
// of the columns CP j .. CP j + CP - 1.  CP 1 makes many small blocks (one sequence), CP 4 fewer whose filter serves more
// columns.  Only the block that owns a channel (its value columns; the q and k of a key head: the first block of its
// first head) writes the channel's history, in rows that no block of the launch reads.
template <bool DELTA, int PER, int CP>
__global__ __launch_bounds__(256) void scan_recurrent_kernel(ScanParams p, uint32_t seq_rows) {
    constexpr uint32_t COLS = 16u * CP;
    __shared__ __attribute__((aligned(16))) float qs[16 * PER], ks[16 * PER], vs[COLS], part[2][4][COLS];
    __shared__ float red[3][4];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, j = tid & 15u, c = tid >> 4;
    const uint32_t head = blockIdx.x, c0 = blockIdx.y * COLS, seq = blockIdx.z, dk = p.dk;
    const uint32_t ratio = p.heads / p.key_heads, key_head = head / ratio;
    const uint32_t base = seq * seq_rows, slot = p.rows.slot_of(base), first = p.rows.position_of(base);
    const uint32_t q_ch = key_head * dk, k_ch = (p.key_heads + key_head) * dk, v_ch = 2u * p.key_heads * dk + head * p.dv + c0;
    float* S = p.state + (((size_t)slot * p.heads + head) * dk) * p.dv + c0 + CP * j;
    float st[PER][CP];
#pragma unroll
    for (int e = 0; e < PER; ++e) {
        const float* at = S + (size_t)min(c * PER + e, dk - 1u) * p.dv;
        if constexpr (CP == 4) *reinterpret_cast<sc_f4*>(st[e]) = *reinterpret_cast<const sc_f4*>(at);
        else st[e][0] = at[0];
    }
    const float rate = expf(bf16_to_f32(p.a_log[head])), dt_bias = bf16_to_f32(p.dt_bias[head]), skip = DELTA ? 0.0f : bf16_to_f32(p.skip[head]);
    const bool keys_owner = head % ratio == 0u && c0 == 0u;
    for (uint32_t t = 0; t < seq_rows; ++t) {
        const float* row = p.proj + (size_t)(base + t) * p.proj_stride;
        const float step = scan_softplus(row[p.a_at + head] + dt_bias), decay = expf(-rate * step);
        const float beta = DELTA ? scan_sigmoid(row[p.b_at + head]) : step;
        float* past = p.history + ((size_t)slot * p.history_rows + (first + t) % p.history_rows) * p.channels;
        float qq = 0.0f, kk = 0.0f, qk = 0.0f;
        for (uint32_t d = tid; d < 16u * PER; d += 256u) {
            float q = 0.0f, k = 0.0f;
            if (d < dk) {
                q = scan_filter(p, slot, base, first, t, q_ch + d);
                k = scan_filter(p, slot, base, first, t, k_ch + d);
                if (keys_owner) {
                    past[q_ch + d] = row[p.conv_at + q_ch + d];
                    past[k_ch + d] = row[p.conv_at + k_ch + d];
                }
            }
            qs[d] = q;
            ks[d] = k;
            qq = fmaf(q, q, qq);
            kk = fmaf(k, k, kk);
            qk = fmaf(q, k, qk);
        }
        if (tid >= 256u - COLS) {                    // the last threads have the fewest q and k channels
            const uint32_t d = tid - (256u - COLS);
            vs[d] = scan_filter(p, slot, base, first, t, v_ch + d);
            past[v_ch + d] = row[p.conv_at + v_ch + d];
        }
        qq = wave_sum_bcast(qq);
        kk = wave_sum_bcast(kk);
        qk = wave_sum_bcast(qk);
        if (lane == 0) { red[0][wave] = qq; red[1][wave] = kk; red[2][wave] = qk; }
        __syncthreads();
        float sq[CP] = {}, sk[CP] = {};              // S^T q, S^T k over this thread's rows
#pragma unroll
        for (int e = 0; e < PER; ++e) {
            const float q = qs[c * PER + e], k = DELTA ? ks[c * PER + e] : 0.0f;
#pragma unroll
            for (int u = 0; u < CP; ++u) {
                sq[u] = fmaf(st[e][u], q, sq[u]);
                if (DELTA) sk[u] = fmaf(st[e][u], k, sk[u]);
            }
        }
#pragma unroll
        for (int u = 0; u < CP; ++u) {
            sq[u] += shfl_xor_f(sq[u], 16);
            sq[u] += shfl_xor_f(sq[u], 32);
            if (DELTA) { sk[u] += shfl_xor_f(sk[u], 16); sk[u] += shfl_xor_f(sk[u], 32); }
            if (lane < 16u) { part[0][wave][CP * j + u] = sq[u]; if (DELTA) part[1][wave][CP * j + u] = sk[u]; }
        }
        const float sum_qk = (red[2][0] + red[2][1]) + (red[2][2] + red[2][3]);
        float qn = 1.0f, kn = 1.0f;
        if (DELTA) {
            qn = p.q_scale / sqrtf((red[0][0] + red[0][1]) + (red[0][2] + red[0][3]) + 1e-6f);
            kn = 1.0f / sqrtf((red[1][0] + red[1][1]) + (red[1][2] + red[1][3]) + 1e-6f);
        }
        __syncthreads();
        float ku[CP], o[CP];
#pragma unroll
        for (int u = 0; u < CP; ++u) {
            const uint32_t d = CP * j + u;
            const float v = vs[d], q_old = (part[0][0][d] + part[0][1][d]) + (part[0][2][d] + part[0][3][d]);
            const float k_old = DELTA ? (part[1][0][d] + part[1][1][d]) + (part[1][2][d] + part[1][3][d]) : 0.0f;
            ku[u] = kn * (DELTA ? beta * (v - decay * (k_old * kn)) : beta * v);
            o[u] = fmaf(decay, q_old * qn, sum_qk * qn * ku[u]) + skip * v;
        }
        if (tid < 16u) {
            float* out = p.out + (size_t)(base + t) * p.out_stride + head * p.out_head + c0 + CP * j;
#pragma unroll
            for (int u = 0; u < CP; ++u) out[u] = o[u];
        }
#pragma unroll
        for (int e = 0; e < PER; ++e) {
            const float k = ks[c * PER + e];
#pragma unroll
            for (int u = 0; u < CP; ++u) st[e][u] = fmaf(decay, st[e][u], k * ku[u]);
        }
        __syncthreads();                             // this row's LDS is free
    }
#pragma unroll
    for (int e = 0; e < PER; ++e)
        if (c * PER + e < dk) {
            float* at = S + (size_t)(c * PER + e) * p.dv;
            if constexpr (CP == 4) *reinterpret_cast<sc_f4*>(at) = *reinterpret_cast<sc_f4*>(st[e]);
            else at[0] = st[e][0];
        }
}

// ---- chunked form: filter, silu, unit vectors ----------------------------------------------------------------
// A wave per (segment, SCAN_RUN rows); a segment is a head of q, k or v.  TAPS 4: the run's inputs are requested at once and
// slide through registers.  Rows past the last one, up to a multiple of SCAN_CHUNK, are written as zeros.  One more segment
// turns the gates' inputs into a row per head.
constexpr uint32_t SCAN_RUN = 16;

template <bool DELTA, int NV, int TAPS, bool FAST>
__global__ __launch_bounds__(256) void scan_filter_kernel(ScanParams p) {
    const uint32_t lane = threadIdx.x & 63u, seg = blockIdx.y * 4u + (threadIdx.x >> 6), t0 = blockIdx.x * SCAN_RUN;
    if (seg > 2u * p.key_heads + p.heads) return;
    if (seg == 2u * p.key_heads + p.heads) {
        const uint32_t t = t0 + (lane & 15u);
        const float* row = p.proj + (size_t)min(t, p.n_rows - 1u) * p.proj_stride;
        for (uint32_t h = lane >> 4; h < p.heads; h += 4u) {
            p.in_a[(size_t)h * p.rows_p + t] = row[p.a_at + h];
            if (DELTA) p.in_b[(size_t)h * p.rows_p + t] = row[p.b_at + h];
        }
        return;
    }
    const bool key = seg < 2u * p.key_heads;
    const uint32_t dim = key ? p.dk : p.dv, at = key ? seg * p.dk : 2u * p.key_heads * p.dk + (seg - 2u * p.key_heads) * p.dv;
    float* out = key ? p.q_of(seg, t0) : p.v_of(seg - 2u * p.key_heads, t0);
    if (t0 >= p.n_rows) {                            // a run behind the last row: there is no row of proj to read
        for (uint32_t e = lane; e < SCAN_RUN * dim; e += 64u) out[e] = 0.0f;
        return;
    }
    const float factor = seg < p.key_heads ? p.q_scale : 1.0f;
    const uint32_t slot = p.rows.slot, first = p.rows.position;
    constexpr int HIST = TAPS > 0 ? TAPS - 1 : 0, IN = TAPS > 0 ? SCAN_RUN + HIST : 1;
    uint32_t ch[NV];
    float w[NV][TAPS > 0 ? TAPS : 1], in[NV][IN], bias[NV];
#pragma unroll
    for (int e = 0; e < NV; ++e) {
        ch[e] = at + min(lane + 64u * e, dim - 1u);
        if (TAPS > 0) {
            bias[e] = p.conv_bias ? bf16_to_f32(p.conv_bias[ch[e]]) : 0.0f;
#pragma unroll
            for (int s = 0; s < TAPS; ++s) w[e][s] = bf16_to_f32(p.conv[(size_t)ch[e] * TAPS + s]);
            const float* x = p.proj + (size_t)t0 * p.proj_stride + p.conv_at;
#pragma unroll
            for (uint32_t t = 0; t < SCAN_RUN; ++t) in[e][HIST + t] = x[(size_t)(t0 + t < p.n_rows ? t : 0u) * p.proj_stride + ch[e]];
#pragma unroll
            for (int s = 0; s < HIST; ++s) in[e][s] = scan_input(p, slot, 0, first, (int32_t)t0 + s - HIST, ch[e]);
        }
    }
#pragma unroll
    for (uint32_t t = 0; t < SCAN_RUN; ++t) {
        const bool live = t0 + t < p.n_rows;         // uniform
        float z[NV], ss = 0.0f;
#pragma unroll
        for (int e = 0; e < NV; ++e) {
            if (TAPS > 0) {
                float a = bias[e];
#pragma unroll
                for (int s = 0; s < TAPS; ++s) a = fmaf(w[e][s], in[e][t + s], a);
                z[e] = FAST ? silu_fast(a) : silu(a);
            } else {
                z[e] = live ? scan_filter(p, slot, 0, first, t0 + t, ch[e]) : 0.0f;
            }
            if (!live) z[e] = 0.0f;
            if (lane + 64u * e < dim) ss = fmaf(z[e], z[e], ss);
        }
        const float f = DELTA && key ? factor / sqrtf(wave_sum_bcast(ss) + 1e-6f) : 1.0f;
#pragma unroll
        for (int e = 0; e < NV; ++e)
            if (lane + 64u * e < dim) out[t * dim + lane + 64u * e] = z[e] * f;
    }
}

// The filter's last taps - 1 inputs, for the rows that follow (after the kernel above has read the old ones).
__global__ __launch_bounds__(256) void scan_history_kernel(ScanParams p) {
    const uint32_t ch = blockIdx.x * 256u + threadIdx.x, back = blockIdx.y + 1u;
    if (ch >= p.channels || back > p.n_rows) return;
    const uint32_t t = p.n_rows - back;
    p.history[((size_t)p.rows.slot * p.history_rows + (p.rows.position + t) % p.history_rows) * p.channels + ch] =
        p.proj[(size_t)t * p.proj_stride + p.conv_at + ch];
}

// ---- chunked form: what needs no state ---------------------------------------------------------------------
// Block (chunk, group of `per` heads of one key head).  The tiles on and below the diagonal of q k^T (and k k^T) are made
// once, dealt to the four waves; W, and for the delta rule L, follow from them head by head.
//   (I + L) X = R for X = [Kt | U0], sixteen rows at a time: the four diagonal blocks of I + L are inverted by forward
//   substitution (a lane per column), X_b = inv_b (R_b - sum_{m < b} L_bm X_m) runs on the matrix cores, a wave per
//   sixteen columns, its X in the accumulators, where it stands as the next product's B operand.
template <bool DELTA>
__global__ __launch_bounds__(256, 2) void scan_prep_kernel(ScanParams p, uint32_t per) {
    constexpr int JOBS = DELTA ? 5 : 3;              // tiles of one wave: ten of q k^T, ten of k k^T
    extern __shared__ __attribute__((aligned(16))) float sc_lds[];
    __shared__ double X[64];
    __shared__ float beta[64], bg[64];
    __shared__ __attribute__((aligned(16))) float inv[DELTA ? 4 : 1][16][20], turn[DELTA ? 4 : 1][16][20];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i = lane & 15u, g = lane >> 4;
    const uint32_t chunk = blockIdx.x, ratio = p.heads / p.key_heads, groups = (ratio + per - 1u) / per;
    const uint32_t key_head = blockIdx.y / groups, h0 = (blockIdx.y % groups) * per, h1 = min(h0 + per, ratio);
    const uint32_t dk = p.dk, dv = p.dv, ld = dk + 4u, t0 = chunk * SCAN_CHUNK;
    const sc_f4 zero = sc_f4{0.0f, 0.0f, 0.0f, 0.0f};
    float *ks = sc_lds, *qs = ks + 64u * ld, *L = qs;        // [64][ld], [64][ld] and then [64][68] (delta)
    // the gates' inputs of a head, a row per lane, requested a head ahead
    float in_a = 0.0f, in_b = 0.0f;
    auto fetch_gates = [&](uint32_t h) {
        const size_t at = (size_t)(key_head * ratio + h) * p.rows_p + t0 + lane;
        in_a = p.in_a[at];
        if (DELTA) in_b = p.in_b[at];
    };
    if (wave == 3u) fetch_gates(h0);
    {
        const float *q = p.q_of(key_head, t0), *k = p.k_of(key_head, t0);             // sixteen lanes to a row
        for (uint32_t r = tid >> 4; r < 64u; r += 16u)
            for (uint32_t d = (tid & 15u) * 4u; d < dk; d += 64u) {
                *reinterpret_cast<sc_f4*>(qs + r * ld + d) = *reinterpret_cast<const sc_f4*>(q + r * dk + d);
                *reinterpret_cast<sc_f4*>(ks + r * ld + d) = *reinterpret_cast<const sc_f4*>(k + r * dk + d);
            }
    }
    scan_barrier();
    if (h0 == 0u) {                                  // one block of the key head: k^T for the chain
        float* kt = p.k_t + ((size_t)chunk * p.key_heads + key_head) * 64u * dk;
        for (uint32_t n = wave; n < dk / 4u; n += 4u) {          // n = 4 tile + row tile
            sc_f4 v;
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = ks[(16u * (n & 3u) + 4u * g + r) * ld + 16u * (n >> 2) + i];
            *reinterpret_cast<sc_f4*>(kt + n * 256u + lane * 4u) = v;
        }
    }
    sc_f4 gram[JOBS];
    auto job = [&](uint32_t n, uint32_t& ti, uint32_t& tm) {         // tile n of ten, row by row
        ti = n < 1u ? 0u : n < 3u ? 1u : n < 6u ? 2u : 3u;
        tm = n - ti * (ti + 1u) / 2u;
    };
#pragma unroll
    for (int n = 0; n < JOBS; ++n) {
        const uint32_t all = wave + 4u * n;
        gram[n] = zero;
        if (all >= (DELTA ? 20u : 10u)) continue;    // uniform
        uint32_t ti, tm;
        job(all < 10u ? all : all - 10u, ti, tm);
        const float *a0 = (all < 10u ? qs : ks) + (16u * ti + i) * ld + 4u * g, *b0 = ks + (16u * tm + i) * ld + 4u * g;
        sc_f4 odd = zero;
#pragma unroll 4
        for (uint32_t d = 0; d < dk; d += 16u) {
            const sc_f4 a = *reinterpret_cast<const sc_f4*>(a0 + d), b = *reinterpret_cast<const sc_f4*>(b0 + d);
            gram[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[0], b[0], gram[n], 0, 0, 0);
            odd = __builtin_amdgcn_mfma_f32_16x16x4f32(a[1], b[1], odd, 0, 0, 0);
            gram[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[2], b[2], gram[n], 0, 0, 0);
            odd = __builtin_amdgcn_mfma_f32_16x16x4f32(a[3], b[3], odd, 0, 0, 0);
        }
        gram[n] += odd;
    }
    for (uint32_t h = h0; h < h1; ++h) {
        const uint32_t head = key_head * ratio + h;
        const size_t cell = (size_t)chunk * p.heads + head;
        float* gates = p.gates + cell * 192u;
        if (wave == 3u) {                            // rows past the end: no decay, u = 0
            const bool live = t0 + lane < p.n_rows;
            const float step = scan_softplus(in_a + bf16_to_f32(p.dt_bias[head]));
            double x = live ? (double)(expf(bf16_to_f32(p.a_log[head])) * step) : 0.0;
            const float b = live ? (DELTA ? scan_sigmoid(in_b) : step) : 0.0f;
            if (h + 1u < h1) fetch_gates(h + 1u);
#pragma unroll
            for (int off = 1; off < 64; off *= 2) {
                const double y = __shfl_up(x, off, 64);
                x += (int)lane >= off ? y : 0.0;
            }
            X[lane] = x;
            beta[lane] = b;
            const float G = expf(-(float)x);
            bg[lane] = b * G;
            gates[lane] = G;
            gates[64u + lane] = expf(-(float)(__shfl(x, 63, 64) - x));
            gates[128u + lane] = b;
        }
        scan_barrier();                             // and, the first time, everyone is done with q
        float* W = p.w + cell * 4096u;
#pragma unroll
        for (int n = 0; n < JOBS; ++n) {
            const uint32_t all = wave + 4u * n;
            if (all >= (DELTA ? 20u : 10u)) continue;
            uint32_t ti, tm;
            job(all < 10u ? all : all - 10u, ti, tm);
            const uint32_t col = 16u * tm + i;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const uint32_t row = 16u * ti + 4u * g + r;
                const float f = col <= row ? expf(-(float)(X[row] - X[col])) : 0.0f;
                if (all < 10u) W[row * 64u + col] = f * gram[n][r];
                else L[row * 68u + col] = col < row ? beta[row] * f * gram[n][r] : 0.0f;
            }
        }
        // the tiles above the diagonal
        for (uint32_t n = wave; n < 6u; n += 4u) {
            const uint32_t ti = n < 3u ? 0u : n < 5u ? 1u : 2u, tm = n < 3u ? n + 1u : n < 5u ? n - 1u : 3u;
#pragma unroll
            for (int r = 0; r < 4; ++r) W[(16u * ti + 4u * g + r) * 64u + 16u * tm + i] = 0.0f;
        }
        if (DELTA) {
            scan_barrier();
            if (wave == 0) {                         // lane group g: the diagonal block g, column i of its inverse
                const float* D = L + (16u * g) * 68u + 16u * g;
                float x[16];
#pragma unroll
                for (int r = 0; r < 16; ++r) {
                    float a = (uint32_t)r == i ? 1.0f : 0.0f, a1 = 0.0f;
#pragma unroll
                    for (int m = 0; m < r; m += 4) {
                        const sc_f4 l = *reinterpret_cast<const sc_f4*>(D + r * 68 + m);
#pragma unroll
                        for (int u = 0; u < 4; ++u)
                            if (m + u < r) {
                                if (u & 1) a1 = fmaf(-l[u], x[m + u], a1);
                                else a = fmaf(-l[u], x[m + u], a);
                            }
                    }
                    x[r] = a + a1;
                }
#pragma unroll
                for (int r = 0; r < 16; ++r) inv[g][r][i] = x[r];
            }
            // the right sides of this wave's tiles, values first: their loads run under the inversion
            const uint32_t vt = dv / 16u, tiles = (dk + dv) / 16u;
            const float* vbase = p.v_of(head, t0);
            const uint32_t v_lane = 4u * g * dv + i;
            auto fetch_v = [&](uint32_t tile, sc_f4 (&R)[4]) {
#pragma unroll
                for (int b = 0; b < 4; ++b)
#pragma unroll
                    for (int r = 0; r < 4; ++r) R[b][r] = (vbase + (16u * b + r) * dv + 16u * tile)[v_lane];
            };
            sc_f4 R[4];
            if (wave < vt) fetch_v(wave, R);
            scan_barrier();
            for (uint32_t tile = wave; tile < tiles; tile += 4u) {
                const bool keys = tile >= vt;        // uniform
                asm volatile("" ::: "memory");       // the tiles of L are read again, not kept in registers
                sc_f4 x[4];
#pragma unroll
                for (int b = 0; b < 4; ++b)
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        x[b][r] = keys ? bg[16u * b + 4u * g + r] * ks[(16u * b + 4u * g + r) * ld + 16u * (tile - vt) + i] : beta[16u * b + 4u * g + r] * R[b][r];
                if (tile + 4u < vt) fetch_v(tile + 4u, R);
#pragma unroll
                for (int b = 0; b < 4; ++b) {
                    sc_f4 a0 = zero, a1 = zero;
#pragma unroll
                    for (int m = 0; m < b; ++m) {
                        const sc_f4 l = *reinterpret_cast<const sc_f4*>(L + (16u * b + i) * 68u + 16u * m + 4u * g);
                        a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(l[0], x[m][0], a0, 0, 0, 0);
                        a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(l[1], x[m][1], a1, 0, 0, 0);
                        a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(l[2], x[m][2], a0, 0, 0, 0);
                        a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(l[3], x[m][3], a1, 0, 0, 0);
                    }
                    const sc_f4 rest = x[b] - (a0 + a1), d = *reinterpret_cast<const sc_f4*>(&inv[b][i][4u * g]);
                    a0 = zero;
                    a1 = zero;
                    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(d[0], rest[0], a0, 0, 0, 0);
                    a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(d[1], rest[1], a1, 0, 0, 0);
                    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(d[2], rest[2], a0, 0, 0, 0);
                    a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(d[3], rest[3], a1, 0, 0, 0);
                    x[b] = a0 + a1;
                    if (!keys) {
                        *reinterpret_cast<sc_f4*>(p.u0 + cell * 64u * dv + (tile * 4u + b) * 256u + lane * 4u) = x[b];
                    } else {                         // rows to lanes, within the wave
#pragma unroll
                        for (int r = 0; r < 4; ++r) turn[wave][4u * g + r][i] = x[b][r];
                        __builtin_amdgcn_wave_barrier();
                        const sc_f4 v = *reinterpret_cast<const sc_f4*>(&turn[wave][i][4u * g]);
                        __builtin_amdgcn_wave_barrier();
                        *reinterpret_cast<sc_f4*>(p.kt + cell * 64u * dk + (b * (dk / 16u) + tile - vt) * 256u + lane * 4u) = v;
                    }
                }
            }
        }
        if (h + 1u < h1) scan_barrier();             // X, beta and L are free
    }
}

// ---- chunked form: the chunks in order -------------------------------------------------------------------------
// Waves 0 .. 3 carry the state: wave w owns the state tiles w TW .. of sixteen rows, and the chunk's rows 16 w .. + 15 of U.
// Waves 4 .. 7 make the outputs of the rows 16 (w - 4) .. + 15.  Per chunk two phases, a barrier behind each:
//   first:  U = U0 - Kt S (SSD: dt V) into LDS;      o = G S^T q
//   second: S = G_63 S + k^T c U, S into LDS;        o += W U, stored
// Each wave requests its operands PF chunks ahead, in PF sets of registers that take turns.  KT: state tiles (16 KT >= dk, KT
// a multiple of 4).
template <bool DELTA, int KT, int PF>
__global__ __launch_bounds__(512) void scan_chain_kernel(ScanParams p, uint32_t chunks) {
    constexpr int TW = KT / 4;
    __shared__ __attribute__((aligned(16))) sc_f4 ss[KT][64], us[4][64], cu[4][64];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i = lane & 15u, g = lane >> 4;
    const uint32_t head = blockIdx.x, c0 = blockIdx.y * 16u, dk = p.dk, dv = p.dv, kt = dk / 16u, w = wave & 3u;
    const uint32_t key_head = head / (p.heads / p.key_heads);
    const sc_f4 zero = sc_f4{0.0f, 0.0f, 0.0f, 0.0f};
    // every address is a uniform base and a lane's offset that the loop does not change; tiles past the last one of the
    // state repeat it, against zeros in ss
    const uint32_t v_lane = (4u * g * dv + i) * 4u, own = lane * 16u;          // bytes: rows 4 g .. of dv columns, column i; this lane's float4
    auto cell_of = [&](uint32_t n) { return (size_t)n * p.heads + head; };
    auto tile_of = [&](uint32_t t) { return min(t, kt - 1u); };
    auto f4_at = [](const float* base, uint32_t bytes) { return *reinterpret_cast<const sc_f4*>(reinterpret_cast<const char*>(base) + bytes); };
    auto f_at = [](const float* base, uint32_t bytes) { return *reinterpret_cast<const float*>(reinterpret_cast<const char*>(base) + bytes); };
    if (wave < 4u) {
        struct Operands {
            sc_f4 kA[DELTA ? KT : 1], u0, c4;        // first phase
            sc_f4 kT[TW][4];                         // second
            float g63_next;
        };
        float* state = p.state + (((size_t)p.rows.slot * p.heads + head) * dk) * dv + c0;
        sc_f4 S[TW];
        auto fetch_kt = [&](uint32_t n, int t, Operands& o) { o.kA[t] = f4_at(p.kt + cell_of(n) * 64u * dk + (w * kt + tile_of(t)) * 256u, own); };
        auto fetch_u = [&](uint32_t n, Operands& o) {
            const size_t cell = cell_of(n);
            const float* gates = p.gates + cell * 192u + 16u * w;
            if (DELTA) {
                o.u0 = f4_at(p.u0 + cell * 64u * dv + (blockIdx.y * 4u + w) * 256u, own);
            } else {
                o.kA[0] = f4_at(gates + 128, 16u * g);
                const float* v = p.v_of(head, n * SCAN_CHUNK + 16u * w) + c0;
#pragma unroll
                for (int r = 0; r < 4; ++r) o.u0[r] = f_at(v + r * dv, v_lane);
            }
            o.c4 = f4_at(gates + 64, 16u * g);
            o.g63_next = p.gates[cell * 192u + 63u];
        };
        auto fetch_k = [&](uint32_t n, int s, Operands& o) {
            const float* k = p.k_t + ((size_t)n * p.key_heads + key_head) * 64u * dk + s * 256;
#pragma unroll
            for (int t = 0; t < TW; ++t) o.kT[t][s] = f4_at(k + tile_of(w * TW + t) * 1024u, own);
        };
        auto keep = [&]() {
#pragma unroll
            for (int t = 0; t < TW; ++t) ss[w * TW + t][lane] = w * TW + t < kt ? S[t] : zero;
        };
        // an operand is requested again, PF chunks on, as soon as its products are under way
        auto chunk = [&](uint32_t n, Operands& o) {
            const uint32_t next = min(n + PF, chunks - 1u);
            const float g63 = o.g63_next;
            sc_f4 u;
            if (DELTA) {
                sc_f4 a0 = zero, a1 = zero, b[KT];
#pragma unroll
                for (int t = 0; t < KT; ++t) b[t] = ss[t][lane];
                __builtin_amdgcn_sched_barrier(0);   // every read is under way before the first product
#pragma unroll
                for (int t = 0; t < KT; ++t) {
                    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kA[t][0], b[t][0], a0, 0, 0, 0);
                    a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kA[t][1], b[t][1], a1, 0, 0, 0);
                    a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kA[t][2], b[t][2], a0, 0, 0, 0);
                    a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kA[t][3], b[t][3], a1, 0, 0, 0);
                    fetch_kt(next, t, o);
                }
                u = o.u0 - (a0 + a1);
            } else {
                u = o.kA[0] * o.u0;
            }
            us[w][lane] = u;
            cu[w][lane] = u * o.c4;
            fetch_u(next, o);
            scan_barrier();
            sc_f4 b[4];
#pragma unroll
            for (int s = 0; s < 4; ++s) b[s] = cu[s][lane];
#pragma unroll
            for (int t = 0; t < TW; ++t) S[t] *= g63;
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int s = 0; s < 4; ++s) {
#pragma unroll
                for (int r = 0; r < 4; ++r)
#pragma unroll
                    for (int t = 0; t < TW; ++t) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(o.kT[t][s][r], b[s][r], S[t], 0, 0, 0);
                fetch_k(next, s, o);
            }
            keep();
            scan_barrier();
        };
        Operands o[PF];
#pragma unroll
        for (int f = 0; f < PF; ++f) {
            const uint32_t n = min((uint32_t)f, chunks - 1u);
            if (DELTA) {
#pragma unroll
                for (int t = 0; t < KT; ++t) fetch_kt(n, t, o[f]);
            }
            fetch_u(n, o[f]);
#pragma unroll
            for (int s = 0; s < 4; ++s) fetch_k(n, s, o[f]);
        }
#pragma unroll
        for (int t = 0; t < TW; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) S[t][r] = (state + (size_t)(16u * tile_of(w * TW + t) + r) * dv)[4u * g * dv + i];
        keep();
        scan_barrier();
        for (uint32_t n = 0; n < chunks; n += PF) {
#pragma unroll
            for (int f = 0; f < PF; ++f)
                if (n + f < chunks) chunk(n + f, o[f]);
        }
#pragma unroll
        for (int t = 0; t < TW; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (w * TW + t < kt) (state + (size_t)(16u * (w * TW + t) + r) * dv)[4u * g * dv + i] = S[t][r];
        return;
    }
    struct Operands {
        sc_f4 qA[KT], G4;                            // first phase
        sc_f4 wA[4];                                 // second
        float v[4];
    };
    const float skip = DELTA ? 0.0f : bf16_to_f32(p.skip[head]);
    const uint32_t q_lane = (i * dk + 4u * g) * 4u, o_lane = 4u * g * p.out_stride + i;
    auto fetch_q = [&](uint32_t n, int t, Operands& o) { o.qA[t] = f4_at(p.q_of(key_head, n * SCAN_CHUNK + 16u * w) + 16u * tile_of(t), q_lane); };
    auto fetch_w = [&](uint32_t n, int t, Operands& o) { o.wA[t] = f4_at(p.w + cell_of(n) * 4096u + 16u * w * 64u + 16 * t, (i * 64u + 4u * g) * 4u); };
    auto fetch_rest = [&](uint32_t n, Operands& o) {
        o.G4 = f4_at(p.gates + cell_of(n) * 192u + 16u * w, 16u * g);
        const float* v = p.v_of(head, n * SCAN_CHUNK + 16u * w) + c0;
#pragma unroll
        for (int r = 0; r < 4; ++r) o.v[r] = DELTA ? 0.0f : f_at(v + r * dv, v_lane);
    };
    auto chunk = [&](uint32_t n, Operands& op) {
        const uint32_t next = min(n + PF, chunks - 1u);
        sc_f4 o = zero, o1 = zero, b[KT];
#pragma unroll
        for (int t = 0; t < KT; ++t) b[t] = ss[t][lane];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int t = 0; t < KT; ++t) {
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(op.qA[t][0], b[t][0], o, 0, 0, 0);
            o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(op.qA[t][1], b[t][1], o1, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(op.qA[t][2], b[t][2], o, 0, 0, 0);
            o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(op.qA[t][3], b[t][3], o1, 0, 0, 0);
            fetch_q(next, t, op);
        }
        o = (o + o1) * op.G4;
        o1 = zero;
        scan_barrier();
#pragma unroll
        for (int t = 0; t < 4; ++t) b[t] = us[t][lane];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int t = 0; t < 4; ++t) {                // W is zero above its diagonal
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(op.wA[t][0], b[t][0], o, 0, 0, 0);
            o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(op.wA[t][1], b[t][1], o1, 0, 0, 0);
            o = __builtin_amdgcn_mfma_f32_16x16x4f32(op.wA[t][2], b[t][2], o, 0, 0, 0);
            o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(op.wA[t][3], b[t][3], o1, 0, 0, 0);
            fetch_w(next, t, op);
        }
        o += o1;
        const uint32_t t0 = n * SCAN_CHUNK + 16u * w;
        float* out = p.out + (size_t)t0 * p.out_stride + head * p.out_head + c0;
#pragma unroll
        for (int r = 0; r < 4; ++r)
            if (t0 + 4u * g + r < p.n_rows) (out + (size_t)r * p.out_stride)[o_lane] = o[r] + skip * op.v[r];
        fetch_rest(next, op);
        scan_barrier();
    };
    Operands o[PF];
#pragma unroll
    for (int f = 0; f < PF; ++f) {
        const uint32_t n = min((uint32_t)f, chunks - 1u);
#pragma unroll
        for (int t = 0; t < KT; ++t) fetch_q(n, t, o[f]);
#pragma unroll
        for (int t = 0; t < 4; ++t) fetch_w(n, t, o[f]);
        fetch_rest(n, o[f]);
    }
    scan_barrier();
    for (uint32_t n = 0; n < chunks; n += PF) {
#pragma unroll
        for (int f = 0; f < PF; ++f)
            if (n + f < chunks) chunk(n + f, o[f]);
    }
}

// ---- the gated norm behind a recurrence -------------------------------------------------------------------------
struct GatedNormParams {
    const float *x, *gate;
    const uint16_t* weight;
    void* out;
    uint64_t x_head;                     // from a head of x to the next
    uint32_t x_stride, gate_stride, out_stride, rows, heads, dv, dv_count, parts;
    float out_scale, eps;
};

template <int ACT>
__device__ __forceinline__ float gated_silu(float z) { return ACT == ACT_FP32 ? silu(z) : silu_fast(z); }

// LANES threads (a piece of a wave, a wave, or several) per (part, row), 256 or LANES threads per block.  VEC: four
// neighbouring elements at a time, KEEP of them in registers; else element by element, those past the registers read
// twice.
template <int ACT, bool FIRST, int LANES, int KEEP, bool VEC>
__global__ __launch_bounds__(LANES > 256 ? LANES : 256) void gated_norm_kernel(GatedNormParams p) {
    constexpr uint32_t PER_BLOCK = LANES < 256 ? 256 / LANES : 1, E = VEC ? 4 : 1;
    __shared__ float red[LANES > 64 ? LANES / 64 : 1];
    const uint32_t tid = threadIdx.x % LANES, part = blockIdx.y * PER_BLOCK + threadIdx.x / LANES, row = blockIdx.x;
    if (LANES <= 64 && part >= p.parts) return;
    const uint32_t n = p.heads * p.dv_count / p.parts, e0 = part * n;
    const float *x = p.x + (size_t)row * p.x_stride, *gate = p.gate + (size_t)row * p.gate_stride;
    struct Place { size_t x; uint32_t at; };         // where element e lies in x, and in gate and out
    auto place = [&](uint32_t e) {
        const uint32_t head = e / p.dv_count, d = e % p.dv_count;
        return Place{head * p.x_head + d, head * p.dv + d};
    };
    float xs[KEEP][E], zs[KEEP][E], ss = 0.0f;
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const Place o = place(e0 + min((tid + LANES * u) * E, n - E));
        if constexpr (VEC) {
            *reinterpret_cast<sc_f4*>(xs[u]) = *reinterpret_cast<const sc_f4*>(x + o.x);
            *reinterpret_cast<sc_f4*>(zs[u]) = *reinterpret_cast<const sc_f4*>(gate + o.at);
        } else {
            xs[u][0] = x[o.x];
            zs[u][0] = gate[o.at];
        }
    }
#pragma unroll
    for (int u = 0; u < KEEP; ++u)
#pragma unroll
        for (uint32_t e = 0; e < E; ++e) {
            if (FIRST) xs[u][e] *= gated_silu<ACT>(zs[u][e]);
            if ((tid + LANES * u) * E < n) ss = fmaf(xs[u][e], xs[u][e], ss);
        }
    if (!VEC)
        for (uint32_t e = tid + LANES * KEEP; e < n; e += LANES) {
            const Place o = place(e0 + e);
            const float v = FIRST ? x[o.x] * gated_silu<ACT>(gate[o.at]) : x[o.x];
            ss = fmaf(v, v, ss);
        }
    if (LANES >= 64) {
        ss = wave_sum_bcast(ss);
        if (LANES > 64) {
            if ((tid & 63u) == 0) red[tid >> 6] = ss;
            __syncthreads();
            ss = 0.0f;
#pragma unroll
            for (int u = 0; u < LANES / 64; ++u) ss += red[u];
        }
    } else {
#pragma unroll
        for (int off = LANES / 2; off >= 1; off >>= 1) ss += shfl_xor_f(ss, off);
    }
    const float inv = p.out_scale / sqrtf(ss / (float)n + p.eps);
    act_t<ACT>* out = static_cast<act_t<ACT>*>(p.out) + (size_t)row * p.out_stride;
    auto value = [&](uint32_t at, float v, float z) {
        return FIRST ? v * inv * bf16_to_f32(p.weight[at]) : v * inv * bf16_to_f32(p.weight[at % p.dv]) * gated_silu<ACT>(z);
    };
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        if ((tid + LANES * u) * E >= n) break;
        const uint32_t at = place(e0 + (tid + LANES * u) * E).at;
        if constexpr (VEC) {
            float v[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = value(at + e, xs[u][e], zs[u][e]);
            if constexpr (ACT == ACT_FP32) *reinterpret_cast<sc_f4*>(out + at) = sc_f4{v[0], v[1], v[2], v[3]};
            else *reinterpret_cast<uint2*>(out + at) = make_uint2(f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16), f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16));
        } else {
            out[at] = f32_to_act<ACT>(value(at, xs[u][0], zs[u][0]));
        }
    }
    if (!VEC)
        for (uint32_t e = tid + LANES * KEEP; e < n; e += LANES) {
            const Place o = place(e0 + e);
            const float z = gate[o.at];
            out[o.at] = f32_to_act<ACT>(value(o.at, FIRST ? x[o.x] * gated_silu<ACT>(z) : x[o.x], z));
        }
}

}  // namespace nvmai
