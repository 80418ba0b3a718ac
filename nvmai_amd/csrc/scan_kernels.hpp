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
    float* out;                          // [rows, out_stride]
    SeqRows rows;
    uint32_t proj_stride, out_stride, n_rows, heads, key_heads, dk, dv, taps, history_rows, conv_at, a_at, b_at, channels;
    float q_scale;
    // chunked form
    float* mixed;                        // [rows, channels]: q | k | v after filter, silu and norm
    float *w, *gates;                    // [chunk, head, 64, 64], [chunk, head, 3, 64]: G, e^(X_i - X_63), dt
    float *kt, *u0;                      // [chunk, head, 64, dk], [chunk, head, 64, dv]
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

// ---- recurrent form --------------------------------------------------------------------------------------
// Block (head, sixteen columns, sequence): thread (column j = tid % 16, group c = tid / 16) owns the state rows
// c PER .. c PER + PER - 1 of its column.  Only the block that owns a channel (its value columns; the q and k of a key
// head: the first block of its first head) writes the channel's history, in rows that no block of the launch reads.
template <bool DELTA, int PER>
__global__ __launch_bounds__(256) void scan_recurrent_kernel(ScanParams p, uint32_t seq_rows) {
    __shared__ __attribute__((aligned(16))) float qs[16 * PER], ks[16 * PER];
    __shared__ float vs[16], red[3][4], part[2][4][16];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, j = tid & 15u, c = tid >> 4;
    const uint32_t head = blockIdx.x, c0 = blockIdx.y * 16u, seq = blockIdx.z, dk = p.dk;
    const uint32_t ratio = p.heads / p.key_heads, key_head = head / ratio;
    const uint32_t base = seq * seq_rows, slot = p.rows.slot_of(base), first = p.rows.position_of(base);
    const uint32_t q_ch = key_head * dk, k_ch = (p.key_heads + key_head) * dk, v_ch = 2u * p.key_heads * dk + head * p.dv + c0;
    float* S = p.state + (((size_t)slot * p.heads + head) * dk) * p.dv + c0 + j;
    float st[PER];
#pragma unroll
    for (int e = 0; e < PER; ++e) st[e] = S[(size_t)min(c * PER + e, dk - 1u) * p.dv];
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
        if (tid >= 240u) {                           // the last sixteen threads have the fewest q and k channels
            vs[j] = scan_filter(p, slot, base, first, t, v_ch + j);
            past[v_ch + j] = row[p.conv_at + v_ch + j];
        }
        qq = wave_sum_bcast(qq);
        kk = wave_sum_bcast(kk);
        qk = wave_sum_bcast(qk);
        if (lane == 0) { red[0][wave] = qq; red[1][wave] = kk; red[2][wave] = qk; }
        __syncthreads();
        float sq = 0.0f, sk = 0.0f;                  // S^T q, S^T k over this thread's rows
#pragma unroll
        for (int e = 0; e < PER; ++e) {
            sq = fmaf(st[e], qs[c * PER + e], sq);
            if (DELTA) sk = fmaf(st[e], ks[c * PER + e], sk);
        }
        sq += shfl_xor_f(sq, 16);
        sq += shfl_xor_f(sq, 32);
        if (DELTA) { sk += shfl_xor_f(sk, 16); sk += shfl_xor_f(sk, 32); }
        if (lane < 16u) { part[0][wave][j] = sq; if (DELTA) part[1][wave][j] = sk; }
        const float sum_qk = (red[2][0] + red[2][1]) + (red[2][2] + red[2][3]);
        float qn = 1.0f, kn = 1.0f;
        if (DELTA) {
            qn = p.q_scale / sqrtf((red[0][0] + red[0][1]) + (red[0][2] + red[0][3]) + 1e-6f);
            kn = 1.0f / sqrtf((red[1][0] + red[1][1]) + (red[1][2] + red[1][3]) + 1e-6f);
        }
        const float v = vs[j];
        __syncthreads();
        sq = (part[0][0][j] + part[0][1][j]) + (part[0][2][j] + part[0][3][j]);
        if (DELTA) sk = (part[1][0][j] + part[1][1][j]) + (part[1][2][j] + part[1][3][j]);
        const float u = DELTA ? beta * (v - decay * (sk * kn)) : beta * v, ku = kn * u;
        if (tid < 16u) p.out[(size_t)(base + t) * p.out_stride + head * p.dv + c0 + j] = fmaf(decay, sq * qn, sum_qk * qn * ku) + skip * v;
#pragma unroll
        for (int e = 0; e < PER; ++e) st[e] = fmaf(decay, st[e], ks[c * PER + e] * ku);
        __syncthreads();                             // this row's LDS is free
    }
#pragma unroll
    for (int e = 0; e < PER; ++e)
        if (c * PER + e < dk) S[(size_t)(c * PER + e) * p.dv] = st[e];
}

// ---- chunked form: filter, silu, unit vectors ----------------------------------------------------------------
// A wave per (segment, SCAN_RUN rows); a segment is a head of q, k or v.  TAPS 4: the inputs slide through registers.
constexpr uint32_t SCAN_RUN = 16;

template <bool DELTA, int NV, int TAPS>
__global__ __launch_bounds__(256) void scan_filter_kernel(ScanParams p) {
    const uint32_t lane = threadIdx.x & 63u, seg = blockIdx.y * 4u + (threadIdx.x >> 6), t0 = blockIdx.x * SCAN_RUN;
    if (seg >= 2u * p.key_heads + p.heads) return;
    const bool key = seg < 2u * p.key_heads;
    const uint32_t dim = key ? p.dk : p.dv, at = key ? seg * p.dk : 2u * p.key_heads * p.dk + (seg - 2u * p.key_heads) * p.dv;
    const float factor = seg < p.key_heads ? p.q_scale : 1.0f;
    const uint32_t slot = p.rows.slot, first = p.rows.position, t1 = min(t0 + SCAN_RUN, p.n_rows);
    uint32_t ch[NV];
    float w[NV][TAPS > 0 ? TAPS : 1], past[NV][TAPS > 0 ? TAPS : 1], bias[NV];
#pragma unroll
    for (int e = 0; e < NV; ++e) {
        ch[e] = at + min(lane + 64u * e, dim - 1u);
        if (TAPS > 0) {
            bias[e] = p.conv_bias ? bf16_to_f32(p.conv_bias[ch[e]]) : 0.0f;
#pragma unroll
            for (int s = 0; s < TAPS; ++s) {
                w[e][s] = bf16_to_f32(p.conv[(size_t)ch[e] * TAPS + s]);
                if (s + 1 < TAPS) past[e][s + 1] = scan_input(p, slot, 0, first, (int32_t)t0 + s + 1 - TAPS, ch[e]);
            }
        }
    }
    for (uint32_t t = t0; t < t1; ++t) {
        float z[NV], ss = 0.0f;
#pragma unroll
        for (int e = 0; e < NV; ++e) {
            if (TAPS > 0) {
#pragma unroll
                for (int s = 0; s + 1 < TAPS; ++s) past[e][s] = past[e][s + 1];
                past[e][TAPS - 1] = p.proj[(size_t)t * p.proj_stride + p.conv_at + ch[e]];
                float a = bias[e];
#pragma unroll
                for (int s = 0; s < TAPS; ++s) a = fmaf(w[e][s], past[e][s], a);
                z[e] = silu(a);
            } else {
                z[e] = scan_filter(p, slot, 0, first, t, ch[e]);
            }
            if (lane + 64u * e < dim) ss = fmaf(z[e], z[e], ss);
        }
        const float f = DELTA && key ? factor / sqrtf(wave_sum_bcast(ss) + 1e-6f) : 1.0f;
#pragma unroll
        for (int e = 0; e < NV; ++e)
            if (lane + 64u * e < dim) p.mixed[(size_t)t * p.channels + ch[e]] = z[e] * f;
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
template <bool DELTA>
__global__ __launch_bounds__(256) void scan_prep_kernel(ScanParams p) {
    extern __shared__ __attribute__((aligned(16))) float sc_lds[];
    __shared__ double X[64];
    __shared__ float beta[64], bg[64];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6, i = lane & 15u, g = lane >> 4;
    const uint32_t chunk = blockIdx.x, head = blockIdx.y, dk = p.dk, dv = p.dv, ld = dk + 4u, t0 = chunk * SCAN_CHUNK;
    float *ks = sc_lds, *qs = ks + 64u * ld, *L = qs;        // [64][ld], [64][ld] and then [64][68] (delta)
    const uint32_t key_head = head / (p.heads / p.key_heads);
    const size_t cell = (size_t)chunk * p.heads + head;
    float* gates = p.gates + cell * 192u;
    if (wave == 0) {                                 // rows past the end: no decay, u = 0
        const bool live = t0 + lane < p.n_rows;
        const float* row = p.proj + (size_t)min(t0 + lane, p.n_rows - 1u) * p.proj_stride;
        const float step = scan_softplus(row[p.a_at + head] + bf16_to_f32(p.dt_bias[head]));
        double x = live ? (double)(expf(bf16_to_f32(p.a_log[head])) * step) : 0.0;
        const float b = live ? (DELTA ? scan_sigmoid(row[p.b_at + head]) : step) : 0.0f;
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
    for (uint32_t e = tid; e < 64u * (dk / 4u); e += 256u) {
        const uint32_t t = e / (dk / 4u), d = (e % (dk / 4u)) * 4u;
        const float* row = p.mixed + (size_t)min(t0 + t, p.n_rows - 1u) * p.channels + key_head * dk + d;
        *reinterpret_cast<sc_f4*>(qs + t * ld + d) = *reinterpret_cast<const sc_f4*>(row);
        *reinterpret_cast<sc_f4*>(ks + t * ld + d) = *reinterpret_cast<const sc_f4*>(row + p.key_heads * dk);
    }
    __syncthreads();
    // the ten tiles on and below the diagonal of W and L, a column of tiles per wave
    float* W = p.w + cell * 4096u;
    sc_f4 low[4];
#pragma unroll
    for (uint32_t ti = 0; ti < 4u; ++ti) {
        const uint32_t tm = wave;
        sc_f4 kk = sc_f4{0.0f, 0.0f, 0.0f, 0.0f}, qk = kk;
        if (tm <= ti) {
            const float *ka = ks + (16u * ti + i) * ld + 4u * g, *qa = qs + (16u * ti + i) * ld + 4u * g, *kb = ks + (16u * tm + i) * ld + 4u * g;
            for (uint32_t d = 0; d < dk; d += 16u) {
                const sc_f4 a = *reinterpret_cast<const sc_f4*>(ka + d), q = *reinterpret_cast<const sc_f4*>(qa + d), b = *reinterpret_cast<const sc_f4*>(kb + d);
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    if (DELTA) kk = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], kk, 0, 0, 0);
                    qk = __builtin_amdgcn_mfma_f32_16x16x4f32(q[r], b[r], qk, 0, 0, 0);
                }
            }
        }
        const uint32_t col = 16u * tm + i;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t row = 16u * ti + 4u * g + r;
            const float ratio = col <= row ? expf(-(float)(X[row] - X[col])) : 0.0f;
            W[row * 64u + col] = col <= row ? ratio * qk[r] : 0.0f;
            low[ti][r] = col < row ? beta[row] * ratio * kk[r] : 0.0f;
        }
    }
    if (!DELTA) return;
    __syncthreads();                                 // everyone is done with q
#pragma unroll
    for (int ti = 0; ti < 4; ++ti)
#pragma unroll
        for (int r = 0; r < 4; ++r) L[(16u * ti + 4u * g + r) * 68u + 16u * wave + i] = low[ti][r];
    __syncthreads();
    for (uint32_t c = tid; c < dk + dv; c += 256u) {
        float x[64];
        float* out = c < dk ? p.kt + cell * 64u * dk + c : p.u0 + cell * 64u * dv + (c - dk);
        const uint32_t out_ld = c < dk ? dk : dv;
        const float* v = p.mixed + 2u * p.key_heads * dk + head * dv + (c < dk ? 0u : c - dk);
#pragma unroll
        for (int r = 0; r < 64; ++r)
            x[r] = c < dk ? bg[r] * ks[r * ld + c] : beta[r] * v[(size_t)min(t0 + r, p.n_rows - 1u) * p.channels];
#pragma unroll
        for (int r = 1; r < 64; ++r) {
            float a0 = 0.0f, a1 = 0.0f;
#pragma unroll
            for (int m = 0; m < r; m += 4) {
                const sc_f4 l = *reinterpret_cast<const sc_f4*>(L + r * 68 + m);         // zero from the diagonal on
                a0 = fmaf(l[0], x[m], a0);
                if (m + 1 < r) a1 = fmaf(l[1], x[m + 1], a1);
                if (m + 2 < r) a0 = fmaf(l[2], x[m + 2], a0);
                if (m + 3 < r) a1 = fmaf(l[3], x[m + 3], a1);
            }
            x[r] -= a0 + a1;
            if (r % 4 == 3) __builtin_amdgcn_sched_barrier(0);           // else every row of L is fetched at once
        }
#pragma unroll
        for (int r = 0; r < 64; ++r) out[(size_t)r * out_ld] = x[r];
    }
}

// A barrier of the block's waves that leaves loads from memory in flight.
__device__ __forceinline__ void scan_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// ---- chunked form: the chunks in order -------------------------------------------------------------------------
// Waves 0 .. 3 carry the state: wave w owns the state tiles w TW .. of sixteen rows, and the chunk's rows 16 w .. + 15 of U.
// Waves 4 .. 7 make the outputs of the rows 16 (w - 4) .. + 15.  Per chunk two phases, a barrier behind each:
//   first:  U = U0 - Kt S (SSD: dt V) into LDS;      o = G S^T q
//   second: S = G_63 S + k^T c U, S into LDS;        o += W U, stored
// Each wave requests its operands of a phase one phase ahead.  KT: state tiles (16 KT >= dk, KT a multiple of 4).
template <bool DELTA, int KT>
__global__ __launch_bounds__(512) void scan_chain_kernel(ScanParams p, uint32_t chunks) {
    constexpr int TW = KT / 4;
    __shared__ __attribute__((aligned(16))) sc_f4 ss[KT][64], us[4][64], cu[4][64];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i = lane & 15u, g = lane >> 4;
    const uint32_t head = blockIdx.x, col = blockIdx.y * 16u + i, dk = p.dk, dv = p.dv, kt = dk / 16u, w = wave & 3u;
    const uint32_t key_head = head / (p.heads / p.key_heads), v_at = 2u * p.key_heads * dk + head * dv + col;
    const sc_f4 zero = sc_f4{0.0f, 0.0f, 0.0f, 0.0f};
    float* state = p.state + (((size_t)p.rows.slot * p.heads + head) * dk) * dv + col;
    auto cell_of = [&](uint32_t n) { return (size_t)n * p.heads + head; };
    if (wave < 4u) {
        sc_f4 S[TW], kA[DELTA ? KT : 1], u0, c4;
        float kcol[TW][4][4], g63;
        auto first_operands = [&](uint32_t n) {      // of phase one of chunk n
            const size_t cell = cell_of(n);
            const uint32_t t0 = n * SCAN_CHUNK + 16u * w;
            if (DELTA) {
#pragma unroll
                for (int t = 0; t < KT; ++t) kA[t] = *reinterpret_cast<const sc_f4*>(p.kt + (cell * 64u + 16u * w + i) * dk + min(16u * t, dk - 16u) + 4u * g);
#pragma unroll
                for (int r = 0; r < 4; ++r) u0[r] = p.u0[(cell * 64u + 16u * w + 4u * g + r) * dv + col];
            } else {
                const sc_f4 b = *reinterpret_cast<const sc_f4*>(p.gates + cell * 192u + 128u + 16u * w + 4u * g);
#pragma unroll
                for (int r = 0; r < 4; ++r) u0[r] = b[r] * p.mixed[(size_t)min(t0 + 4u * g + r, p.n_rows - 1u) * p.channels + v_at];
            }
            c4 = *reinterpret_cast<const sc_f4*>(p.gates + cell * 192u + 64u + 16u * w + 4u * g);
        };
        auto second_operands = [&](uint32_t n) {
            g63 = p.gates[cell_of(n) * 192u + 63u];
#pragma unroll
            for (int s = 0; s < 4; ++s)
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float* k = p.mixed + (size_t)min(n * SCAN_CHUNK + 16u * s + 4u * g + r, p.n_rows - 1u) * p.channels + (p.key_heads + key_head) * dk + i;
#pragma unroll
                    for (int t = 0; t < TW; ++t) kcol[t][s][r] = k[min(16u * (w * TW + t), dk - 16u)];
                }
        };
        first_operands(0);
        second_operands(0);
#pragma unroll
        for (int t = 0; t < TW; ++t) {
            const uint32_t tile = w * TW + t;
#pragma unroll
            for (int r = 0; r < 4; ++r) S[t][r] = tile < kt ? state[(size_t)(16u * tile + 4u * g + r) * dv] : 0.0f;
            ss[tile][lane] = S[t];
        }
        scan_barrier();
        for (uint32_t n = 0; n < chunks; ++n) {
            const uint32_t next = min(n + 1u, chunks - 1u);
            sc_f4 u = u0;
            if (DELTA) {
                sc_f4 a0 = zero, a1 = zero;
#pragma unroll
                for (int t = 0; t < KT; ++t) {
                    if ((uint32_t)t < kt) {          // uniform
                        const sc_f4 b = ss[t][lane];
                        a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(kA[t][0], b[0], a0, 0, 0, 0);
                        a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(kA[t][1], b[1], a1, 0, 0, 0);
                        a0 = __builtin_amdgcn_mfma_f32_16x16x4f32(kA[t][2], b[2], a0, 0, 0, 0);
                        a1 = __builtin_amdgcn_mfma_f32_16x16x4f32(kA[t][3], b[3], a1, 0, 0, 0);
                    }
                }
                u -= a0 + a1;
            }
            us[w][lane] = u;
            cu[w][lane] = u * c4;
            first_operands(next);
            scan_barrier();
#pragma unroll
            for (int t = 0; t < TW; ++t) S[t] *= g63;
#pragma unroll
            for (int s = 0; s < 4; ++s) {
                const sc_f4 b = cu[s][lane];
#pragma unroll
                for (int r = 0; r < 4; ++r)
#pragma unroll
                    for (int t = 0; t < TW; ++t) S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(kcol[t][s][r], b[r], S[t], 0, 0, 0);
            }
#pragma unroll
            for (int t = 0; t < TW; ++t) ss[w * TW + t][lane] = S[t];
            second_operands(next);
            scan_barrier();
        }
#pragma unroll
        for (int t = 0; t < TW; ++t) {
            const uint32_t tile = w * TW + t;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (tile < kt) state[(size_t)(16u * tile + 4u * g + r) * dv] = S[t][r];
        }
        return;
    }
    sc_f4 qA[KT], wA[4], G4;
    float v[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    const float skip = DELTA ? 0.0f : bf16_to_f32(p.skip[head]);
    auto first_operands = [&](uint32_t n) {
        const float* q = p.mixed + (size_t)min(n * SCAN_CHUNK + 16u * w + i, p.n_rows - 1u) * p.channels + key_head * dk + 4u * g;
#pragma unroll
        for (int t = 0; t < KT; ++t) qA[t] = *reinterpret_cast<const sc_f4*>(q + min(16u * t, dk - 16u));
        G4 = *reinterpret_cast<const sc_f4*>(p.gates + cell_of(n) * 192u + 16u * w + 4u * g);
    };
    auto second_operands = [&](uint32_t n) {
#pragma unroll
        for (int t = 0; t < 4; ++t) wA[t] = *reinterpret_cast<const sc_f4*>(p.w + cell_of(n) * 4096u + (16u * w + i) * 64u + 16u * t + 4u * g);
        if (!DELTA) {
#pragma unroll
            for (int r = 0; r < 4; ++r) v[r] = p.mixed[(size_t)min(n * SCAN_CHUNK + 16u * w + 4u * g + r, p.n_rows - 1u) * p.channels + v_at];
        }
    };
    first_operands(0);
    second_operands(0);
    scan_barrier();
    for (uint32_t n = 0; n < chunks; ++n) {
        const uint32_t next = min(n + 1u, chunks - 1u);
        sc_f4 o = zero, o1 = zero;
#pragma unroll
        for (int t = 0; t < KT; ++t) {
            if ((uint32_t)t < kt) {                  // uniform
                const sc_f4 b = ss[t][lane];
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(qA[t][0], b[0], o, 0, 0, 0);
                o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qA[t][1], b[1], o1, 0, 0, 0);
                o = __builtin_amdgcn_mfma_f32_16x16x4f32(qA[t][2], b[2], o, 0, 0, 0);
                o1 = __builtin_amdgcn_mfma_f32_16x16x4f32(qA[t][3], b[3], o1, 0, 0, 0);
            }
        }
        o = (o + o1) * G4;
        first_operands(next);
        scan_barrier();
#pragma unroll
        for (int t = 0; t < 4; ++t) {
            if ((uint32_t)t <= w) {                  // uniform
                const sc_f4 b = us[t][lane];
#pragma unroll
                for (int r = 0; r < 4; ++r) o = __builtin_amdgcn_mfma_f32_16x16x4f32(wA[t][r], b[r], o, 0, 0, 0);
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const uint32_t t = n * SCAN_CHUNK + 16u * w + 4u * g + r;
            if (t < p.n_rows) p.out[(size_t)t * p.out_stride + head * dv + col] = o[r] + skip * v[r];
        }
        second_operands(next);
        scan_barrier();
    }
}

// ---- the gated norm behind a recurrence -------------------------------------------------------------------------
struct GatedNormParams {
    const float *x, *gate;
    const uint16_t* weight;
    void* out;
    uint32_t x_stride, gate_stride, out_stride, rows, heads, dv, dv_count, parts;
    float out_scale, eps;
};

// THREADS per (part, row): a wave (four of them in a block) or a block.  Elements of a part are read twice, the second
// time from the caches, unless they fit into KEEP registers per thread.
template <int ACT, bool FIRST, int THREADS>
__global__ __launch_bounds__(256) void gated_norm_kernel(GatedNormParams p) {
    constexpr int KEEP = 8;
    __shared__ float red[4];
    const uint32_t tid = threadIdx.x % THREADS, part = THREADS == 64 ? blockIdx.y * 4u + threadIdx.x / 64u : blockIdx.y, row = blockIdx.x;
    if (THREADS == 64 && part >= p.parts) return;
    const uint32_t n = p.heads * p.dv_count / p.parts, e0 = part * n;
    const float *x = p.x + (size_t)row * p.x_stride, *gate = p.gate + (size_t)row * p.gate_stride;
    auto place = [&](uint32_t e) { return p.dv == p.dv_count ? e : e / p.dv_count * p.dv + e % p.dv_count; };
    float xs[KEEP], zs[KEEP], ss = 0.0f;
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const uint32_t at = place(e0 + min(tid + THREADS * u, n - 1u));
        xs[u] = x[at];
        zs[u] = gate[at];
    }
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        if (FIRST) xs[u] *= silu(zs[u]);
        if (tid + THREADS * u < n) ss = fmaf(xs[u], xs[u], ss);
    }
    for (uint32_t e = tid + THREADS * KEEP; e < n; e += THREADS) {
        const uint32_t at = place(e0 + e);
        const float v = FIRST ? x[at] * silu(gate[at]) : x[at];
        ss = fmaf(v, v, ss);
    }
    ss = wave_sum_bcast(ss);
    if (THREADS == 256) {
        if ((tid & 63u) == 0) red[tid >> 6] = ss;
        __syncthreads();
        ss = (red[0] + red[1]) + (red[2] + red[3]);
    }
    const float inv = p.out_scale / sqrtf(ss / (float)n + p.eps);
    act_t<ACT>* out = static_cast<act_t<ACT>*>(p.out) + (size_t)row * p.out_stride;
    auto put = [&](uint32_t at, float v, float z) {
        out[at] = f32_to_act<ACT>(FIRST ? v * inv * bf16_to_f32(p.weight[at]) : v * inv * bf16_to_f32(p.weight[at % p.dv]) * silu(z));
    };
#pragma unroll
    for (int u = 0; u < KEEP; ++u)
        if (tid + THREADS * u < n) put(place(e0 + tid + THREADS * u), xs[u], zs[u]);
    for (uint32_t e = tid + THREADS * KEEP; e < n; e += THREADS) {
        const uint32_t at = place(e0 + e);
        const float z = gate[at];
        put(at, FIRST ? x[at] * silu(z) : x[at], z);
    }
}

}  // namespace nvmai
