// Kernels of the dense models (BF16 weights; 16-bit BF16 or 32-bit activations; a 32-bit residual stream):
// the matrix products.  gfx950, wave64.
#pragma once

#include "dense_internal.hpp"
#include "common.hpp"

namespace nvmai {

typedef __bf16 dn_b8 __attribute__((ext_vector_type(8)));
typedef float dn_f4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ dn_f4 dn_mfma(const uint4& a, const uint4& b, dn_f4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(dn_b8, a), __builtin_bit_cast(dn_b8, b), c, 0, 0, 0);
}

// z/2 (1 + erf(z / sqrt 2))
__device__ __forceinline__ float gelu_erf(float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f)); }

// z/2 (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3)))
__device__ __forceinline__ float gelu_tanh(float z) { return 0.5f * z * (1.0f + tanhf(0.79788456080286536f * fmaf(0.044715f * z * z, z, z))); }

// What stands between a sum and its store, fixed when a kernel is built: a tile's store is unrolled many times, and code
// that a call does not need costs instruction fetches in all of them.  PLAIN: the activation NONE; ERF: GELU_ERF; BIAS: a
// bias; PAIRS: SILU_PAIRS; FULL: bias, any activation, the token's own multiplier.
enum DenseEpilogue : int { DE_PLAIN, DE_ERF, DE_BIAS, DE_PAIRS, DE_FULL };

template <int EPI>
__device__ __forceinline__ float dense_finish(const DenseLinearParams& p, uint32_t t, uint32_t r, float v) {
    if (EPI == DE_ERF) return gelu_erf(v);
    if (EPI == DE_BIAS) return v + bf16_to_f32(p.bias[r]);
    if (EPI != DE_FULL) return v;
    if (p.bias) v += bf16_to_f32(p.bias[r]);
    v = p.activation == NVMAI_LINEAR_GELU_ERF ? gelu_erf(v) : p.activation == NVMAI_LINEAR_GELU_TANH ? gelu_tanh(v) : v;
    if (p.mul) {                                     // an id past the table: zero
        const uint32_t id = p.mul_ids[t];
        v *= id < p.mul_rows ? bf16_to_f32(p.mul[(size_t)id * p.mul_stride + r]) : 0.0f;
    }
    return v;
}

template <int ACT>
__device__ __forceinline__ void dense_put(const DenseLinearParams& p, uint32_t t, uint32_t r, float v) {
    if (p.y) static_cast<act_t<ACT>*>(p.y)[(size_t)t * p.y_stride + r] = f32_to_act<ACT>(v);
    if (p.y_f32) p.y_f32[(size_t)t * p.y_stride + r] = v;
}

template <int EPI, int ACT>
__device__ __forceinline__ void dense_store(const DenseLinearParams& p, uint32_t t, uint32_t r, float v) {
    dense_put<ACT>(p, t, r, dense_finish<EPI>(p, t, r, v));
}

// Rows 2 j and 2 j + 1 of the matrix make output j: silu(gate) * up.
template <int ACT>
__device__ __forceinline__ float dense_pair(float gate, float up) { return (ACT == ACT_FP32 ? silu(gate) : silu_fast(gate)) * up; }

// Four neighbouring outputs of one token (r0 a multiple of 4).
template <int EPI>
__device__ __forceinline__ void dense_store4_bf16(const DenseLinearParams& p, uint32_t t, uint32_t r0, dn_f4 v) {
    if (EPI == DE_PAIRS) {                           // n and the row stride are even
        const float a = dense_pair<ACT_BF16>(v[0], v[1]), b = dense_pair<ACT_BF16>(v[2], v[3]);
        if (r0 + 4u <= p.n) {
            if (p.y) *reinterpret_cast<uint32_t*>(static_cast<uint16_t*>(p.y) + (size_t)t * p.y_stride + r0 / 2u) = f32_to_bf16(a) | ((uint32_t)f32_to_bf16(b) << 16);
            if (p.y_f32) *reinterpret_cast<float2*>(p.y_f32 + (size_t)t * p.y_stride + r0 / 2u) = float2{a, b};
        } else if (r0 < p.n) {
            dense_put<ACT_BF16>(p, t, r0 / 2u, a);
        }
    } else if (r0 + 4u <= p.n && (p.y_stride & 3u) == 0) {
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = dense_finish<EPI>(p, t, r0 + j, v[j]);
        if (p.y) {
            uint2 q;
            q.x = f32_to_bf16(v[0]) | ((uint32_t)f32_to_bf16(v[1]) << 16);
            q.y = f32_to_bf16(v[2]) | ((uint32_t)f32_to_bf16(v[3]) << 16);
            *reinterpret_cast<uint2*>(static_cast<uint16_t*>(p.y) + (size_t)t * p.y_stride + r0) = q;
        }
        if (p.y_f32) *reinterpret_cast<dn_f4*>(p.y_f32 + (size_t)t * p.y_stride + r0) = v;
    } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (r0 + j < p.n) dense_store<EPI, ACT_BF16>(p, t, r0 + j, v[j]);
    }
}

// ---- 1 .. 4 input rows: a wave owns RW weight rows, its lanes split k in 16-byte pieces -------------
// Bound by the matrix's bytes.  The inputs are read from L1 / L2 beside the weights (no LDS, no barrier): every
// load of a k step is independent of the others, so a wave has RW + NT (32-bit inputs: RW + 2 NT) 16-byte loads per lane
// in flight.
template <int EPI, int ACT, int NT, int RW>
__global__ __launch_bounds__(256) void dense_gemv_kernel(DenseLinearParams p) {
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6;
    const uint32_t r0 = (blockIdx.x * 4u + wave) * RW;
    if (r0 >= p.n) return;
    const uint16_t* wp[RW];
#pragma unroll
    for (int r = 0; r < RW; ++r) wp[r] = p.w + (size_t)min(r0 + r, p.n - 1u) * p.w_stride;
    const act_t<ACT>* x = static_cast<const act_t<ACT>*>(p.x);
    float acc[NT][RW];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < RW; ++r) acc[t][r] = 0.0f;
    constexpr int XP = ACT == ACT_FP32 ? 2 : 1;
    constexpr int U = NT * XP + RW <= 3 ? 4 : 2;             // steps of 512 k whose loads are all issued before the first product
    for (uint32_t k0 = 0; k0 < p.k; k0 += 512u * U) {
        uint4 wv[U][RW], xv[U][NT][XP];
#pragma unroll
        for (int s = 0; s < U; ++s) {
            const uint32_t at = min(k0 + 512u * s + lane * 8u, p.k - 8u);        // past the end: the last piece, multiplied by zero
#pragma unroll
            for (int r = 0; r < RW; ++r) wv[s][r] = *reinterpret_cast<const uint4*>(wp[r] + at);
#pragma unroll
            for (int t = 0; t < NT; ++t)
#pragma unroll
                for (int u = 0; u < XP; ++u) xv[s][t][u] = reinterpret_cast<const uint4*>(x + (size_t)t * p.x_stride + at)[u];
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int s = 0; s < U; ++s) {
            const bool live = k0 + 512u * s + lane * 8u < p.k;
            float wf[RW][8];
#pragma unroll
            for (int r = 0; r < RW; ++r) {
                const uint4 q = live ? wv[s][r] : make_uint4(0u, 0u, 0u, 0u);
                act2_to_f32<ACT_BF16>(q.x, wf[r][0], wf[r][1]);
                act2_to_f32<ACT_BF16>(q.y, wf[r][2], wf[r][3]);
                act2_to_f32<ACT_BF16>(q.z, wf[r][4], wf[r][5]);
                act2_to_f32<ACT_BF16>(q.w, wf[r][6], wf[r][7]);
            }
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                float xf[8];
                if constexpr (ACT == ACT_FP32) {
#pragma unroll
                    for (int u = 0; u < 2; ++u) {
                        xf[4 * u] = __uint_as_float(xv[s][t][u].x); xf[4 * u + 1] = __uint_as_float(xv[s][t][u].y);
                        xf[4 * u + 2] = __uint_as_float(xv[s][t][u].z); xf[4 * u + 3] = __uint_as_float(xv[s][t][u].w);
                    }
                } else {
                    act2_to_f32<ACT_BF16>(xv[s][t][0].x, xf[0], xf[1]);
                    act2_to_f32<ACT_BF16>(xv[s][t][0].y, xf[2], xf[3]);
                    act2_to_f32<ACT_BF16>(xv[s][t][0].z, xf[4], xf[5]);
                    act2_to_f32<ACT_BF16>(xv[s][t][0].w, xf[6], xf[7]);
                }
#pragma unroll
                for (int r = 0; r < RW; ++r)
#pragma unroll
                    for (int j = 0; j < 8; ++j) acc[t][r] = fmaf(wf[r][j], xf[j], acc[t][r]);
            }
        }
    }
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        float v[RW];
#pragma unroll
        for (int r = 0; r < RW; ++r) v[r] = wave_sum_bcast(acc[t][r]);
#pragma unroll
        for (int r = 0; r < RW; r += EPI == DE_PAIRS ? 2 : 1) {
            if (lane != (uint32_t)(t * RW + r) || r0 + r >= p.n || (uint32_t)t >= p.rows) continue;
            if constexpr (EPI == DE_PAIRS) dense_put<ACT>(p, t, (r0 + r) / 2u, dense_pair<ACT>(v[r], v[r + 1]));
            else dense_store<EPI, ACT>(p, t, r0 + r, v[r]);
        }
    }
}

// ---- 5 .. 64 input rows: 16 NR weight rows per block, the waves split k, MFMA, sums through LDS ---------
// Weight rows are the A operand as they lie in memory: lane (i = lane % 16, g = lane / 16) loads the 32 bytes
// W[r0 + i, k + 16 g .. + 16), four lanes cover 128 contiguous bytes of a row; the inputs are the B operand in
// the same order of k, read from L2 once per NR row tiles.
template <int EPI, int TT, int NR, int NW>
__global__ __launch_bounds__(64 * NW) void dense_skinny_kernel(DenseLinearParams p) {
    __shared__ __attribute__((aligned(16))) float part[NW - 1][64][TT * NR * 4];
    const uint32_t lane = threadIdx.x & 63u, wave = threadIdx.x >> 6, i = lane & 15u, g = lane >> 4;
    const uint32_t r0 = blockIdx.x * (16u * NR);
    const uint16_t* wp[NR];
#pragma unroll
    for (int r = 0; r < NR; ++r) wp[r] = p.w + (size_t)min(r0 + 16u * r + i, p.n - 1u) * p.w_stride + g * 16u;
    const uint16_t* x = static_cast<const uint16_t*>(p.x);
    const uint16_t* xp[TT];
#pragma unroll
    for (int t = 0; t < TT; ++t) xp[t] = x + (size_t)min(16u * t + i, p.rows - 1u) * p.x_stride + g * 16u;
    dn_f4 acc[NR][TT];
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
        for (int t = 0; t < TT; ++t) acc[r][t] = dn_f4{0.0f, 0.0f, 0.0f, 0.0f};
    const uint32_t steps = p.k / 64u;
#pragma unroll 4
    for (uint32_t st = wave; st < steps; st += NW) {
        uint4 a0[NR], a1[NR], b0[TT], b1[TT];
#pragma unroll
        for (int r = 0; r < NR; ++r) {
            a0[r] = *reinterpret_cast<const uint4*>(wp[r] + st * 64u);
            a1[r] = *reinterpret_cast<const uint4*>(wp[r] + st * 64u + 8u);
        }
#pragma unroll
        for (int t = 0; t < TT; ++t) {
            b0[t] = *reinterpret_cast<const uint4*>(xp[t] + st * 64u);
            b1[t] = *reinterpret_cast<const uint4*>(xp[t] + st * 64u + 8u);
        }
#pragma unroll
        for (int r = 0; r < NR; ++r)
#pragma unroll
            for (int t = 0; t < TT; ++t) {
                acc[r][t] = dn_mfma(a0[r], b0[t], acc[r][t]);
                acc[r][t] = dn_mfma(a1[r], b1[t], acc[r][t]);
            }
    }
    if (wave != 0) {
#pragma unroll
        for (int r = 0; r < NR; ++r)
#pragma unroll
            for (int t = 0; t < TT; ++t) *reinterpret_cast<dn_f4*>(&part[wave - 1][lane][4 * (r * TT + t)]) = acc[r][t];
    }
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
        for (int t = 0; t < TT; ++t) {
#pragma unroll
            for (int w = 0; w < NW - 1; ++w) acc[r][t] += *reinterpret_cast<const dn_f4*>(&part[w][lane][4 * (r * TT + t)]);
            // acc[r][t][j] = y[token 16 t + i, row r0 + 16 r + 4 g + j]
            if (16u * t + i < p.rows) dense_store4_bf16<EPI>(p, 16u * t + i, r0 + 16u * r + 4u * g, acc[r][t]);
        }
}

// ---- many input rows: tiles of BN weight rows x BM tokens, k in steps of 64 through double-buffered LDS --------
// Four waves, each a quarter of the tile (BN / 2 x BM / 2) in 16 x 16 x 32 products.  A tile's rows are 128 bytes
// of LDS; the eight 16-byte pieces of row r lie in the order piece ^ (r % 8), so that the sixteen rows of an
// operand read fall into different banks.  Loads go straight from memory into LDS.
template <int EPI, int BN, int BM>
__global__ __launch_bounds__(256) void dense_gemm_kernel(DenseLinearParams p, uint32_t tiles_n, uint32_t tiles_m) {
    constexpr int LA = BN / 32, LB = BM / 32;                // 1 KB pieces per wave
    constexpr int TN = BN / 32, TM = BM / 32;                // 16 x 16 tiles per wave
    constexpr uint32_t STAGE = (BN + BM) * 128u;
    __shared__ __attribute__((aligned(16))) uint8_t lds[2 * STAGE];
    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // blocks are dealt to the eight XCDs in turn: give each XCD a run of neighbouring tiles (shared L2 lines)
    const uint32_t total = tiles_n * tiles_m, xcd = blockIdx.x & 7u, nth = blockIdx.x >> 3;
    const uint32_t base = total / 8u, extra = total % 8u;
    const uint32_t tile = xcd * base + min(xcd, extra) + nth;
    // in bands of eight token tiles, weight tiles outermost within the band
    const uint32_t band = tile / (8u * tiles_n), in_band = tile % (8u * tiles_n);
    const uint32_t band_m = min(8u, tiles_m - band * 8u);
    const uint32_t m0 = (band * 8u + in_band % band_m) * BM, n0 = (in_band / band_m) * BN;

    [[maybe_unused]] const __amdgpu_buffer_rsrc_t wrs = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<uint16_t*>(p.w), 0, (int)(uint32_t)((size_t)(p.n - 1u) * p.w_stride * 2u + p.k * 2u), 0x00020000);
    [[maybe_unused]] const __amdgpu_buffer_rsrc_t xrs = __builtin_amdgcn_make_buffer_rsrc(
        const_cast<void*>(p.x), 0, (int)(uint32_t)((size_t)(p.rows - 1u) * p.x_stride * 2u + p.k * 2u), 0x00020000);
    uint32_t aoff[LA], boff[LB];
    const uint32_t lr = lane >> 3, piece = (lane & 7u) ^ (lr & 7u);
#pragma unroll
    for (int j = 0; j < LA; ++j) aoff[j] = min(n0 + (wave * LA + j) * 8u + lr, p.n - 1u) * p.w_stride * 2u + piece * 16u;
#pragma unroll
    for (int j = 0; j < LB; ++j) boff[j] = min(m0 + (wave * LB + j) * 8u + lr, p.rows - 1u) * p.x_stride * 2u + piece * 16u;
    auto issue = [&](uint32_t st, uint8_t* dst) {
#if defined(__HIP_DEVICE_COMPILE__)     // the host pass rejects the 16-byte form of the load
#pragma unroll
        for (int j = 0; j < LA; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(wrs, (__attribute__((address_space(3))) void*)(dst + (wave * LA + j) * 1024u), 16, aoff[j], st * 128u, 0, 0);
#pragma unroll
        for (int j = 0; j < LB; ++j)
            __builtin_amdgcn_raw_ptr_buffer_load_lds(xrs, (__attribute__((address_space(3))) void*)(dst + BN * 128u + (wave * LB + j) * 1024u), 16, boff[j], st * 128u, 0, 0);
#endif
    };
    dn_f4 acc[TN][TM];
#pragma unroll
    for (int a = 0; a < TN; ++a)
#pragma unroll
        for (int b = 0; b < TM; ++b) acc[a][b] = dn_f4{0.0f, 0.0f, 0.0f, 0.0f};
    const uint32_t i = lane & 15u, g = lane >> 4;
    const uint32_t wn = (wave >> 1) * (BN / 2), wm = (wave & 1u) * (BM / 2);
    const uint32_t steps = p.k / 64u;
    issue(0, lds);
    __syncthreads();
    for (uint32_t st = 0; st < steps; ++st) {
        uint8_t* cur = lds + (st & 1u) * STAGE;
        if (st + 1u < steps) issue(st + 1u, lds + ((st + 1u) & 1u) * STAGE);
#pragma unroll
        for (uint32_t ks = 0; ks < 2; ++ks) {
            const uint32_t sw = ((ks * 4u + g) ^ (i & 7u)) * 16u;
            uint4 af[TN], bf[TM];
#pragma unroll
            for (int a = 0; a < TN; ++a) af[a] = *reinterpret_cast<const uint4*>(cur + (wn + 16 * a + i) * 128u + sw);
#pragma unroll
            for (int b = 0; b < TM; ++b) bf[b] = *reinterpret_cast<const uint4*>(cur + BN * 128u + (wm + 16 * b + i) * 128u + sw);
#pragma unroll
            for (int a = 0; a < TN; ++a)
#pragma unroll
                for (int b = 0; b < TM; ++b) acc[a][b] = dn_mfma(af[a], bf[b], acc[a][b]);
        }
        __syncthreads();                 // the next stage has landed, this one may be overwritten
    }
#pragma unroll
    for (int b = 0; b < TM; ++b) {
        const uint32_t t = m0 + wm + 16 * b + i;
        if (t >= p.rows) continue;
#pragma unroll
        for (int a = 0; a < TN; ++a) {
            const uint32_t r = n0 + wn + 16 * a + 4u * g;
            if (r < p.n) dense_store4_bf16<EPI>(p, t, r, acc[a][b]);
        }
    }
}

// ---- 32-bit activations, more than four rows: 64 x 64 tiles on the vector pipe, BF16 weights widened, fp32 FMA ------------
// Sums are two-level (a step of 16 k, then the running total), which keeps the rounding error of a long k small.
template <int EPI>
__global__ __launch_bounds__(256) void dense_f32_kernel(DenseLinearParams p) {
    __shared__ float ws[16][65], xs[16][65];
    const uint32_t tid = threadIdx.x, tx = tid & 15u, ty = tid >> 4;
    const uint32_t n0 = blockIdx.x * 64u, m0 = blockIdx.y * 64u;
    const float* x = static_cast<const float*>(p.x);
    float acc[4][4] = {};
    for (uint32_t k0 = 0; k0 < p.k; k0 += 16u) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const uint32_t r = (tid >> 4) + 16u * j, k = tid & 15u;
            ws[k][r] = bf16_to_f32(p.w[(size_t)min(n0 + r, p.n - 1u) * p.w_stride + k0 + k]);
            xs[k][r] = x[(size_t)min(m0 + r, p.rows - 1u) * p.x_stride + k0 + k];
        }
        __syncthreads();
        float part[4][4] = {};
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            float a[4], b[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) { a[j] = xs[k][ty + 16 * j]; b[j] = ws[k][tx + 16 * j]; }
#pragma unroll
            for (int m = 0; m < 4; ++m)
#pragma unroll
                for (int n = 0; n < 4; ++n) part[m][n] = fmaf(a[m], b[n], part[m][n]);
        }
#pragma unroll
        for (int m = 0; m < 4; ++m)
#pragma unroll
            for (int n = 0; n < 4; ++n) acc[m][n] += part[m][n];
        __syncthreads();
    }
#pragma unroll
    for (int m = 0; m < 4; ++m)
#pragma unroll
        for (int n = 0; n < 4; ++n) {
            const uint32_t t = m0 + ty + 16u * m, r = n0 + tx + 16u * n;
            const float next = EPI == DE_PAIRS ? shfl_xor_f(acc[m][n], 1) : 0.0f;        // the neighbouring weight row's sum
            if (t >= p.rows || r >= p.n) continue;
            if (EPI != DE_PAIRS) dense_store<EPI, ACT_FP32>(p, t, r, acc[m][n]);
            else if ((r & 1u) == 0) dense_put<ACT_FP32>(p, t, r / 2u, dense_pair<ACT_FP32>(acc[m][n], next));
        }
}

// ---- launches ---------------------------------------------------------------------------------------------
template <int EPI, int ACT, int NT>
void launch_gemv(const DenseLinearParams& p, hipStream_t s) {
    // rows per wave: one (short blocks, many of them) until the inputs' own loads weigh more than that
    if (p.n >= 65536) dense_gemv_kernel<EPI, ACT, NT, 4><<<(p.n + 15) / 16, 256, 0, s>>>(p);
    else if (EPI == DE_PAIRS || (NT * (ACT == ACT_FP32 ? 2 : 1) > 2 && p.n >= 8192)) dense_gemv_kernel<EPI, ACT, NT, 2><<<(p.n + 7) / 8, 256, 0, s>>>(p);
    else if constexpr (EPI != DE_PAIRS) dense_gemv_kernel<EPI, ACT, NT, 1><<<(p.n + 3) / 4, 256, 0, s>>>(p);
}

template <int EPI, int ACT>
int gemv(const DenseLinearParams& p, hipStream_t s) {
    if (p.rows == 1) launch_gemv<EPI, ACT, 1>(p, s);
    else if (p.rows == 2) launch_gemv<EPI, ACT, 2>(p, s);
    else if (p.rows == 3) launch_gemv<EPI, ACT, 3>(p, s);
    else launch_gemv<EPI, ACT, 4>(p, s);
    return launch_status();
}

template <int EPI>
int dense_launch(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) {
    if (p.rows <= 4) return ctx->act == NVMAI_ACT_FP32 ? gemv<EPI, ACT_FP32>(p, s) : gemv<EPI, ACT_BF16>(p, s);
    if (ctx->act == NVMAI_ACT_FP32) {
        const dim3 grid((p.n + 63) / 64, (p.rows + 63) / 64);
        if (grid.y > 65535) return NVMAI_ERR_UNSUPPORTED;
        dense_f32_kernel<EPI><<<grid, 256, 0, s>>>(p);
        return launch_status();
    }
    if (p.rows <= 64) {
        // row tiles per block: as many as leave every compute unit several blocks; waves: about four steps of k each
        const int nr = p.n >= 32768 ? 4 : p.n >= 8192 ? 2 : 1;
        const uint32_t blocks = (p.n + 16 * nr - 1) / (16 * nr);
#define NVMAI_SKINNY(TT)                                                              \
    do {                                                                              \
        if (nr == 4) dense_skinny_kernel<EPI, TT, 4, 4><<<blocks, 256, 0, s>>>(p);         \
        else if (nr == 2) dense_skinny_kernel<EPI, TT, 2, 4><<<blocks, 256, 0, s>>>(p);    \
        else if (p.k <= 1024) dense_skinny_kernel<EPI, TT, 1, 4><<<blocks, 256, 0, s>>>(p); \
        else if (p.k <= 2048) dense_skinny_kernel<EPI, TT, 1, 8><<<blocks, 512, 0, s>>>(p); \
        else dense_skinny_kernel<EPI, TT, 1, 16><<<blocks, 1024, 0, s>>>(p);               \
    } while (0)
        if (p.rows <= 16) NVMAI_SKINNY(1);
        else if (p.rows <= 32) NVMAI_SKINNY(2);
        else NVMAI_SKINNY(4);
#undef NVMAI_SKINNY
        return launch_status();
    }
    // the largest tile that still gives every compute unit one
    const uint32_t cus = (uint32_t)ctx->compute_units;
    auto tiles = [](uint32_t v, uint32_t b) { return (v + b - 1) / b; };
    if (tiles(p.n, 128) * tiles(p.rows, 128) >= cus)
        dense_gemm_kernel<EPI, 128, 128><<<tiles(p.n, 128) * tiles(p.rows, 128), 256, 0, s>>>(p, tiles(p.n, 128), tiles(p.rows, 128));
    else if (tiles(p.n, 64) * tiles(p.rows, 128) >= cus)
        dense_gemm_kernel<EPI, 64, 128><<<tiles(p.n, 64) * tiles(p.rows, 128), 256, 0, s>>>(p, tiles(p.n, 64), tiles(p.rows, 128));
    else if (tiles(p.n, 64) * tiles(p.rows, 64) <= cus)      // one tile per compute unit waits for each of its loads: halve them
        dense_gemm_kernel<EPI, 32, 64><<<tiles(p.n, 32) * tiles(p.rows, 64), 256, 0, s>>>(p, tiles(p.n, 32), tiles(p.rows, 64));
    else
        dense_gemm_kernel<EPI, 64, 64><<<tiles(p.n, 64) * tiles(p.rows, 64), 256, 0, s>>>(p, tiles(p.n, 64), tiles(p.rows, 64));
    return launch_status();
}

}  // namespace nvmai
