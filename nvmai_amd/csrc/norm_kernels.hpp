// Norms over the 32-bit residual stream of the dense models: the norm, scale and add that close a sublayer and the norm
// that opens the next one, in one launch.  gfx950, wave64.
#pragma once

#include "common.hpp"

namespace nvmai {

typedef float nr_f4 __attribute__((ext_vector_type(4)));

// Sum over the 256 threads of a block, every thread gets it.  `lds` holds four floats per call site.
__device__ __forceinline__ float block_sum256(float v, float* lds) {
    v = wave_sum_bcast(v);
    if ((threadIdx.x & 63u) == 0) lds[threadIdx.x >> 6] = v;
    __syncthreads();
    return (lds[0] + lds[1]) + (lds[2] + lds[3]);
}

// (v - mean) / sqrt(mean((v - mean)^2) + eps) over the row's d elements, dead slots zero before and after.
// Thread t holds the elements 4 (t + 256 j) .. + 3.
template <int VPT>
__device__ __forceinline__ void block_layernorm(float (&v)[VPT][4], uint32_t d, float eps, float* lds) {
    float s = 0.0f;
#pragma unroll
    for (int j = 0; j < VPT; ++j) s += (v[j][0] + v[j][1]) + (v[j][2] + v[j][3]);
    const float mean = block_sum256(s, lds) / (float)d;
    float q = 0.0f;
#pragma unroll
    for (int j = 0; j < VPT; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[j][e] = 4u * (threadIdx.x + 256u * j) + e < d ? v[j][e] - mean : 0.0f;
            q = fmaf(v[j][e], v[j][e], q);
        }
    const float inv = 1.0f / sqrtf(block_sum256(q, lds + 4) / (float)d + eps);
#pragma unroll
    for (int j = 0; j < VPT; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) v[j][e] *= inv;
}

// v / sqrt(mean(v^2) + eps), the same layout.
template <int VPT>
__device__ __forceinline__ void block_rmsnorm(float (&v)[VPT][4], uint32_t d, float eps, float* lds) {
    float q = 0.0f;
#pragma unroll
    for (int j = 0; j < VPT; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) q = fmaf(v[j][e], v[j][e], q);
    const float inv = 1.0f / sqrtf(block_sum256(q, lds) / (float)d + eps);
#pragma unroll
    for (int j = 0; j < VPT; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) v[j][e] *= inv;
}

// How a row is normed: not at all, as a layer norm (weight and bias), by its root mean square (plain weight, or a
// weight stored around zero: post_add, next_add = 1), or handed on as it is.
enum NormKind : int { NORM_NONE = 0, NORM_LAYER = 1, NORM_RMS = 2, NORM_COPY = 3 };

struct NormResidualParams {
    float* x;                        // [rows, x_stride] residual stream
    const float* delta;              // sublayer output
    const uint16_t *post_w, *post_b; // norm of delta
    const uint16_t *next_w, *next_b; // norm that opens the next sublayer
    void* out;
    uint32_t x_stride, delta_stride, out_stride, d;
    float mult, eps, post_add, next_add;
};

__device__ __forceinline__ void norm_bf4(const uint16_t* p, float* v) {
    const uint2 q = *reinterpret_cast<const uint2*>(p);
    act2_to_f32<ACT_BF16>(q.x, v[0], v[1]);
    act2_to_f32<ACT_BF16>(q.y, v[2], v[3]);
}

// x += mult * post(delta) (DELTA; POST NORM_NONE: x += mult * delta); out = next(x) (NEXT not NORM_NONE): one block per row,
// the row in registers.  Every operand is requested before the first sum.  VEC: four elements per load (d and the
// strides are multiples of 4); dead slots reread the row's last elements.
template <int ACT, int VPT, bool DELTA, int POST, int NEXT, bool VEC>
__global__ __launch_bounds__(256) void norm_residual_kernel(NormResidualParams p) {
    constexpr bool PW = POST != NORM_NONE, PB = POST == NORM_LAYER, NW = NEXT == NORM_LAYER || NEXT == NORM_RMS, NB = NEXT == NORM_LAYER;
    __shared__ float lds[16];
    const uint32_t row = blockIdx.x, tid = threadIdx.x;
    float* x = p.x + (size_t)row * p.x_stride;
    const float* delta = p.delta + (size_t)row * p.delta_stride;
    float xv[VPT][4], dv[VPT][4], pw[VPT][4], pb[VPT][4], nw[VPT][4], nb[VPT][4];
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const uint32_t at = 4u * (tid + 256u * j);
        if (VEC) {
            const uint32_t c = min(at, p.d - 4u);
            *reinterpret_cast<nr_f4*>(xv[j]) = *reinterpret_cast<const nr_f4*>(x + c);
            if (DELTA) *reinterpret_cast<nr_f4*>(dv[j]) = *reinterpret_cast<const nr_f4*>(delta + c);
            if (PW) norm_bf4(p.post_w + c, pw[j]);
            if (PB) norm_bf4(p.post_b + c, pb[j]);
            if (NW) norm_bf4(p.next_w + c, nw[j]);
            if (NB) norm_bf4(p.next_b + c, nb[j]);
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const uint32_t c = min(at + e, p.d - 1u);
                xv[j][e] = x[c];
                if (DELTA) dv[j][e] = delta[c];
                if (PW) pw[j][e] = bf16_to_f32(p.post_w[c]);
                if (PB) pb[j][e] = bf16_to_f32(p.post_b[c]);
                if (NW) nw[j][e] = bf16_to_f32(p.next_w[c]);
                if (NB) nb[j][e] = bf16_to_f32(p.next_b[c]);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            if (POST == NORM_RMS) pw[j][e] += p.post_add;
            if (NEXT == NORM_RMS) nw[j][e] += p.next_add;
            if (at + e >= p.d) { xv[j][e] = 0.0f; if (DELTA) dv[j][e] = 0.0f; }
        }
    }
    if (DELTA) {
        if (POST == NORM_LAYER) block_layernorm<VPT>(dv, p.d, p.eps, lds);
        if (POST == NORM_RMS) block_rmsnorm<VPT>(dv, p.d, p.eps, lds);
#pragma unroll
        for (int j = 0; j < VPT; ++j) {
            const uint32_t at = 4u * (tid + 256u * j);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float add = POST == NORM_LAYER ? fmaf(dv[j][e], pw[j][e], pb[j][e]) : POST == NORM_RMS ? dv[j][e] * pw[j][e] : dv[j][e];
                xv[j][e] = at + e < p.d ? fmaf(p.mult, add, xv[j][e]) : 0.0f;
            }
            if (VEC) {
                if (at < p.d) *reinterpret_cast<nr_f4*>(x + at) = *reinterpret_cast<nr_f4*>(xv[j]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (at + e < p.d) x[at + e] = xv[j][e];
            }
        }
    }
    if (NEXT == NORM_NONE) return;
    if (NEXT == NORM_LAYER) block_layernorm<VPT>(xv, p.d, p.eps, lds + 8);
    if (NEXT == NORM_RMS) block_rmsnorm<VPT>(xv, p.d, p.eps, lds + 8);
    act_t<ACT>* out = static_cast<act_t<ACT>*>(p.out) + (size_t)row * p.out_stride;
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const uint32_t at = 4u * (tid + 256u * j);
        act_t<ACT> o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e)
            o[e] = f32_to_act<ACT>(NEXT == NORM_LAYER ? fmaf(xv[j][e], nw[j][e], nb[j][e]) : NEXT == NORM_RMS ? xv[j][e] * nw[j][e] : xv[j][e]);
        if (VEC) {
            if (at < p.d) {
                if constexpr (ACT == ACT_FP32) *reinterpret_cast<nr_f4*>(out + at) = nr_f4{o[0], o[1], o[2], o[3]};
                else *reinterpret_cast<uint2*>(out + at) = make_uint2(o[0] | ((uint32_t)o[1] << 16), o[2] | ((uint32_t)o[3] << 16));
            }
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (at + e < p.d) out[at + e] = o[e];
        }
    }
}

}  // namespace nvmai
