// The dense product, callable from other entry-point files.
#pragma once

#include "ctx.hpp"

namespace nvmai {

struct DenseLinearParams {
    const uint16_t* w;      // [n, w_stride] BF16
    const void* x;          // [rows, x_stride] activations
    void* y;                // activations, or nullptr
    float* y_f32;           // floats, or nullptr
    uint32_t w_stride, x_stride, y_stride, rows, n, k;
    int activation;         // NVMAI_LINEAR_*
    const uint16_t* bias;   // [n] BF16, or nullptr
    const uint16_t* mul;    // BF16 table [mul_rows, mul_stride]: y[t, r] *= mul[mul_ids[t], r]; or nullptr
    const uint32_t* mul_ids;
    uint32_t mul_stride, mul_rows;
};

int dense_linear_check(const nvmai_hip_ctx* ctx, const DenseLinearParams& p);
// The launches behind it by what stands between sum and store (dense_*_api.hip, built side by side).
int dense_launch_erf(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p);
int dense_launch_bias(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p);
int dense_launch_pairs(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p);
int dense_launch_full(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p);
int dense_linear(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p);

}  // namespace nvmai
