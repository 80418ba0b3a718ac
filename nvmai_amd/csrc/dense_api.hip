// Entry points of the dense models: matrix products against BF16 weights, layer norms over the 32-bit residual,
// embedding rows, argmax.
#include "ctx.hpp"
#include "dense_kernels.hpp"
#include "dense_internal.hpp"

using namespace nvmai;

namespace nvmai {

int dense_linear_check(const nvmai_hip_ctx* ctx, const DenseLinearParams& p) {
    if (!ctx || !p.w || !p.x || (!p.y && !p.y_f32)) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (p.k == 0 || p.k % 64 || p.n == 0 || p.w_stride < p.k || p.x_stride < p.k || p.y_stride < p.n) return NVMAI_ERR_INVALID_ARG;
    if (p.activation != NVMAI_LINEAR_NONE && p.activation != NVMAI_LINEAR_GELU_ERF) return NVMAI_ERR_UNSUPPORTED;
    if (!aligned16(p.w) || !aligned16(p.x) || p.w_stride % 8 || p.x_stride % 8) return NVMAI_ERR_ALIGNMENT;
    if ((p.y && !aligned16(p.y)) || (p.y_f32 && !aligned16(p.y_f32))) return NVMAI_ERR_ALIGNMENT;
    // 32-bit byte offsets inside an operand
    if ((uint64_t)p.n * p.w_stride * 2 > 0xFFFFFFFFull || (uint64_t)p.rows * p.x_stride * 4 > 0xFFFFFFFFull) return NVMAI_ERR_UNSUPPORTED;
    return NVMAI_OK;
}

template <int NT>
static void launch_gemv(const DenseLinearParams& p, hipStream_t s) {
    // rows per wave: enough blocks for the device first, then more loads in flight per wave
    if (p.n >= 8192) dense_gemv_kernel<NT, 4><<<(p.n + 15) / 16, 256, 0, s>>>(p);
    else if (p.n >= 3072) dense_gemv_kernel<NT, 2><<<(p.n + 7) / 8, 256, 0, s>>>(p);
    else dense_gemv_kernel<NT, 1><<<(p.n + 3) / 4, 256, 0, s>>>(p);
}

int dense_linear(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) {
    const int rc = dense_linear_check(ctx, p);
    if (rc) return rc;
    if (p.rows == 0) return NVMAI_OK;
    if (ctx->act == NVMAI_ACT_FP32) {
        const dim3 grid((p.n + 63) / 64, (p.rows + 63) / 64);
        if (grid.y > 65535) return NVMAI_ERR_UNSUPPORTED;
        dense_f32_kernel<<<grid, 256, 0, s>>>(p);
        return launch_status();
    }
    if (p.rows <= 4) {
        if (p.rows == 1) launch_gemv<1>(p, s);
        else if (p.rows == 2) launch_gemv<2>(p, s);
        else if (p.rows == 3) launch_gemv<3>(p, s);
        else launch_gemv<4>(p, s);
        return launch_status();
    }
    if (p.rows <= 64) {
        const uint32_t blocks = (p.n + 15) / 16;
        if (p.rows <= 16) dense_skinny_kernel<1><<<blocks, 256, 0, s>>>(p);
        else if (p.rows <= 32) dense_skinny_kernel<2><<<blocks, 256, 0, s>>>(p);
        else dense_skinny_kernel<4><<<blocks, 256, 0, s>>>(p);
        return launch_status();
    }
    // the largest tile that still gives every compute unit one
    const uint32_t cus = (uint32_t)ctx->compute_units;
    auto tiles = [](uint32_t v, uint32_t b) { return (v + b - 1) / b; };
    if (tiles(p.n, 128) * tiles(p.rows, 128) >= cus)
        dense_gemm_kernel<128, 128><<<tiles(p.n, 128) * tiles(p.rows, 128), 256, 0, s>>>(p, tiles(p.n, 128), tiles(p.rows, 128));
    else if (tiles(p.n, 64) * tiles(p.rows, 128) >= cus)
        dense_gemm_kernel<64, 128><<<tiles(p.n, 64) * tiles(p.rows, 128), 256, 0, s>>>(p, tiles(p.n, 64), tiles(p.rows, 128));
    else
        dense_gemm_kernel<64, 64><<<tiles(p.n, 64) * tiles(p.rows, 64), 256, 0, s>>>(p, tiles(p.n, 64), tiles(p.rows, 64));
    return launch_status();
}

}  // namespace nvmai

extern "C" int nvmai_hip_dense_linear(nvmai_hip_ctx* ctx, nvmai_stream stream, const uint16_t* w, uint32_t w_stride,
                                      const void* x, uint32_t x_stride, uint32_t rows, uint32_t n, uint32_t k, void* y,
                                      float* y_f32, uint32_t y_stride, int activation) {
    const DenseLinearParams p{w, x, y, y_f32, w_stride, x_stride, y_stride, rows, n, k, activation};
    return dense_linear(ctx, (hipStream_t)stream, p);
}

extern "C" int nvmai_hip_norm_residual(nvmai_hip_ctx* ctx, nvmai_stream stream, float* x, uint32_t x_stride, const float* delta,
                                       uint32_t delta_stride, const uint16_t* post_weight, const uint16_t* post_bias, float mult,
                                       const uint16_t* next_weight, const uint16_t* next_bias, void* out, uint32_t out_stride,
                                       uint32_t rows, uint32_t d, float eps) {
    if (!ctx || !x || d == 0 || x_stride < d || (delta && delta_stride < d)) return NVMAI_ERR_INVALID_ARG;
    if ((next_weight == nullptr) != (out == nullptr) || (out && out_stride < d)) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (d > 16384) return NVMAI_ERR_UNSUPPORTED;
    if (rows == 0) return NVMAI_OK;
    const NormResidualParams p{x, delta, post_weight, post_bias, next_weight, next_bias, out, x_stride, delta_stride, out_stride, d, mult, eps};
    hipStream_t s = (hipStream_t)stream;
    const uint32_t vpt = (d + 255) / 256;
#define NVMAI_NR(ACT)                                                                            \
    do {                                                                                         \
        if (vpt <= 1) norm_residual_kernel<ACT, 1><<<rows, 256, 0, s>>>(p);                      \
        else if (vpt <= 2) norm_residual_kernel<ACT, 2><<<rows, 256, 0, s>>>(p);                 \
        else if (vpt <= 4) norm_residual_kernel<ACT, 4><<<rows, 256, 0, s>>>(p);                 \
        else if (vpt <= 8) norm_residual_kernel<ACT, 8><<<rows, 256, 0, s>>>(p);                 \
        else if (vpt <= 16) norm_residual_kernel<ACT, 16><<<rows, 256, 0, s>>>(p);               \
        else if (vpt <= 32) norm_residual_kernel<ACT, 32><<<rows, 256, 0, s>>>(p);               \
        else norm_residual_kernel<ACT, 64><<<rows, 256, 0, s>>>(p);                              \
    } while (0)
    if (ctx->act == NVMAI_ACT_BF16) NVMAI_NR(ACT_BF16); else NVMAI_NR(ACT_FP32);
#undef NVMAI_NR
    return launch_status();
}

extern "C" int nvmai_hip_embed_rows(nvmai_hip_ctx* ctx, nvmai_stream stream, const uint16_t* table, uint32_t table_stride,
                                    const uint32_t* token_ids, uint32_t n_tokens, float* out, uint32_t out_stride, uint32_t d,
                                    uint32_t vocab) {
    if (!ctx || !table || !token_ids || !out || d == 0 || table_stride < d || out_stride < d || vocab == 0) return NVMAI_ERR_INVALID_ARG;
    if (n_tokens == 0) return NVMAI_OK;
    if (n_tokens > 65535) return NVMAI_ERR_UNSUPPORTED;
    embed_rows_kernel<<<dim3((d + 255) / 256, n_tokens), 256, 0, (hipStream_t)stream>>>(table, table_stride, token_ids, out, out_stride, d, vocab);
    return launch_status();
}

extern "C" int nvmai_hip_argmax_rows(nvmai_hip_ctx* ctx, nvmai_stream stream, const float* x, uint32_t x_stride, uint32_t rows,
                                     uint32_t n, uint32_t* out_index) {
    if (!ctx || !x || !out_index || n == 0 || x_stride < n) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    argmax_rows_kernel<<<rows, 1024, 0, (hipStream_t)stream>>>(x, x_stride, n, out_index);
    return launch_status();
}
