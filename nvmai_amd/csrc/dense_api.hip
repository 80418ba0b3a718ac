// Entry points of the dense models: matrix products against BF16 weights, embedding rows, the cap of the
// logits, argmax.
#include "ctx.hpp"
#include "dense_kernels.hpp"
#include "ends_kernels.hpp"

using namespace nvmai;

namespace nvmai {

int dense_linear_check(const nvmai_hip_ctx* ctx, const DenseLinearParams& p) {
    if (!ctx || !p.w || !p.x || (!p.y && !p.y_f32)) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (p.k == 0 || p.k % 64 || p.n == 0 || p.w_stride < p.k || p.x_stride < p.k) return NVMAI_ERR_INVALID_ARG;
    if (p.activation < NVMAI_LINEAR_NONE || p.activation > NVMAI_LINEAR_SILU_PAIRS) return NVMAI_ERR_UNSUPPORTED;
    const bool pairs = p.activation == NVMAI_LINEAR_SILU_PAIRS;
    if (p.y_stride < (pairs ? p.n / 2 : p.n)) return NVMAI_ERR_INVALID_ARG;
    if (pairs && (p.n % 2 || p.y_stride % 2 || p.bias || p.mul)) return NVMAI_ERR_INVALID_ARG;
    if (p.mul && (!p.mul_ids || p.mul_stride < p.n)) return NVMAI_ERR_INVALID_ARG;
    if (!aligned16(p.w) || !aligned16(p.x) || p.w_stride % 8 || p.x_stride % 8) return NVMAI_ERR_ALIGNMENT;
    if ((p.y && !aligned16(p.y)) || (p.y_f32 && !aligned16(p.y_f32))) return NVMAI_ERR_ALIGNMENT;
    // 32-bit byte offsets inside an operand
    if ((uint64_t)p.n * p.w_stride * 2 > 0xFFFFFFFFull || (uint64_t)p.rows * p.x_stride * 4 > 0xFFFFFFFFull) return NVMAI_ERR_UNSUPPORTED;
    return NVMAI_OK;
}

int dense_linear(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) {
    const int rc = dense_linear_check(ctx, p);
    if (rc) return rc;
    if (p.rows == 0) return NVMAI_OK;
    if (p.activation == NVMAI_LINEAR_SILU_PAIRS) return dense_launch_pairs(ctx, s, p);
    if (p.mul || p.activation == NVMAI_LINEAR_GELU_TANH || (p.bias && p.activation != NVMAI_LINEAR_NONE)) return dense_launch_full(ctx, s, p);
    if (p.bias) return dense_launch_bias(ctx, s, p);
    return p.activation == NVMAI_LINEAR_GELU_ERF ? dense_launch_erf(ctx, s, p) : dense_launch<DE_PLAIN>(ctx, s, p);
}

}  // namespace nvmai

extern "C" int nvmai_hip_dense_linear(nvmai_hip_ctx* ctx, nvmai_stream stream, const uint16_t* w, uint32_t w_stride,
                                      const void* x, uint32_t x_stride, uint32_t rows, uint32_t n, uint32_t k, void* y,
                                      float* y_f32, uint32_t y_stride, int activation) {
    const DenseLinearParams p{w, x, y, y_f32, w_stride, x_stride, y_stride, rows, n, k, activation};
    return dense_linear(ctx, (hipStream_t)stream, p);
}

extern "C" int nvmai_hip_dense_linear_ex(nvmai_hip_ctx* ctx, nvmai_stream stream, const uint16_t* w, uint32_t w_stride, const void* x,
                                         uint32_t x_stride, uint32_t rows, uint32_t n, uint32_t k, void* y, float* y_f32,
                                         uint32_t y_stride, const nvmai_linear_epilogue* e) {
    if (!e) return NVMAI_ERR_INVALID_ARG;
    const DenseLinearParams p{w, x, y, y_f32, w_stride, x_stride, y_stride, rows, n, k, e->activation, e->bias, e->mul, e->mul_ids,
                              e->mul_stride, e->mul_rows};
    return dense_linear(ctx, (hipStream_t)stream, p);
}

extern "C" int nvmai_hip_embed_rows(nvmai_hip_ctx* ctx, nvmai_stream stream, const uint16_t* table, uint32_t table_stride,
                                    const uint32_t* token_ids, uint32_t n_tokens, float* out, uint32_t out_stride, uint32_t d,
                                    uint32_t vocab) {
    return nvmai_hip_embed_positions(ctx, stream, table, table_stride, token_ids, n_tokens, 1.0f, nullptr, nullptr, out, out_stride, nullptr, 0, d, vocab);
}

extern "C" int nvmai_hip_embed_positions(nvmai_hip_ctx* ctx, nvmai_stream stream, const uint16_t* table, uint32_t table_stride,
                                         const uint32_t* token_ids, uint32_t n_tokens, float scale, const double* inv_freq,
                                         const nvmai_row_map* map, float* out, uint32_t out_stride, void* act, uint32_t act_stride,
                                         uint32_t d, uint32_t vocab) {
    if (!ctx || !table || !token_ids || !out || d == 0 || table_stride < d || out_stride < d || vocab == 0) return NVMAI_ERR_INVALID_ARG;
    if ((inv_freq && !map) || (act && act_stride < d)) return NVMAI_ERR_INVALID_ARG;
    if (act && ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (n_tokens == 0) return NVMAI_OK;
    if (n_tokens > 65535) return NVMAI_ERR_UNSUPPORTED;
    EmbedParams p{table, token_ids, out, act, inv_freq, SeqRows{}, table_stride, out_stride, act_stride, d, vocab, scale};
    if (map) p.rows = SeqRows{map->slots, map->positions, map->slot, map->position};
    const dim3 grid((d + 511) / 512, n_tokens);
    if (ctx->act == NVMAI_ACT_FP32) embed_rows_kernel<ACT_FP32><<<grid, 256, 0, (hipStream_t)stream>>>(p);
    else embed_rows_kernel<ACT_BF16><<<grid, 256, 0, (hipStream_t)stream>>>(p);
    return launch_status();
}

extern "C" int nvmai_hip_softcap_rows(nvmai_hip_ctx* ctx, nvmai_stream stream, float* x, uint32_t x_stride, uint32_t rows, uint32_t n,
                                      float cap) {
    if (!ctx || !x || n == 0 || x_stride < n || !(cap > 0.0f)) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    if (rows > 65535) return NVMAI_ERR_UNSUPPORTED;
    softcap_rows_kernel<<<dim3((n + 255) / 256, rows), 256, 0, (hipStream_t)stream>>>(x, x_stride, n, cap);
    return launch_status();
}

extern "C" int nvmai_hip_argmax_rows(nvmai_hip_ctx* ctx, nvmai_stream stream, const float* x, uint32_t x_stride, uint32_t rows,
                                     uint32_t n, uint32_t* out_index) {
    if (!ctx || !x || !out_index || n == 0 || x_stride < n) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    if (rows > 65535) return NVMAI_ERR_UNSUPPORTED;
    const int rc = ws_begin(ctx, stream, ws_round((size_t)rows * ARGMAX_BLOCKS * 8));
    if (rc) return rc;
    uint64_t* part = ws_take<uint64_t>(ctx, (size_t)rows * ARGMAX_BLOCKS);
    uint32_t blocks = (n + 1023) / 1024;
    if (blocks > ARGMAX_BLOCKS) blocks = ARGMAX_BLOCKS;
    argmax_stage1_kernel<<<dim3(blocks, rows), 256, 0, (hipStream_t)stream>>>(x, x_stride, n, part);
    argmax_stage2_kernel<<<rows, 256, 0, (hipStream_t)stream>>>(part, blocks, out_index);
    return launch_status();
}
