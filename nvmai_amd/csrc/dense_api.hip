// Entry points of the dense models: matrix products against BF16 weights, embedding rows, the cap of the
// logits, argmax.
#include "ctx.hpp"
#include "dense_kernels.hpp"
#include "dense_internal.hpp"

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

template <int ACT, int NT>
static void launch_gemv(const DenseLinearParams& p, hipStream_t s) {
    // rows per wave: one (short blocks, many of them) until the inputs' own loads weigh more than that
    if (p.n >= 65536) dense_gemv_kernel<ACT, NT, 4><<<(p.n + 15) / 16, 256, 0, s>>>(p);
    else if (p.activation == NVMAI_LINEAR_SILU_PAIRS || (NT * (ACT == ACT_FP32 ? 2 : 1) > 2 && p.n >= 8192)) dense_gemv_kernel<ACT, NT, 2><<<(p.n + 7) / 8, 256, 0, s>>>(p);
    else dense_gemv_kernel<ACT, NT, 1><<<(p.n + 3) / 4, 256, 0, s>>>(p);
}

template <int ACT>
static int gemv(const DenseLinearParams& p, hipStream_t s) {
    if (p.rows == 1) launch_gemv<ACT, 1>(p, s);
    else if (p.rows == 2) launch_gemv<ACT, 2>(p, s);
    else if (p.rows == 3) launch_gemv<ACT, 3>(p, s);
    else launch_gemv<ACT, 4>(p, s);
    return launch_status();
}

int dense_linear(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) {
    const int rc = dense_linear_check(ctx, p);
    if (rc) return rc;
    if (p.rows == 0) return NVMAI_OK;
    if (p.rows <= 4) return ctx->act == NVMAI_ACT_FP32 ? gemv<ACT_FP32>(p, s) : gemv<ACT_BF16>(p, s);
    if (ctx->act == NVMAI_ACT_FP32) {
        const dim3 grid((p.n + 63) / 64, (p.rows + 63) / 64);
        if (grid.y > 65535) return NVMAI_ERR_UNSUPPORTED;
        dense_f32_kernel<<<grid, 256, 0, s>>>(p);
        return launch_status();
    }
    if (p.rows <= 64) {
        // row tiles per block: as many as leave every compute unit several blocks; waves: about four steps of k each
        const int nr = p.n >= 32768 ? 4 : p.n >= 8192 ? 2 : 1;
        const uint32_t blocks = (p.n + 16 * nr - 1) / (16 * nr);
#define NVMAI_SKINNY(TT)                                                              \
    do {                                                                              \
        if (nr == 4) dense_skinny_kernel<TT, 4, 4><<<blocks, 256, 0, s>>>(p);         \
        else if (nr == 2) dense_skinny_kernel<TT, 2, 4><<<blocks, 256, 0, s>>>(p);    \
        else if (p.k <= 1024) dense_skinny_kernel<TT, 1, 4><<<blocks, 256, 0, s>>>(p); \
        else if (p.k <= 2048) dense_skinny_kernel<TT, 1, 8><<<blocks, 512, 0, s>>>(p); \
        else dense_skinny_kernel<TT, 1, 16><<<blocks, 1024, 0, s>>>(p);               \
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
