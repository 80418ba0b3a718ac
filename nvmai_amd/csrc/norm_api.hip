// Entry points of the norms over the 32-bit residual.
#include "ctx.hpp"
#include "norm_kernels.hpp"

using namespace nvmai;

namespace {

template <int ACT, bool DELTA, int POST, int NEXT>
void norm_residual_sized(const NormResidualParams& p, uint32_t rows, hipStream_t s) {
    const bool vec = p.d % 4 == 0 && p.x_stride % 4 == 0 && aligned16(p.x) && (!DELTA || (p.delta_stride % 4 == 0 && aligned16(p.delta))) &&
                     (NEXT == NORM_NONE || (p.out_stride % 4 == 0 && aligned16(p.out))) && aligned16(p.post_w) && aligned16(p.post_b) &&
                     aligned16(p.next_w) && aligned16(p.next_b);
    const uint32_t vpt = (p.d + 1023) / 1024;
    if (!vec) {
        if (vpt <= 2) norm_residual_kernel<ACT, 2, DELTA, POST, NEXT, false><<<rows, 256, 0, s>>>(p);
        else norm_residual_kernel<ACT, 16, DELTA, POST, NEXT, false><<<rows, 256, 0, s>>>(p);
    } else if (vpt <= 1) norm_residual_kernel<ACT, 1, DELTA, POST, NEXT, true><<<rows, 256, 0, s>>>(p);
    else if (vpt <= 2) norm_residual_kernel<ACT, 2, DELTA, POST, NEXT, true><<<rows, 256, 0, s>>>(p);
    else if (vpt <= 4) norm_residual_kernel<ACT, 4, DELTA, POST, NEXT, true><<<rows, 256, 0, s>>>(p);
    else if (vpt <= 8) norm_residual_kernel<ACT, 8, DELTA, POST, NEXT, true><<<rows, 256, 0, s>>>(p);
    else norm_residual_kernel<ACT, 16, DELTA, POST, NEXT, true><<<rows, 256, 0, s>>>(p);
}

template <int ACT>
int norm_residual(const NormResidualParams& p, int post, int next, uint32_t rows, hipStream_t s) {
#define NVMAI_NR(POST, NEXT) \
    if (p.delta && post == POST && next == NEXT) return norm_residual_sized<ACT, true, POST, NEXT>(p, rows, s), launch_status()
#define NVMAI_NR0(NEXT) \
    if (!p.delta && post == NORM_NONE && next == NEXT) return norm_residual_sized<ACT, false, NORM_NONE, NEXT>(p, rows, s), launch_status()
    NVMAI_NR(NORM_LAYER, NORM_LAYER);
    NVMAI_NR(NORM_LAYER, NORM_NONE);
    NVMAI_NR(NORM_NONE, NORM_LAYER);
    NVMAI_NR(NORM_NONE, NORM_NONE);
    NVMAI_NR(NORM_RMS, NORM_RMS);
    NVMAI_NR(NORM_RMS, NORM_COPY);
    NVMAI_NR(NORM_RMS, NORM_NONE);
    NVMAI_NR0(NORM_LAYER);
    NVMAI_NR0(NORM_RMS);
    if (!p.delta && next == NORM_NONE) return NVMAI_OK;
    return NVMAI_ERR_UNSUPPORTED;
#undef NVMAI_NR
#undef NVMAI_NR0
}

int norm_residual_checked(nvmai_hip_ctx* ctx, nvmai_stream stream, const NormResidualParams& p, int post, int next, uint32_t rows) {
    if (!ctx || !p.x || p.d == 0 || p.x_stride < p.d || (p.delta && p.delta_stride < p.d)) return NVMAI_ERR_INVALID_ARG;
    if ((next == NORM_NONE) != (p.out == nullptr) || (p.out && p.out_stride < p.d)) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (p.d > 16384) return NVMAI_ERR_UNSUPPORTED;
    if (rows == 0) return NVMAI_OK;
    if (post != NORM_NONE && !p.delta) return NVMAI_ERR_INVALID_ARG;
    auto given = [](int kind, const uint16_t* w, const uint16_t* b) {
        return (w != nullptr) == (kind == NORM_LAYER || kind == NORM_RMS) && (b != nullptr) == (kind == NORM_LAYER);
    };
    if (!given(post, p.post_w, p.post_b) || !given(next, p.next_w, p.next_b)) return NVMAI_ERR_INVALID_ARG;
    return ctx->act == NVMAI_ACT_BF16 ? norm_residual<ACT_BF16>(p, post, next, rows, (hipStream_t)stream)
                                      : norm_residual<ACT_FP32>(p, post, next, rows, (hipStream_t)stream);
}

}  // namespace

extern "C" int nvmai_hip_norm_residual(nvmai_hip_ctx* ctx, nvmai_stream stream, float* x, uint32_t x_stride, const float* delta,
                                       uint32_t delta_stride, const uint16_t* post_weight, const uint16_t* post_bias, float mult,
                                       const uint16_t* next_weight, const uint16_t* next_bias, void* out, uint32_t out_stride,
                                       uint32_t rows, uint32_t d, float eps) {
    const NormResidualParams p{x, delta, post_weight, post_bias, next_weight, next_bias, out, x_stride, delta_stride, out_stride, d, mult, eps, 0.0f, 0.0f};
    return norm_residual_checked(ctx, stream, p, post_weight ? NORM_LAYER : NORM_NONE, next_weight ? NORM_LAYER : NORM_NONE, rows);
}

extern "C" int nvmai_hip_rms_residual(nvmai_hip_ctx* ctx, nvmai_stream stream, float* x, uint32_t x_stride, const float* delta,
                                      uint32_t delta_stride, const uint16_t* post_weight, float post_add, const uint16_t* next_weight,
                                      float next_add, void* out, uint32_t out_stride, uint32_t rows, uint32_t d, float eps) {
    const NormResidualParams p{x, delta, post_weight, nullptr, next_weight, nullptr, out, x_stride, delta_stride, out_stride, d, 1.0f, eps, post_add, next_add};
    return norm_residual_checked(ctx, stream, p, post_weight ? NORM_RMS : NORM_NONE, next_weight ? NORM_RMS : out ? NORM_COPY : NORM_NONE, rows);
}
