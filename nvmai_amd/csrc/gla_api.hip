// Entry point of gated linear attention.
#include "ctx.hpp"
#include "gla_kernels.hpp"

using namespace nvmai;

namespace {

template <int ACT, int PER, uint32_t NTH>
int gla_recurrent_sized(const GlaParams& p, uint32_t batch, hipStream_t s) {
    const size_t groups = NTH / p.dv, chans = PER > 0 ? groups * PER : p.dk;
    if (chans > NTH) return NVMAI_ERR_UNSUPPORTED;
    const size_t lds = (3 * chans + 16 + groups * p.dv + p.rank) * 4;
    if (lds > 64 * 1024) return NVMAI_ERR_UNSUPPORTED;
    gla_recurrent_kernel<ACT, PER, NTH><<<dim3(p.heads, batch), NTH, lds, s>>>(p);
    return launch_status();
}

template <int ACT>
int gla_recurrent(const GlaParams& p, uint32_t batch, hipStream_t s) {
    auto per = [&](uint32_t threads) { return (p.dk + threads / p.dv - 1) / (threads / p.dv); };
    if (per(1024) <= 4) return gla_recurrent_sized<ACT, 4, 1024>(p, batch, s);
    if (per(1024) <= 8) return gla_recurrent_sized<ACT, 8, 1024>(p, batch, s);
    if (per(1024) <= 16) return gla_recurrent_sized<ACT, 16, 1024>(p, batch, s);
    if (per(1024) <= 32) return gla_recurrent_sized<ACT, 32, 1024>(p, batch, s);
    return gla_recurrent_sized<ACT, 0, 1024>(p, batch, s);
}

template <int ACT, int KT>
void gla_spans(const GlaParams& p, uint32_t subs, uint32_t spans, hipStream_t s) {
    const dim3 grid(spans, p.heads);
    const uint32_t threads = p.dv * 4u;              // a wave per sixteen value columns
    gla_span_kernel<ACT, KT, false><<<grid, threads, 0, s>>>(p);
    gla_span_decay_kernel<<<dim3((p.heads * p.dk + 255) / 256, spans), 256, 0, s>>>(p, subs);
    gla_scan_kernel<<<dim3((p.dk * p.dv / 4 + 255) / 256, p.heads), 256, 0, s>>>(p, spans);
    gla_span_kernel<ACT, KT, true><<<grid, threads, 0, s>>>(p);
}

template <int ACT>
int gla_chunked(const GlaParams& p, hipStream_t s) {
    const uint32_t subs = (p.rows + GLA_SUB - 1) / GLA_SUB, spans = (subs + p.span - 1) / p.span;
    const size_t lds = ((size_t)48 * (p.dk + 4) + 2 * (size_t)p.dk + 1024 + (size_t)16 * p.rank) * 4;
    static bool raised = false;
    if (!raised) {
        NVMAI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(gla_prep_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024));
        raised = true;
    }
    if (lds > 128 * 1024) return NVMAI_ERR_UNSUPPORTED;
    gla_prep_kernel<<<dim3(subs, p.heads), 256, lds, s>>>(p);
    const uint32_t kt = (p.dk + 15) / 16;
    if (kt <= 2) gla_spans<ACT, 2>(p, subs, spans, s);
    else if (kt <= 4) gla_spans<ACT, 4>(p, subs, spans, s);
    else if (kt <= 8) gla_spans<ACT, 8>(p, subs, spans, s);
    else gla_spans<ACT, 16>(p, subs, spans, s);
    return launch_status();
}

}  // namespace

extern "C" int nvmai_hip_gla(nvmai_hip_ctx* ctx, nvmai_stream stream, const nvmai_gla_config* config, const float* q, const float* k,
                             const float* v, const float* g, const float* a1, uint32_t proj_stride, const uint16_t* a2,
                             const uint16_t* a2_bias, const uint16_t* norm_weight, float* state, const uint32_t* slots,
                             uint32_t slot, void* out, uint32_t out_stride, uint32_t rows, uint32_t batch, int form) {
    if (!ctx || !config || !q || !k || !v || !g || !a1 || !a2 || !a2_bias || !norm_weight || !state || !out) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    const nvmai_gla_config& c = *config;
    if (c.heads == 0 || c.key_dim == 0 || c.value_dim == 0 || c.rank == 0 || c.value_count == 0 || c.value_count > c.value_dim) return NVMAI_ERR_INVALID_ARG;
    if (c.key_dim % 16 || c.value_dim % 16 || c.rank % 8) return NVMAI_ERR_INVALID_ARG;
    if (c.value_dim > 512 || c.key_dim > 512 || c.rank > 512) return NVMAI_ERR_UNSUPPORTED;
    if (!(c.tau > 0.0f)) return NVMAI_ERR_INVALID_ARG;
    if (proj_stride < c.heads * c.key_dim || proj_stride < c.heads * c.value_dim || proj_stride < c.rank || out_stride < c.heads * c.value_dim)
        return NVMAI_ERR_INVALID_ARG;
    if (!aligned16(a2) || !aligned16(state)) return NVMAI_ERR_ALIGNMENT;
    if (form < NVMAI_FORM_AUTO || form > NVMAI_GLA_CHUNKED) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0 || batch == 0) return NVMAI_OK;
    if (batch > 65535) return NVMAI_ERR_UNSUPPORTED;
    GlaParams p{};
    p.q = q; p.k = k; p.v = v; p.g = g; p.a1 = a1; p.a2 = a2; p.a2_bias = a2_bias; p.norm_weight = norm_weight;
    p.state = state; p.slots = slots; p.slot0 = slot; p.out = out; p.proj_stride = proj_stride; p.out_stride = out_stride;
    p.heads = c.heads; p.dk = c.key_dim; p.dv = c.value_dim; p.dv_count = c.value_count; p.rank = c.rank; p.rows = rows;
    p.inv_tau = 1.0f / c.tau; p.q_scale = c.q_scale; p.eps = c.eps;
    hipStream_t s = (hipStream_t)stream;
    const bool can_chunk = batch == 1 && !slots && c.key_dim <= GLA_MAX_DIM && c.value_dim <= GLA_MAX_DIM;
    if (form == NVMAI_GLA_CHUNKED && !can_chunk) return NVMAI_ERR_UNSUPPORTED;
    // below two spans' worth of rows the launches of the chunked form cost more than the rows
    const bool chunk = form == NVMAI_GLA_CHUNKED || (form == NVMAI_FORM_AUTO && can_chunk && rows >= 32);
    if (!chunk) return ctx->act == NVMAI_ACT_BF16 ? gla_recurrent<ACT_BF16>(p, batch, s) : gla_recurrent<ACT_FP32>(p, batch, s);
    const size_t subs = (rows + GLA_SUB - 1) / GLA_SUB;
    // long spans (fewer states through memory) as soon as they still make two blocks per compute unit
    p.span = (subs / 8) * c.heads >= 2 * (size_t)ctx->compute_units ? 8 : 4;
    const size_t spans = (subs + p.span - 1) / p.span;
    if (spans > 65535) return NVMAI_ERR_UNSUPPORTED;
    const size_t n_qd = subs * c.heads * 16 * c.key_dim, n_edge = subs * c.heads * c.key_dim, n_att = subs * c.heads * 256;
    const size_t n_spans = spans * c.heads * c.key_dim * c.value_dim, n_dec = spans * c.heads * c.key_dim;
    const int rc = ws_begin(ctx, stream, 2 * ws_round(n_qd * 4) + ws_round(n_edge * 4) + ws_round(n_att * 4) + ws_round(n_spans * 4) + ws_round(n_dec * 4));
    if (rc) return rc;
    p.qd = ws_take<float>(ctx, n_qd);
    p.kd = ws_take<float>(ctx, n_qd);
    p.edge = ws_take<float>(ctx, n_edge);
    p.att = ws_take<float>(ctx, n_att);
    p.spans = ws_take<float>(ctx, n_spans);
    p.span_decay = ws_take<float>(ctx, n_dec);
    return ctx->act == NVMAI_ACT_BF16 ? gla_chunked<ACT_BF16>(p, s) : gla_chunked<ACT_FP32>(p, s);
}
