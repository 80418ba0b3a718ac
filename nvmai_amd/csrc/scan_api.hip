// Entry points of the recurrences with one decay per head and of their gated norm.
#include "ctx.hpp"
#include "scan_kernels.hpp"

using namespace nvmai;

namespace {

template <bool DELTA, int CP>
int recurrent_launch(const ScanParams& p, uint32_t sequences, uint32_t seq_rows, hipStream_t s) {
    const uint32_t per = (p.dk + 15) / 16;
    const dim3 grid(p.heads, p.dv / (16 * CP), sequences);
    if (per <= 2) scan_recurrent_kernel<DELTA, 2, CP><<<grid, 256, 0, s>>>(p, seq_rows);
    else if (per <= 4) scan_recurrent_kernel<DELTA, 4, CP><<<grid, 256, 0, s>>>(p, seq_rows);
    else if (per <= 8) scan_recurrent_kernel<DELTA, 8, CP><<<grid, 256, 0, s>>>(p, seq_rows);
    else if (CP == 1 && per <= 16) scan_recurrent_kernel<DELTA, 16, 1><<<grid, 256, 0, s>>>(p, seq_rows);
    else if (CP == 1) scan_recurrent_kernel<DELTA, 32, 1><<<grid, 256, 0, s>>>(p, seq_rows);
    return launch_status();
}

template <bool DELTA>
int recurrent(ScanParams p, bool by_arrays, uint32_t compute_units, hipStream_t s) {
    // four columns per thread when blocks of sixteen columns would come in several rounds
    const bool wide = by_arrays && p.dv % 64 == 0 && p.dk <= 128 && aligned16(p.state) && (uint64_t)p.heads * (p.dv / 16) * p.n_rows > 4ull * compute_units;
    if (wide) return recurrent_launch<DELTA, 4>(p, p.n_rows, 1, s);
    if (by_arrays) return recurrent_launch<DELTA, 1>(p, p.n_rows, 1, s);
    // consecutive rows: SCAN_AHEAD of them per launch, so that a launch overwrites no history it reads
    const uint32_t rows = p.n_rows;
    for (uint32_t t0 = 0; t0 < rows; t0 += SCAN_AHEAD) {
        p.n_rows = rows - t0 < SCAN_AHEAD ? rows - t0 : SCAN_AHEAD;
        const int rc = recurrent_launch<DELTA, 1>(p, 1, p.n_rows, s);
        if (rc) return rc;
        p.proj += (size_t)p.n_rows * p.proj_stride;
        p.out += (size_t)p.n_rows * p.out_stride;
        p.rows.position += p.n_rows;
    }
    return NVMAI_OK;
}

template <bool DELTA, int TAPS, bool FAST>
void filter(const ScanParams& p, hipStream_t s) {
    const dim3 grid((p.n_rows + SCAN_CHUNK - 1) / SCAN_CHUNK * (SCAN_CHUNK / SCAN_RUN), (2 * p.key_heads + p.heads + 4) / 4);
    const uint32_t dim = p.dk > p.dv ? p.dk : p.dv;
    if (dim <= 64) scan_filter_kernel<DELTA, 1, TAPS, FAST><<<grid, 256, 0, s>>>(p);
    else if (dim <= 128) scan_filter_kernel<DELTA, 2, TAPS, FAST><<<grid, 256, 0, s>>>(p);
    else scan_filter_kernel<DELTA, 4, TAPS, FAST><<<grid, 256, 0, s>>>(p);
}

template <bool DELTA>
int chunked(const ScanParams& p, uint32_t chunks, bool fast, hipStream_t s) {
    const size_t q_part = (size_t)64 * (p.dk + 4), l_part = DELTA ? 64 * 68 : 0, lds = (q_part + (q_part > l_part ? q_part : l_part)) * 4;
    if (lds > 159 * 1024) return NVMAI_ERR_UNSUPPORTED;
    if (lds > 63 * 1024) NVMAI_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void*>(scan_prep_kernel<DELTA>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    if (p.taps != 4) filter<DELTA, 0, false>(p, s);
    else if (fast) filter<DELTA, 4, true>(p, s);
    else filter<DELTA, 4, false>(p, s);
    if (p.taps > 1) scan_history_kernel<<<dim3((p.channels + 255) / 256, p.taps - 1), 256, 0, s>>>(p);
    // heads of one block: the state-space form shares q k^T among the heads of a group
    const uint32_t ratio = p.heads / p.key_heads, per = DELTA ? 1 : ratio < 8 ? ratio : 8;
    scan_prep_kernel<DELTA><<<dim3(chunks, p.key_heads * ((ratio + per - 1) / per)), 256, lds, s>>>(p, per);
    const dim3 grid(p.heads, p.dv / 16);
    if (p.dk <= 64) scan_chain_kernel<DELTA, 4, 2><<<grid, 512, 0, s>>>(p, chunks);
    else if (p.dk <= 128) scan_chain_kernel<DELTA, 8, 2><<<grid, 512, 0, s>>>(p, chunks);
    else scan_chain_kernel<DELTA, 16, 1><<<grid, 512, 0, s>>>(p, chunks);
    return launch_status();
}

template <int ACT, bool FIRST>
int gated_norm(const GatedNormParams& p, hipStream_t s) {
    const uint32_t n = p.heads * p.dv_count / p.parts;
    const bool vec = p.dv_count % 4 == 0 && n % 4 == 0 && p.x_head % 4 == 0 && p.dv % 4 == 0 && p.x_stride % 4 == 0 && p.gate_stride % 4 == 0 && p.out_stride % 4 == 0 && aligned16(p.x) &&
                     aligned16(p.gate) && aligned16(p.out);
    if (vec && n <= 128) gated_norm_kernel<ACT, FIRST, 32, 1, true><<<dim3(p.rows, (p.parts + 7) / 8), 256, 0, s>>>(p);
    else if (vec && n <= 512) gated_norm_kernel<ACT, FIRST, 64, 2, true><<<dim3(p.rows, (p.parts + 3) / 4), 256, 0, s>>>(p);
    else if (vec && n <= 4096) gated_norm_kernel<ACT, FIRST, 256, 4, true><<<dim3(p.rows, p.parts), 256, 0, s>>>(p);
    else if (vec && n <= 16384) gated_norm_kernel<ACT, FIRST, 1024, 4, true><<<dim3(p.rows, p.parts), 1024, 0, s>>>(p);
    else if (n <= 512) gated_norm_kernel<ACT, FIRST, 64, 8, false><<<dim3(p.rows, (p.parts + 3) / 4), 256, 0, s>>>(p);
    else gated_norm_kernel<ACT, FIRST, 256, 8, false><<<dim3(p.rows, p.parts), 256, 0, s>>>(p);
    return launch_status();
}

}  // namespace

extern "C" int nvmai_hip_scan(nvmai_hip_ctx* ctx, nvmai_stream stream, const nvmai_scan_config* config, const float* proj, uint32_t proj_stride,
                              const uint16_t* conv, const uint16_t* conv_bias, const uint16_t* a_log, const uint16_t* dt_bias, const uint16_t* skip,
                              float* history, float* state, const nvmai_row_map* map, float* out, uint32_t out_stride, uint64_t out_head_stride, uint32_t rows, int form) {
    if (!ctx || !config || !proj || !conv || !a_log || !dt_bias || !history || !state || !map || !out) return NVMAI_ERR_INVALID_ARG;
    const nvmai_scan_config& c = *config;
    const bool delta = c.kind == NVMAI_SCAN_DELTA;
    if ((c.kind != NVMAI_SCAN_DELTA && c.kind != NVMAI_SCAN_SSD) || (!delta && !skip)) return NVMAI_ERR_INVALID_ARG;
    if (c.heads == 0 || c.key_heads == 0 || c.heads % c.key_heads || c.key_dim == 0 || c.value_dim == 0 || c.key_dim % 16 || c.value_dim % 16 || c.taps == 0)
        return NVMAI_ERR_INVALID_ARG;
    if (c.key_dim > 512 || c.value_dim > 512 || c.heads > 65535) return NVMAI_ERR_UNSUPPORTED;
    const uint64_t channels = 2ull * c.key_heads * c.key_dim + (uint64_t)c.heads * c.value_dim;
    if (c.history_rows < c.taps - 1 + SCAN_AHEAD || proj_stride < c.conv_at + channels || proj_stride < c.a_at + c.heads ||
        (delta && proj_stride < c.b_at + c.heads) || out_stride < c.value_dim || out_head_stride < c.value_dim) return NVMAI_ERR_INVALID_ARG;
    if ((map->slots == nullptr) != (map->positions == nullptr) || form < NVMAI_FORM_AUTO || form > NVMAI_SCAN_CHUNKED) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    const bool by_arrays = map->positions != nullptr;
    if (by_arrays && rows > 65535) return NVMAI_ERR_UNSUPPORTED;
    ScanParams p{};
    p.proj = proj; p.conv = conv; p.conv_bias = conv_bias; p.a_log = a_log; p.dt_bias = dt_bias; p.skip = skip; p.history = history; p.state = state;
    p.out = out; p.out_head = out_head_stride; p.rows = SeqRows{map->slots, map->positions, map->slot, map->position}; p.proj_stride = proj_stride; p.out_stride = out_stride;
    p.n_rows = rows; p.heads = c.heads; p.key_heads = c.key_heads; p.dk = c.key_dim; p.dv = c.value_dim; p.taps = c.taps;
    p.history_rows = c.history_rows; p.conv_at = c.conv_at; p.a_at = c.a_at; p.b_at = c.b_at; p.channels = (uint32_t)channels; p.q_scale = c.q_scale;
    hipStream_t s = (hipStream_t)stream;
    const uint32_t chunks = (rows + SCAN_CHUNK - 1) / SCAN_CHUNK;
    const bool can_chunk = !by_arrays && c.key_dim <= 256 && c.value_dim <= 256 && c.taps <= 65536 && channels <= (1u << 24);
    if (form == NVMAI_SCAN_CHUNKED && !can_chunk) return NVMAI_ERR_UNSUPPORTED;
    if (form != NVMAI_SCAN_CHUNKED && !(form == NVMAI_FORM_AUTO && can_chunk && rows >= SCAN_AHEAD))
        return delta ? recurrent<true>(p, by_arrays, (uint32_t)ctx->compute_units, s) : recurrent<false>(p, by_arrays, (uint32_t)ctx->compute_units, s);
    p.rows_p = chunks * SCAN_CHUNK;
    const size_t cells = (size_t)chunks * c.heads, n_mixed = (size_t)p.rows_p * channels, n_in = (size_t)p.rows_p * c.heads, n_kt = delta ? cells * 64 * c.key_dim : 0, n_u0 = delta ? cells * 64 * c.value_dim : 0, n_k = (size_t)chunks * c.key_heads * 64 * c.key_dim;
    const int rc = ws_begin(ctx, stream, ws_round(n_mixed * 4) + 2 * ws_round(n_in * 4) + ws_round(cells * 4096 * 4) + ws_round(cells * 192 * 4) + ws_round(n_kt * 4) + ws_round(n_u0 * 4) + ws_round(n_k * 4));
    if (rc) return rc;
    p.mixed = ws_take<float>(ctx, n_mixed);
    p.in_a = ws_take<float>(ctx, n_in);
    p.in_b = ws_take<float>(ctx, n_in);
    p.w = ws_take<float>(ctx, cells * 4096);
    p.gates = ws_take<float>(ctx, cells * 192);
    p.kt = ws_take<float>(ctx, n_kt);
    p.u0 = ws_take<float>(ctx, n_u0);
    p.k_t = ws_take<float>(ctx, n_k);
    const bool fast = ctx->act != NVMAI_ACT_FP32;    // the filter's activation by the hardware exponential (1e-6)
    return delta ? chunked<true>(p, chunks, fast, s) : chunked<false>(p, chunks, fast, s);
}

extern "C" int nvmai_hip_gated_norm(nvmai_hip_ctx* ctx, nvmai_stream stream, const float* x, uint32_t x_stride, uint64_t x_head_stride,
                                    const float* gate, uint32_t gate_stride, const uint16_t* weight, void* out, uint32_t out_stride, uint32_t rows, uint32_t heads,
                                    uint32_t value_dim, uint32_t value_count, uint32_t parts, int gate_first, float out_scale, float eps) {
    if (!ctx || !x || !gate || !weight || !out || heads == 0 || value_count == 0 || value_count > value_dim || parts == 0) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if ((heads * value_count) % parts || x_stride < value_dim || x_head_stride < value_dim || gate_stride < heads * value_dim || out_stride < heads * value_dim || parts > 65535)
        return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    const GatedNormParams p{x, gate, weight, out, x_head_stride, x_stride, gate_stride, out_stride, rows, heads, value_dim, value_count, parts, out_scale, eps};
    hipStream_t s = (hipStream_t)stream;
    if (ctx->act == NVMAI_ACT_BF16) return gate_first ? gated_norm<ACT_BF16, true>(p, s) : gated_norm<ACT_BF16, false>(p, s);
    return gate_first ? gated_norm<ACT_FP32, true>(p, s) : gated_norm<ACT_FP32, false>(p, s);
}
