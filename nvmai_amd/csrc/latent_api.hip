// Entry points of latent attention.
#include "ctx.hpp"
#include "dense_internal.hpp"
#include "latent_kernels.hpp"

using namespace nvmai;

namespace {

int check_config(const nvmai_hip_ctx* ctx, const nvmai_latent_config* c, const nvmai_latent_cache* cache) {
    if (!ctx || !c || !cache || !cache->base) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (c->heads == 0 || c->nope_dim == 0 || c->value_dim == 0 || c->rank == 0) return NVMAI_ERR_INVALID_ARG;
    if (c->nope_dim % 16 || c->rope_dim % 16 || c->value_dim % 16 || c->rank % 64) return NVMAI_ERR_INVALID_ARG;
    if (c->rotary_dims > c->rope_dim || c->rotary_dims % 2 || (c->rotary_dims && !c->inv_freq)) return NVMAI_ERR_INVALID_ARG;
    if (c->rank_count == 0 || c->rank_count > c->rank) return NVMAI_ERR_INVALID_ARG;
    if (cache->type != ctx->act && !(ctx->act == NVMAI_ACT_FP32 && cache->type == NVMAI_ACT_BF16)) return NVMAI_ERR_UNSUPPORTED;
    if (cache->row_stride < c->rank + c->rope_dim || cache->row_stride % 32 || cache->capacity < 64) return NVMAI_ERR_INVALID_ARG;
    if (!aligned16(cache->base) || cache->slot_stride % 8 || cache->slot_stride < (uint64_t)cache->capacity * cache->row_stride) return NVMAI_ERR_ALIGNMENT;
    return NVMAI_OK;
}

SeqRows rows_of(const nvmai_row_map* m) { return SeqRows{m->slots, m->positions, m->slot, m->position}; }
LatentCache cache_of(const nvmai_latent_cache* c) { return LatentCache{c->base, c->slot_stride, c->row_stride, c->capacity}; }

int raise_lds(const void* kernel, size_t bytes) {
    if (bytes > 160 * 1024) return NVMAI_ERR_UNSUPPORTED;
    if (bytes > 64 * 1024) NVMAI_HIP_TRY(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
    return NVMAI_OK;
}

template <int NT>
int launch_partial(const LatentAttnParams& p, hipStream_t s) {
    const size_t lds = (size_t)p.rank * 80;
    const int rc = raise_lds(reinterpret_cast<const void*>(latent_partial_mfma_kernel<NT>), lds);
    if (rc) return rc;
    latent_partial_mfma_kernel<NT><<<dim3(p.splits, (p.heads + 15) / 16, p.n_rows), 256, lds, s>>>(p);
    return NVMAI_OK;
}

template <int ACT, int CT>
int absorbed(const LatentAttnParams& p, hipStream_t s) {
    const size_t lds_a = (size_t)p.nope * 4;
    int rc = raise_lds(reinterpret_cast<const void*>(latent_absorb_kernel<ACT, CT>), lds_a);
    if (rc) return rc;
    latent_absorb_kernel<ACT, CT><<<dim3(p.heads, p.n_rows, (p.rank + 127) / 128 + 1), 256, lds_a, s>>>(p);
    const uint32_t rest = p.cache.row_stride - p.rank;
    if (CT == ACT_BF16 && p.rank <= 1024 && rest <= 128) {
        rc = p.rank <= 128 ? launch_partial<2>(p, s) : p.rank <= 256 ? launch_partial<4>(p, s) : p.rank <= 512 ? launch_partial<8>(p, s) : launch_partial<16>(p, s);
    } else {
        const size_t lds = ((size_t)p.cache.row_stride + p.rank + 256 + 8) * 4;
        rc = raise_lds(reinterpret_cast<const void*>(latent_partial_plain_kernel<CT>), lds);
        if (!rc) latent_partial_plain_kernel<CT><<<dim3(p.splits, p.heads, p.n_rows), 256, lds, s>>>(p);
    }
    if (rc) return rc;
    const size_t lds_c = (9 * (size_t)p.rank + p.splits) * 4;
    rc = raise_lds(reinterpret_cast<const void*>(latent_combine_kernel<ACT>), lds_c);
    if (rc) return rc;
    latent_combine_kernel<ACT><<<dim3(p.heads, p.n_rows), 1024, lds_c, s>>>(p);
    return launch_status();
}

template <int NP, int RP, int DV>
int launch_flash(const LatentAttnParams& p, hipStream_t s) {
    const size_t lds = 2 * ((size_t)64 * (NP + RP) * 2 + (size_t)DV * 128);
    const int rc = raise_lds(reinterpret_cast<const void*>(latent_flash_kernel<NP, RP, DV>), lds);
    if (rc) return rc;
    latent_flash_kernel<NP, RP, DV><<<(p.n_rows + 127) / 128 * p.heads, 256, lds, s>>>(p);
    return launch_status();
}

template <int NP, int RP>
int launch_flash_v(const LatentAttnParams& p, hipStream_t s) {
    return p.vdim <= 64 ? launch_flash<NP, RP, 64>(p, s) : launch_flash<NP, RP, 128>(p, s);
}

}  // namespace

extern "C" int nvmai_hip_latent_epilogue(nvmai_hip_ctx* ctx, nvmai_stream stream, const nvmai_latent_config* config, const void* proj,
                                         uint32_t proj_stride, uint32_t q_at, uint32_t q_count, const uint16_t* q_norm,
                                         uint32_t kv_at, uint32_t rope_at, const uint16_t* kv_norm, void* cq, uint32_t cq_stride,
                                         const nvmai_latent_cache* cache, const nvmai_row_map* map, uint32_t rows) {
    const int rc = check_config(ctx, config, cache);
    if (rc) return rc;
    const nvmai_latent_config& c = *config;
    if (!proj || !q_norm || !kv_norm || !cq || !map || q_count == 0 || cq_stride < q_count) return NVMAI_ERR_INVALID_ARG;
    if (q_at % 8 || kv_at % 8 || proj_stride % 8 || cq_stride % 8 || !aligned16(proj) || !aligned16(cq) || !aligned16(q_norm) || !aligned16(kv_norm))
        return NVMAI_ERR_ALIGNMENT;
    if (cq_stride < (q_count + 7) / 8 * 8) return NVMAI_ERR_INVALID_ARG;
    if (proj_stride < q_at + q_count || proj_stride < kv_at + c.rank_count || proj_stride < rope_at + c.rope_dim) return NVMAI_ERR_INVALID_ARG;
    if (!map->positions && rows > cache->capacity) return NVMAI_ERR_INVALID_ARG;       // two rows of one call in one place
    if (rows == 0) return NVMAI_OK;
    LatentEpilogueParams p{};
    p.proj = proj; p.q_norm = q_norm; p.kv_norm = kv_norm; p.inv_freq = c.inv_freq; p.cq = cq; p.rows = rows_of(map); p.cache = cache_of(cache);
    p.proj_stride = proj_stride; p.q_at = q_at; p.kv_at = kv_at; p.rot_at = rope_at; p.cq_stride = cq_stride; p.q_count = q_count;
    p.rank_count = c.rank_count; p.rank = c.rank; p.rot_dim = c.rope_dim; p.rot_dims = c.rotary_dims; p.eps = c.eps;
    hipStream_t s = (hipStream_t)stream;
    const uint32_t pieces = (q_count + 7) / 8 + (c.rank_count + 7) / 8;
#define NVMAI_LE(NP)                                                                              \
    do {                                                                                          \
        if (ctx->act == NVMAI_ACT_BF16) latent_epilogue_kernel<ACT_BF16, ACT_BF16, NP><<<rows, 256, 0, s>>>(p); \
        else if (cache->type == NVMAI_ACT_BF16) latent_epilogue_kernel<ACT_FP32, ACT_BF16, NP><<<rows, 256, 0, s>>>(p); \
        else latent_epilogue_kernel<ACT_FP32, ACT_FP32, NP><<<rows, 256, 0, s>>>(p);              \
    } while (0)
    if (pieces <= 256) NVMAI_LE(1);
    else if (pieces <= 512) NVMAI_LE(2);
    else if (pieces <= 2048) NVMAI_LE(8);
    else return NVMAI_ERR_UNSUPPORTED;
#undef NVMAI_LE
    return launch_status();
}

extern "C" int nvmai_hip_latent_attention(nvmai_hip_ctx* ctx, nvmai_stream stream, const nvmai_latent_config* config, void* q,
                                          uint32_t q_stride, const void* gate, uint32_t gate_stride, const uint16_t* uk,
                                          const uint16_t* uv, const nvmai_latent_cache* cache, const nvmai_row_map* map, void* out,
                                          uint32_t out_stride, uint32_t rows, int form) {
    int rc = check_config(ctx, config, cache);
    if (rc) return rc;
    const nvmai_latent_config& c = *config;
    if (!q || !uk || !uv || !map || !out) return NVMAI_ERR_INVALID_ARG;
    if (q_stride < c.heads * (c.nope_dim + c.rope_dim) || out_stride < c.heads * c.value_dim || (gate && gate_stride < c.heads)) return NVMAI_ERR_INVALID_ARG;
    if (!aligned16(q) || q_stride % 8 || !aligned16(out) || out_stride % 4 || !aligned16(uk) || !aligned16(uv)) return NVMAI_ERR_ALIGNMENT;
    if (form < NVMAI_FORM_AUTO || form > NVMAI_LATENT_EXPANDED) return NVMAI_ERR_INVALID_ARG;
    if ((map->slots == nullptr) != (map->positions == nullptr)) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    if (rows > 65535) return NVMAI_ERR_UNSUPPORTED;
    const bool known = map->positions == nullptr;
    // every key a row may look at has to be in the ring while the call runs
    const uint32_t last = known ? map->position + rows : 0;
    if (known) {
        const uint64_t span = c.window ? (uint64_t)c.window + rows - 1 : (uint64_t)last;
        if ((span < last ? span : last) > cache->capacity) return NVMAI_ERR_INVALID_ARG;
    }
    LatentAttnParams p{};
    p.q = q; p.gate = gate; p.uk = uk; p.uv = uv; p.inv_freq = c.inv_freq; p.rows = rows_of(map); p.cache = cache_of(cache); p.out = out;
    p.q_stride = q_stride; p.gate_stride = gate_stride; p.out_stride = out_stride; p.n_rows = rows; p.heads = c.heads; p.nope = c.nope_dim;
    p.rot = c.rope_dim; p.vdim = c.value_dim; p.rank = c.rank; p.rot_dims = c.rotary_dims; p.window = c.window;
    p.scale_log2 = c.scale * LA_LOG2E;
    hipStream_t s = (hipStream_t)stream;
    const bool f32 = ctx->act == NVMAI_ACT_FP32, cache32 = cache->type == NVMAI_ACT_FP32;
    const size_t esz = cache32 ? 4 : 2;
    if (form == NVMAI_LATENT_EXPANDED && (!known || f32 != cache32)) return NVMAI_ERR_UNSUPPORTED;
    const bool expand = form == NVMAI_LATENT_EXPANDED || (form == NVMAI_FORM_AUTO && known && f32 == cache32 && rows >= 32);
    if (!expand) {
        uint32_t keys = known ? last : cache->capacity;
        if (c.window && c.window < keys) keys = c.window;
        // about two blocks per compute unit, at least 32 keys each
        const uint32_t groups = cache32 ? c.heads : (c.heads + 15) / 16;
        const uint32_t want = 2u * (uint32_t)ctx->compute_units / (rows * groups) + 1u;
        const uint32_t per = ((keys + want - 1) / want + 31) / 32 * 32;
        p.split_keys = per;
        p.splits = (keys + per - 1) / per;
        const size_t cells = (size_t)rows * c.heads * p.splits, n_qa = (size_t)rows * c.heads * cache->row_stride;
        rc = ws_begin(ctx, stream, ws_round(n_qa * esz) + ws_round(cells * c.rank * 4) + 2 * ws_round(cells * 4));
        if (rc) return rc;
        p.qa = ws_take<uint8_t>(ctx, n_qa * esz);
        p.part_o = ws_take<float>(ctx, cells * c.rank);
        p.part_m = ws_take<float>(ctx, cells);
        p.part_l = ws_take<float>(ctx, cells);
        if (!f32) return absorbed<ACT_BF16, ACT_BF16>(p, s);
        return cache32 ? absorbed<ACT_FP32, ACT_FP32>(p, s) : absorbed<ACT_FP32, ACT_BF16>(p, s);
    }
    p.key0 = c.window && map->position + 1 > c.window ? map->position + 1 - c.window : 0;
    p.nk = last - p.key0;
    p.nk_pad = (p.nk + 63) / 64 * 64;
    const uint32_t dq = c.nope_dim + c.rope_dim;
    bool flash = !f32 && c.nope_dim <= 256 && c.rope_dim <= 128 && c.value_dim <= 256;
    // rows an odd number of 128-byte lines apart: a tile's rows then spread over the memory channels
    auto odd_lines = [](uint32_t n) { return (n + 63) / 64 % 2 ? (n + 63) / 64 * 64 : ((n + 63) / 64 + 1) * 64; };
    const uint32_t nh = c.heads * c.nope_dim, vh = c.heads * c.value_dim;
    p.kn_stride = odd_lines(nh);
    // 31-bit byte offsets inside its operands
    const uint64_t widest = (uint64_t)p.nk_pad * (p.kn_stride > cache->row_stride ? p.kn_stride : cache->row_stride);
    flash = flash && widest * 2 < 0x7FFFFFFFull && (uint64_t)vh * (p.nk_pad + 64) * 2 < 0x7FFFFFFFull;
    p.v_stride = odd_lines(flash ? p.nk_pad : vh);
    const size_t n_lat = (size_t)p.nk_pad * cache->row_stride, n_kn = (size_t)p.nk_pad * p.kn_stride, n_v = (size_t)(flash ? vh : p.nk_pad) * p.v_stride;
    rc = ws_begin(ctx, stream, ws_round(n_lat * esz) + ws_round(n_kn * esz) + ws_round(n_v * esz));
    if (rc) return rc;
    p.lat = ws_take<uint8_t>(ctx, n_lat * esz);
    p.kn = ws_take<uint8_t>(ctx, n_kn * esz);
    p.v = ws_take<uint8_t>(ctx, n_v * esz);
    const DenseLinearParams lk{uk, p.lat, p.kn, nullptr, c.rank, cache->row_stride, p.kn_stride, p.nk_pad, nh, c.rank, NVMAI_LINEAR_NONE};
    const DenseLinearParams lv = flash ? DenseLinearParams{static_cast<const uint16_t*>(p.lat), uv, p.v, nullptr, cache->row_stride, c.rank, p.v_stride, vh, p.nk_pad, c.rank, NVMAI_LINEAR_NONE}
                                       : DenseLinearParams{uv, p.lat, p.v, nullptr, c.rank, cache->row_stride, p.v_stride, p.nk_pad, vh, c.rank, NVMAI_LINEAR_NONE};
    if ((rc = dense_linear_check(ctx, lk)) || (rc = dense_linear_check(ctx, lv))) return rc;
    const size_t lds_rot = (size_t)c.rotary_dims * 4;
    if (f32) {
        latent_gather_kernel<ACT_FP32><<<p.nk_pad, 256, 0, s>>>(p);
        if (c.rotary_dims) latent_rotate_q_kernel<ACT_FP32><<<rows, 256, lds_rot, s>>>(p);
    } else {
        latent_gather_kernel<ACT_BF16><<<p.nk_pad, 256, 0, s>>>(p);
        if (c.rotary_dims) latent_rotate_q_kernel<ACT_BF16><<<rows, 256, lds_rot, s>>>(p);
    }
    if ((rc = dense_linear(ctx, s, lk)) || (rc = dense_linear(ctx, s, lv))) return rc;
    if (!flash) {
        const size_t lds = ((size_t)dq + c.value_dim + 256 + 8) * 4;
        if (f32) {
            if ((rc = raise_lds(reinterpret_cast<const void*>(latent_expanded_plain_kernel<ACT_FP32>), lds))) return rc;
            latent_expanded_plain_kernel<ACT_FP32><<<dim3(c.heads, rows), 256, lds, s>>>(p);
        } else {
            if ((rc = raise_lds(reinterpret_cast<const void*>(latent_expanded_plain_kernel<ACT_BF16>), lds))) return rc;
            latent_expanded_plain_kernel<ACT_BF16><<<dim3(c.heads, rows), 256, lds, s>>>(p);
        }
        return launch_status();
    }
    if (c.nope_dim > 128 || c.rope_dim > 64 || c.value_dim > 128) return launch_flash<256, 128, 256>(p, s);
    if (c.nope_dim <= 64) return c.rope_dim <= 32 ? launch_flash_v<64, 32>(p, s) : launch_flash_v<64, 64>(p, s);
    return c.rope_dim <= 32 ? launch_flash_v<128, 32>(p, s) : launch_flash_v<128, 64>(p, s);
}
