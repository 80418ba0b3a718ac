// Entry points of windowed grouped-query attention.
#include "ctx.hpp"
#include "window_kernels.hpp"

using namespace nvmai;

namespace {

int check_config(const nvmai_hip_ctx* ctx, const nvmai_window_config* c, const nvmai_kv_ring* cache) {
    if (!ctx || !c || !cache || !cache->k || !cache->v) return NVMAI_ERR_INVALID_ARG;
    if (ctx->act != NVMAI_ACT_BF16 && ctx->act != NVMAI_ACT_FP32) return NVMAI_ERR_UNSUPPORTED;
    if (c->heads == 0 || cache->kv_heads == 0 || c->heads % cache->kv_heads || cache->key_dim == 0 || cache->value_dim == 0) return NVMAI_ERR_INVALID_ARG;
    if (cache->key_dim % 32 || cache->value_dim % 16 || c->key_count == 0 || c->key_count > cache->key_dim) return NVMAI_ERR_INVALID_ARG;
    if (cache->key_dim > 512 || cache->value_dim > 512) return NVMAI_ERR_UNSUPPORTED;
    if (cache->ring == 0 || cache->ring % 64 || cache->pinned % 64 || c->keep_first > cache->pinned) return NVMAI_ERR_INVALID_ARG;
    if (cache->type != ctx->act && !(ctx->act == NVMAI_ACT_FP32 && cache->type == NVMAI_ACT_BF16)) return NVMAI_ERR_UNSUPPORTED;
    if (!aligned16(cache->k) || !aligned16(cache->v)) return NVMAI_ERR_ALIGNMENT;
    return NVMAI_OK;
}

int check_map(const nvmai_row_map* map, const nvmai_kv_ring* cache, uint32_t window, uint32_t rows) {
    if (!map || (map->slots == nullptr) != (map->positions == nullptr)) return NVMAI_ERR_INVALID_ARG;
    if (map->positions) return NVMAI_OK;
    // every position the rows look at is in the ring while the call runs
    const uint64_t last = (uint64_t)map->position + rows, span = window ? (uint64_t)window + rows - 1 : last;
    if (last > 0xFFFFFF00ull || (span < last ? span : last) > cache->ring) return NVMAI_ERR_INVALID_ARG;
    return NVMAI_OK;
}

KvRing ring_of(const nvmai_kv_ring* c) { return KvRing{c->k, c->v, c->kv_heads, c->key_dim, c->value_dim, c->pinned, c->ring}; }
SeqRows rows_of(const nvmai_row_map* m) { return SeqRows{m->slots, m->positions, m->slot, m->position}; }

int raise_lds(const void* kernel, size_t bytes) {
    if (bytes > 160 * 1024) return NVMAI_ERR_UNSUPPORTED;
    if (bytes > 64 * 1024) NVMAI_HIP_TRY(hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
    return NVMAI_OK;
}

template <int CT>
void epilogue(const WindowEpilogueParams& p, hipStream_t s) {
    const uint32_t G = p.cache.kv_heads, units = p.heads + (p.k_norm ? (p.values ? 2 * G : G) : 0);
    const dim3 grid(p.n_rows, (units + 3) / 4);
    if (p.cache.dk <= 64) window_epilogue_kernel<CT, 1><<<grid, 256, 0, s>>>(p);
    else if (p.cache.dk <= 128) window_epilogue_kernel<CT, 2><<<grid, 256, 0, s>>>(p);
    else window_epilogue_kernel<CT, 8><<<grid, 256, 0, s>>>(p);
    if (p.k_norm && !p.values) {
        const uint32_t tiles = (p.rows.position + p.n_rows - 1) / 64 - p.rows.position / 64 + 1;
        window_values_kernel<CT><<<dim3(tiles, G, (p.cache.dv + 63) / 64), 256, 0, s>>>(p);
    }
}

template <int DK, int DV, bool BOUND>
int launch_flash_as(const WindowParams& p, hipStream_t s) {
    const size_t lds = 2 * ((size_t)64 * DK * 2 + (size_t)DV * 128);
    const int rc = raise_lds(reinterpret_cast<const void*>(window_flash_kernel<DK, DV, BOUND>), lds);
    if (rc) return rc;
    window_flash_kernel<DK, DV, BOUND><<<(p.n_rows + 127) / 128 * p.heads, 256, lds, s>>>(p);
    return launch_status();
}

template <int DK, int DV>
int launch_flash(const WindowParams& p, hipStream_t s) {
    return p.capped && !p.alibi && p.b <= WA_BOUND ? launch_flash_as<DK, DV, true>(p, s) : launch_flash_as<DK, DV, false>(p, s);
}

template <int ACT, int CT>
int plain(const WindowParams& p, hipStream_t s) {
    const size_t lds = ((size_t)p.cache.dk + p.cache.dv + 256 + 8) * 4;
    window_plain_kernel<ACT, CT><<<dim3(p.heads, p.n_rows), 256, lds, s>>>(p);
    return launch_status();
}

}  // namespace

extern "C" int nvmai_hip_window_epilogue(nvmai_hip_ctx* ctx, nvmai_stream stream, const nvmai_window_config* config, const float* proj,
                                         uint32_t proj_stride, uint32_t q_at, uint32_t k_at, uint32_t v_at, const uint16_t* q_norm,
                                         const uint16_t* k_norm, void* q, uint32_t q_stride, const nvmai_kv_ring* cache,
                                         const nvmai_row_map* map, uint32_t rows) {
    int rc = check_config(ctx, config, cache);
    if (rc) return rc;
    if (!proj || !q_norm || !q || q_stride < config->heads * cache->key_dim || proj_stride < q_at + config->heads * cache->key_dim) return NVMAI_ERR_INVALID_ARG;
    if (k_norm && (proj_stride < k_at + cache->kv_heads * cache->key_dim || proj_stride < v_at + cache->kv_heads * cache->value_dim)) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    if ((rc = check_map(map, cache, config->window, rows))) return rc;
    WindowEpilogueParams p{};
    p.proj = proj; p.q_norm = q_norm; p.k_norm = k_norm; p.q = q; p.cache = ring_of(cache); p.rows = rows_of(map);
    p.proj_stride = proj_stride; p.q_at = q_at; p.k_at = k_at; p.v_at = v_at; p.q_stride = q_stride; p.n_rows = rows;
    p.heads = config->heads; p.key_count = config->key_count; p.values = map->positions != nullptr || rows < 16; p.eps = config->eps;
    if (cache->type == NVMAI_ACT_BF16) epilogue<ACT_BF16>(p, (hipStream_t)stream);
    else epilogue<ACT_FP32>(p, (hipStream_t)stream);
    return launch_status();
}

extern "C" int nvmai_hip_window_attention(nvmai_hip_ctx* ctx, nvmai_stream stream, const nvmai_window_config* config, const void* q,
                                          uint32_t q_stride, const float* gate, uint32_t gate_stride, const nvmai_kv_ring* cache,
                                          const nvmai_row_map* map, uint32_t max_position, float out_scale, void* out,
                                          uint32_t out_stride, uint32_t rows, int form) {
    int rc = check_config(ctx, config, cache);
    if (rc) return rc;
    const nvmai_window_config& c = *config;
    const uint32_t dk = cache->key_dim, dv = cache->value_dim;
    if (!q || !out || q_stride < c.heads * dk || out_stride < c.heads * dv || (gate && gate_stride < c.heads)) return NVMAI_ERR_INVALID_ARG;
    if (form < NVMAI_FORM_AUTO || form > NVMAI_WINDOW_PLAIN) return NVMAI_ERR_INVALID_ARG;
    if (rows == 0) return NVMAI_OK;
    if (rows > 65535) return NVMAI_ERR_UNSUPPORTED;
    if ((rc = check_map(map, cache, c.window, rows))) return rc;
    const bool known = map->positions == nullptr, f32 = ctx->act == NVMAI_ACT_FP32, cache32 = cache->type == NVMAI_ACT_FP32;
    WindowParams p{};
    p.q = q; p.gate = gate; p.out = out; p.cache = ring_of(cache); p.rows = rows_of(map); p.q_stride = q_stride; p.gate_stride = gate_stride;
    p.out_stride = out_stride; p.n_rows = rows; p.heads = c.heads; p.window = c.window; p.keep = c.keep_first; p.out_scale = out_scale;
    p.capped = c.softcap > 0.0f; p.alibi = c.alibi != 0;
    p.a = p.capped ? c.scale / c.softcap : c.scale * WA_LOG2E;
    p.b = c.softcap * WA_LOG2E;
    hipStream_t s = (hipStream_t)stream;
    const bool can16 = !cache32 && dk <= 256 && dv <= 256 && aligned16(q) && q_stride % 8 == 0;
    // 31-bit byte offsets inside its operands, 16-bit outputs four at a time
    const uint64_t total = (uint64_t)cache->pinned + cache->ring;
    const bool can_flash = can16 && known && !f32 && total * (dk > dv ? dk : dv) * 2 < 0x7FFFFFFFull && out_stride % 4 == 0 && (reinterpret_cast<uintptr_t>(out) & 7u) == 0;
    if ((form == NVMAI_WINDOW_SPLIT && !can16) || (form == NVMAI_WINDOW_FLASH && !can_flash)) return NVMAI_ERR_UNSUPPORTED;
    if (form == NVMAI_FORM_AUTO) form = can_flash && rows >= 32 ? NVMAI_WINDOW_FLASH : can16 ? NVMAI_WINDOW_SPLIT : NVMAI_WINDOW_PLAIN;
    if (form == NVMAI_WINDOW_PLAIN) {
        if (cache32) return plain<ACT_FP32, ACT_FP32>(p, s);
        return f32 ? plain<ACT_FP32, ACT_BF16>(p, s) : plain<ACT_BF16, ACT_BF16>(p, s);
    }
    if (form == NVMAI_WINDOW_FLASH) {
        if (dk > 128 || dv > 128) return launch_flash<256, 256>(p, s);
        if (dk <= 64) return dv <= 64 ? launch_flash<64, 64>(p, s) : launch_flash<64, 128>(p, s);
        return dv <= 64 ? launch_flash<128, 64>(p, s) : launch_flash<128, 128>(p, s);
    }
    // tiles of 32 positions that a row can look at
    const uint32_t last = known ? map->position + rows - 1 : max_position;
    const uint32_t kept = (c.keep_first + 31) / 32;
    uint32_t tiles = last / 32 + 1;
    if (c.window && (c.window + 30) / 32 + 1 + kept < tiles) tiles = (c.window + 30) / 32 + 1 + kept;
    // about two blocks per compute unit, a tile per wave at least
    const uint32_t groups = cache->kv_heads * ((c.heads / cache->kv_heads + 15) / 16);
    const uint32_t want = 2u * (uint32_t)ctx->compute_units / (rows * groups) + 1u;
    uint32_t per = (tiles + want - 1) / want;
    per = per < 4 ? 4 : per;
    p.tiles_per_split = per;
    p.splits = (tiles + per - 1) / per;
    const size_t cells = (size_t)rows * c.heads * p.splits;
    rc = ws_begin(ctx, stream, ws_round(cells * dv * 4) + 2 * ws_round(cells * 4));
    if (rc) return rc;
    p.part_o = ws_take<float>(ctx, cells * dv);
    p.part_m = ws_take<float>(ctx, cells);
    p.part_l = ws_take<float>(ctx, cells);
    const dim3 grid(p.splits, groups, rows);
    if (dk <= 64 && dv <= 64) window_split_kernel<64, 64><<<grid, 256, 0, s>>>(p);
    else if (dk <= 128 && dv <= 128) window_split_kernel<128, 128><<<grid, 256, 0, s>>>(p);
    else window_split_kernel<256, 256><<<grid, 256, 0, s>>>(p);
    const size_t lds = ((size_t)(p.splits + 3) / 4 * 4 + 256 * 4) * 4;
    if (lds > 64 * 1024) return NVMAI_ERR_UNSUPPORTED;
    if (f32) window_combine_kernel<ACT_FP32><<<dim3(c.heads, rows), 256, lds, s>>>(p);
    else window_combine_kernel<ACT_BF16><<<dim3(c.heads, rows), 256, lds, s>>>(p);
    return launch_status();
}
