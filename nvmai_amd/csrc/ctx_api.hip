// Entry points: the context every call takes, its workspace, per-kernel timing, status strings.
#include <atomic>
#include <new>

#include "ctx.hpp"

using namespace nvmai;

namespace {

// Scratch of the allocation-free decode entry point: one array per device, in the library's image,
// so that a caller which may not allocate (HIP graph capture, a serving loop, a harness that
// forbids hipMalloc) still has the step's intermediate buffers.  Host code never uses the
// array's name as an address: the device address comes from hipGetSymbolAddress, once per device.
static __device__ __align__(256) __attribute__((used)) uint8_t scratch[STATIC_SCRATCH_BYTES];
constexpr int STATIC_SCRATCH_MAX_DEVICES = 64;
// Device address of `scratch` on each device, nullptr = not asked yet.  Contexts may be created from several
// threads: the slots are atomics (every thread that fills one stores the same address, so no lock is needed).
std::atomic<uint8_t*> g_static_scratch[STATIC_SCRATCH_MAX_DEVICES];

// The device address of this device's copy of the array (the device must be current).
int static_scratch_ptr(int device, uint8_t** out) {
    if (device < 0 || device >= STATIC_SCRATCH_MAX_DEVICES) return NVMAI_ERR_INVALID_ARG;
    uint8_t* known = g_static_scratch[device].load(std::memory_order_acquire);
    if (!known) {
        void* ptr = nullptr;
        if (hipGetSymbolAddress(&ptr, HIP_SYMBOL(scratch)) != hipSuccess || !ptr) {
            (void)hipGetLastError();
            return NVMAI_ERR_HIP;
        }
        known = static_cast<uint8_t*>(ptr);
        g_static_scratch[device].store(known, std::memory_order_release);
    }
    *out = known;
    return NVMAI_OK;
}

}  // namespace

extern "C" int nvmai_hip_ctx_create(int device, int act_dtype, nvmai_hip_ctx** out) {
    if (!out || (act_dtype != NVMAI_ACT_BF16 && act_dtype != NVMAI_ACT_FP16 && act_dtype != NVMAI_ACT_FP32)) return NVMAI_ERR_INVALID_ARG;
    int count = 0;
    if (hipGetDeviceCount(&count) != hipSuccess || count <= 0) return NVMAI_ERR_NO_DEVICE;
    if (device < 0 || device >= count) return NVMAI_ERR_INVALID_ARG;
    NVMAI_HIP_TRY(hipSetDevice(device));
    nvmai_hip_ctx* ctx = new (std::nothrow) nvmai_hip_ctx();
    if (!ctx) return NVMAI_ERR_HIP;
    ctx->device = device;
    ctx->compute_units = 256;
    {
        int cus = 0;
        if (hipDeviceGetAttribute(&cus, hipDeviceAttributeMultiprocessorCount, device) == hipSuccess && cus > 0)
            ctx->compute_units = cus;
    }
    ctx->act = act_dtype;
    ctx->ws = nullptr;
    ctx->ws_cap = 0;
    ctx->ws_used = 0;
    ctx->prof_on = false;
    ctx->tickets = nullptr;
    if (hipMalloc(reinterpret_cast<void**>(&ctx->tickets), TICKET_WORDS * 4) != hipSuccess ||
        hipMemset(ctx->tickets, 0, TICKET_WORDS * 4) != hipSuccess) {
        delete ctx;
        return NVMAI_ERR_HIP;
    }
    // device address of this device's static scratch array (nullptr if the lookup fails: only the
    // allocation-free entry point needs it, and it then reports the failure)
    ctx->static_scratch = nullptr;
    (void)static_scratch_ptr(device, &ctx->static_scratch);
    *out = ctx;
    return NVMAI_OK;
}

extern "C" void nvmai_hip_ctx_destroy(nvmai_hip_ctx* ctx) {
    if (!ctx) return;
    if (ctx->ws) (void)hipFree(ctx->ws);
    for (void* block : ctx->ws_retired) (void)hipFree(block);
    if (ctx->tickets) (void)hipFree(ctx->tickets);
    for (auto& sp : ctx->prof_spans) { (void)hipEventDestroy(sp.start); (void)hipEventDestroy(sp.stop); }
    for (auto& e : ctx->prof_free) (void)hipEventDestroy(e);
    delete ctx;
}

extern "C" int nvmai_hip_ctx_reserve(nvmai_hip_ctx* ctx, size_t bytes) {
    if (!ctx) return NVMAI_ERR_INVALID_ARG;
    NVMAI_HIP_TRY(hipSetDevice(ctx->device));
    return ws_begin(ctx, nullptr, bytes);
}

extern "C" size_t nvmai_hip_ctx_workspace_bytes(const nvmai_hip_ctx* ctx) { return ctx ? ctx->ws_cap : 0; }

extern "C" int nvmai_hip_profile_enable(nvmai_hip_ctx* ctx, int on) {
    if (!ctx) return NVMAI_ERR_INVALID_ARG;
    if (on) {
        for (auto& sp : ctx->prof_spans) {
            NVMAI_HIP_TRY(hipEventSynchronize(sp.stop));
            ctx->prof_free.push_back(sp.start);
            ctx->prof_free.push_back(sp.stop);
        }
        ctx->prof_spans.clear();
    }
    ctx->prof_on = on != 0;
    return NVMAI_OK;
}

extern "C" int nvmai_hip_profile_read(nvmai_hip_ctx* ctx, int tag, double* total_ms, uint32_t* launches) {
    if (!ctx || !total_ms || !launches) return NVMAI_ERR_INVALID_ARG;
    double total = 0.0;
    uint32_t n = 0;
    for (auto& sp : ctx->prof_spans) {
        if (sp.tag != tag) continue;
        NVMAI_HIP_TRY(hipEventSynchronize(sp.stop));
        float ms = 0.0f;
        NVMAI_HIP_TRY(hipEventElapsedTime(&ms, sp.start, sp.stop));
        total += ms;
        ++n;
    }
    *total_ms = total;
    *launches = n;
    return NVMAI_OK;
}

extern "C" const char* nvmai_hip_status_string(int status) {
    switch (status) {
        case NVMAI_OK: return "ok";
        case NVMAI_ERR_INVALID_ARG: return "invalid argument";
        case NVMAI_ERR_UNSUPPORTED: return "unsupported configuration";
        case NVMAI_ERR_ALIGNMENT: return "pointer or stride not 16-byte aligned";
        case NVMAI_ERR_SCRATCH: return "scratch too small";
        case NVMAI_ERR_HIP: return "HIP runtime error";
        case NVMAI_ERR_NO_DEVICE: return "no HIP device";
        default: return "unknown status";
    }
}
