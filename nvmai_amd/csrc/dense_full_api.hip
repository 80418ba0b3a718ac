// The dense product with bias, activation and a multiplier per token between sum and store.
#include "ctx.hpp"
#include "dense_kernels.hpp"

namespace nvmai {
int dense_launch_full(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) { return dense_launch<DE_FULL>(ctx, s, p); }
}  // namespace nvmai
