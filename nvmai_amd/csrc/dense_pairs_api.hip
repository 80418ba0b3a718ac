// The dense product with silu(gate) * up from rows in turn between sum and store.
#include "ctx.hpp"
#include "dense_kernels.hpp"

namespace nvmai {
int dense_launch_pairs(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) { return dense_launch<DE_PAIRS>(ctx, s, p); }
}  // namespace nvmai
