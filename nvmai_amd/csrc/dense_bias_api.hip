// The dense product with a bias between sum and store.
#include "ctx.hpp"
#include "dense_kernels.hpp"

namespace nvmai {
int dense_launch_bias(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) { return dense_launch<DE_BIAS>(ctx, s, p); }
}  // namespace nvmai
