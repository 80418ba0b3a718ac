// The dense product with the GELU of the error function between sum and store.
#include "ctx.hpp"
#include "dense_kernels.hpp"

namespace nvmai {
int dense_launch_erf(nvmai_hip_ctx* ctx, hipStream_t s, const DenseLinearParams& p) { return dense_launch<DE_ERF>(ctx, s, p); }
}  // namespace nvmai
