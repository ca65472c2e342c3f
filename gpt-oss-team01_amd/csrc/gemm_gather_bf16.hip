// bf16-weight instantiations of the GEMM kernel with the token gather and the SwiGLU epilogue.
#include "gemm_kernel.hpp"

namespace gptoss {
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, true, EPI_SWIGLU, false)
hipError_t gemm_set_attrs_gather_bf16() {
  hipError_t err = hipSuccess;
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, true, EPI_SWIGLU, false)
  return err;
}
}  // namespace gptoss
