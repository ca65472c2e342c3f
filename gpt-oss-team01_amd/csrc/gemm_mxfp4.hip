// MXFP4-weight instantiations of the grouped GEMM kernel.
#include "gemm_kernel.hpp"

namespace gptoss {
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, true, EPI_SWIGLU, true)
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, false, EPI_F32, true)
hipError_t gemm_set_attrs_mxfp4() {
  hipError_t err = hipSuccess;
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, true, EPI_SWIGLU, true)
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, false, EPI_F32, true)
  return err;
}
}  // namespace gptoss
