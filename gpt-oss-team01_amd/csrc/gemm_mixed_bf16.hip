// bf16-weight instantiations of the dense GEMM with bf16 column ranges and with partial sums over K.
#include "gemm_kernel.hpp"

namespace gptoss {
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, false, EPI_MIXED, false)
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, false, EPI_PARTIAL, false)
hipError_t gemm_set_attrs_mixed_bf16() {
  hipError_t err = hipSuccess;
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, false, EPI_MIXED, false)
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, false, EPI_PARTIAL, false)
  return err;
}
}  // namespace gptoss
