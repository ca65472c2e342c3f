// bf16-weight instantiations of the GEMM kernel without the token gather.
#include "gemm_kernel.hpp"

namespace gptoss {
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, false, EPI_F32, false)
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, false, EPI_ARGMAX, false)
hipError_t gemm_set_attrs_bf16() {
  hipError_t err = hipSuccess;
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, false, EPI_F32, false)
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, false, EPI_ARGMAX, false)
  return err;
}
int gemm_col_tiles(int N) { return (N + BN - 1) / BN; }
}  // namespace gptoss
