// The 256-row GEMM kernel with the token gather and the SwiGLU epilogue: the experts' first GEMM.
#include "gemm_tall_kernel.hpp"

namespace gptoss {

int run_gemm_tall_gather(const GemmParams &p, int max_tiles, long long max_rows, hipStream_t s) {
  const int rc = check_gemm_tall(p, true, EPI_SWIGLU, max_rows);
  if (rc != GPTOSS_OK) return rc;
  return launch_tall<Tall256, true, EPI_SWIGLU>(p, max_tiles, s);
}

}  // namespace gptoss
