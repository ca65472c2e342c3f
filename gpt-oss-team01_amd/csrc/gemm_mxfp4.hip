// MXFP4-weight instantiations of the grouped GEMM kernel, and their dispatch.
#include <mutex>

#include "gemm_kernel.hpp"

namespace gptoss {
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, true, EPI_SWIGLU, true)
GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_INSTANTIATE, false, EPI_F32, true)

static hipError_t set_attrs() {
  hipError_t err = hipSuccess;
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, true, EPI_SWIGLU, true)
  GPTOSS_GEMM_EACH_TILE(GPTOSS_GEMM_SET_ATTR, false, EPI_F32, true)
  return err;
}

template <bool GATHER, int EPI>
static int dispatch_rows(const GemmParams &p, int rows_per_tile, int max_tiles, hipStream_t s) {
  switch (rows_per_tile) {
    case 32: return launch_gemm<1, GATHER, EPI, true>(p, max_tiles, s);
    case 64: return launch_gemm<2, GATHER, EPI, true>(p, max_tiles, s);
    case 96: return launch_gemm<3, GATHER, EPI, true>(p, max_tiles, s);
    case 128: return launch_gemm<4, GATHER, EPI, true>(p, max_tiles, s);
    case 160: return launch_gemm<5, GATHER, EPI, true>(p, max_tiles, s);
  }
  return fail(GPTOSS_ERR_DIM, "run_gemm: unsupported rows_per_tile %d", rows_per_tile);
}

static int dispatch(const GemmParams &p, bool gather, int epi, int rows_per_tile, int max_tiles, hipStream_t s) {
  constexpr int MAX_DEV = 64;
  static std::mutex mu;
  static bool done[MAX_DEV];
  int dev = 0;
  GPTOSS_HIP(hipGetDevice(&dev));
  GPTOSS_REQUIRE(dev >= 0 && dev < MAX_DEV, GPTOSS_ERR_STATE, "run_gemm: device ordinal %d outside 0..%d", dev, MAX_DEV - 1);
  {
    std::lock_guard<std::mutex> lock(mu);
    if (!done[dev]) GPTOSS_HIP(set_attrs());
    done[dev] = true;
  }
  if (gather && epi == EPI_SWIGLU) return dispatch_rows<true, EPI_SWIGLU>(p, rows_per_tile, max_tiles, s);
  if (!gather && epi == EPI_F32) return dispatch_rows<false, EPI_F32>(p, rows_per_tile, max_tiles, s);
  return fail(GPTOSS_ERR_DIM, "run_gemm: unsupported combination (gather=%d epi=%d)", (int)gather, epi);
}

// a library of model classes without MXFP4 experts is linked without this file
static const bool registered = [] {
  run_gemm_mxfp4 = dispatch;
  return true;
}();
}  // namespace gptoss
