// The 256-row GEMM kernel without the token gather: the dense GEMMs and the down projections of experts.
#include "gemm_tall_kernel.hpp"

namespace gptoss {

bool gemm_tall_applies(const GemmParams &p, bool gather, int epi) {
  const bool kind = (gather && epi == EPI_SWIGLU) || (!gather && (epi == EPI_F32 || epi == EPI_MIXED)) ||
                    (!gather && epi == EPI_ARGMAX && p.tiles == nullptr && p.amax_val && p.amax_idx);
  // whole A chunks of 64 k, and at least 8 stages: an item's first loads are requested during the
  // last four stages of the item before it
  static_assert(2 * TALL_BK == 64, "gemm_tall_shape_ok states the chunk size");
  return kind && !p.w_mxfp4 && gemm_tall_shape_ok(p.N, p.K, 0);
}

int check_gemm_tall(const GemmParams &p, bool gather, int epi, long long max_rows) {
  GPTOSS_REQUIRE(gemm_tall_applies(p, gather, epi), GPTOSS_ERR_DIM,
                 "run_gemm: 256-row tiles need bf16 weights, K %% 64 == 0, K >= 256, N %% 32 == 0 and the "
                 "gather+SwiGLU, plain fp32 or dense arg-max form (gather=%d epi=%d N=%d K=%d)", (int)gather, epi, p.N, p.K);
  // a row of A is addressed by a 32-bit byte offset
  GPTOSS_REQUIRE(max_rows * p.K * 2 < (1ll << 32), GPTOSS_ERR_DIM,
                 "run_gemm: 256-row tiles need rows x K below 2^31 elements (rows<=%lld K=%d)", max_rows, p.K);
  return GPTOSS_OK;
}

int run_gemm_tall(const GemmParams &p, int epi, int max_tiles, long long max_rows, hipStream_t s) {
  const int rc = check_gemm_tall(p, false, epi, max_rows);
  if (rc != GPTOSS_OK) return rc;
  static_assert(Tall256::WC == 2, "dense_gemm reports two arg-max pairs per row and column tile");
  if (epi == EPI_ARGMAX) return launch_tall<Tall256, false, EPI_ARGMAX>(p, max_tiles, s);
  if (epi == EPI_MIXED) return launch_tall<Tall256, false, EPI_MIXED>(p, max_tiles, s);
  return launch_tall<Tall256, false, EPI_F32>(p, max_tiles, s);
}

}  // namespace gptoss
