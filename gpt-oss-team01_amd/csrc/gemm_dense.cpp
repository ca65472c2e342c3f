// Host side of the dense bf16 GEMMs (kernel dispatch) and the weight repacking kernel.  The GEMM kernels
// themselves are in gemm_kernel.hpp and gemm_tall_kernel.hpp.
#include <stdlib.h>

#include <mutex>

#include "common.hpp"
#include "gemm.hpp"

namespace gptoss {

// Repack row-major [n_out, n_in] matrices into fragment order:
//   dst[((nb*KS + ks)*64 + lane)*8 + j] = W[row(nb*32 + lane%32)][ks*16 + (lane/32)*8 + j]
// With GLU pairing, virtual row v of a 32-row block maps to pair (v/32)*16 + v%16, gate for the
// first 16 virtual rows and up for the second 16.
template <typename SRC>
__global__ __launch_bounds__(256) void pack_weight_kernel(const SRC *__restrict__ src,
                                                          bf16_t *__restrict__ dst, int n_out,
                                                          int n_in, int glu) {
  const int ksteps = n_in / 16;
  const size_t frags_per_mat = (size_t)(n_out / 32) * ksteps;
  const size_t gid = (size_t)blockIdx.x * 256 + threadIdx.x;  // one (fragment, lane) per thread
  const size_t frag = gid >> 6;
  const int lane = (int)(gid & 63);
  const int mat = blockIdx.y;
  if (frag >= frags_per_mat) return;
  const int nb = (int)(frag / ksteps), ks = (int)(frag - (size_t)nb * ksteps);
  int v = nb * 32 + (lane & 31);
  int row = v;
  if (glu) row = 2 * ((v >> 5) * 16 + (v & 15)) + ((v >> 4) & 1);
  const SRC *sp = src + ((size_t)mat * n_out + row) * n_in + ks * 16 + (lane >> 5) * 8;
  uint32_t o[4];
#pragma unroll
  for (int j = 0; j < 4; j++) {
    if constexpr (sizeof(SRC) == 4) {
      o[j] = pack_bf16x2((float)sp[2 * j], (float)sp[2 * j + 1]);
    } else {
      o[j] = (uint32_t)sp[2 * j] | ((uint32_t)sp[2 * j + 1] << 16);
    }
  }
  u32x4 *dp = reinterpret_cast<u32x4 *>(dst + ((size_t)mat * frags_per_mat + frag) * 512 + lane * 8);
  *dp = u32x4{o[0], o[1], o[2], o[3]};
}

// Host-side dispatcher of the form without gather.  rows_per_tile selects the kernel.
template <int MBMAX, bool GATHER, int EPI, bool FP4>
int launch_gemm(const GemmParams &p, int max_tiles, hipStream_t s);  // gemm_bf16.hip, gemm_mixed_bf16.hip

template <int EPI>
static int dispatch_rows(const GemmParams &p, int rows_per_tile, int max_tiles, hipStream_t s) {
  switch (rows_per_tile) {
    case 32: return launch_gemm<1, false, EPI, false>(p, max_tiles, s);
    case 64: return launch_gemm<2, false, EPI, false>(p, max_tiles, s);
    case 96: return launch_gemm<3, false, EPI, false>(p, max_tiles, s);
    case 128: return launch_gemm<4, false, EPI, false>(p, max_tiles, s);
    case 160: return launch_gemm<5, false, EPI, false>(p, max_tiles, s);
  }
  return fail(GPTOSS_ERR_DIM, "run_gemm: unsupported rows_per_tile %d", rows_per_tile);
}

hipError_t gemm_set_attrs_bf16();        // gemm_bf16.hip
hipError_t gemm_set_attrs_mixed_bf16();  // gemm_mixed_bf16.hip

// Raises the dynamic-LDS limit of every such kernel on the calling thread's current device, the
// first time that device launches one.
static int gemm_prepare_device() {
  constexpr int MAX_DEV = 64;
  static std::mutex mu;
  static bool done[MAX_DEV];
  int dev = 0;
  GPTOSS_HIP(hipGetDevice(&dev));
  GPTOSS_REQUIRE(dev >= 0 && dev < MAX_DEV, GPTOSS_ERR_STATE, "run_gemm: device ordinal %d outside 0..%d", dev, MAX_DEV - 1);
  std::lock_guard<std::mutex> lock(mu);
  if (!done[dev]) {
    GPTOSS_HIP(gemm_set_attrs_bf16());
    GPTOSS_HIP(gemm_set_attrs_mixed_bf16());
    done[dev] = true;
  }
  return GPTOSS_OK;
}

int run_gemm_dense(const GemmParams &p, int epi, int rows_per_tile, int max_tiles, hipStream_t s) {
  // output and operand offsets inside the kernels are 32-bit element counts
  const long long max_rows = p.tiles ? (long long)max_tiles * rows_per_tile : p.dense_rows;
  GPTOSS_REQUIRE(max_rows * p.N < (1ll << 32) && max_rows * p.K < (1ll << 32), GPTOSS_ERR_DIM,
                 "run_gemm: rows x columns must stay below 2^32 elements (rows<=%lld N=%d K=%d)", max_rows, p.N, p.K);
  if (rows_per_tile == 256) return run_gemm_tall(p, epi, max_tiles, max_rows, s);
  int prc = gemm_prepare_device();
  if (prc != GPTOSS_OK) return prc;
  if (epi == EPI_F32) return dispatch_rows<EPI_F32>(p, rows_per_tile, max_tiles, s);
  if (epi == EPI_MIXED && p.tiles == nullptr) return dispatch_rows<EPI_MIXED>(p, rows_per_tile, max_tiles, s);
  if (epi == EPI_PARTIAL && p.tiles == nullptr) return dispatch_rows<EPI_PARTIAL>(p, rows_per_tile, max_tiles, s);
  if (epi == EPI_ARGMAX && p.tiles == nullptr && p.amax_val && p.amax_idx)
    return dispatch_rows<EPI_ARGMAX>(p, rows_per_tile, max_tiles, s);
  return fail(GPTOSS_ERR_DIM, "run_gemm: unsupported combination (dense, epi=%d)", epi);
}

// rows from which a dense fp32-output GEMM uses the 256-row kernel of gemm_tall.hip
static int dense_tall_min_rows() {
  static const int v = [] {
    const char *e = getenv("GPTOSS_DENSE_TALL_MIN_ROWS");
    const int n = e ? atoi(e) : 0;
    return n > 0 ? n : 2048;
  }();
  return v;
}

// rows from which the classifier's arg-max GEMM uses it (measured, vocabulary 201088 x 2880: 256 rows
// 360 -> 295 us, 512 rows 716 -> 556, 1024 rows 1194 -> 986-1007, 2048 rows 2319 -> 1859)
static int argmax_tall_min_rows() {
  static const int v = [] {
    const char *e = getenv("GPTOSS_ARGMAX_TALL_MIN_ROWS");
    const int n = e ? atoi(e) : 0;
    return n > 0 ? n : 256;
  }();
  return v;
}

// Row tile of a dense GEMM on the streaming kernels.  Up to 96 rows: the smallest size that holds every
// row, so the weights are requested once.  A prompt pass (thousands of rows): 160 rows, every weight
// fragment feeds five MFMAs.  In between the launch is a handful of rounds of work items on 256 CUs, and
// an item of MB 32-row blocks takes (0.39 + 0.115 MB) us per 64-k slab (measured at 1024 rows: 0.50 /
// 0.64 / 0.76 / 0.85 us for 32 / 64 / 96 / 128 rows), so the tile that needs the least rounds x slab time
// wins: 96 rows for the QKV projection of 1024 rows (220 items, one round), 64 for the output
// projection (192 items instead of 132: 48 -> 41 us).
static double slab_us(int mb) { return 0.39 + 0.115 * mb; }

static int dense_rows_per_tile(int B, int n_col_tiles) {
  if (B <= 96) return align_up(B, 32);
  if (B < 2048 && n_col_tiles >= 64) return 128;  // the unembedding: hundreds of column tiles, measured best at 1024 rows
  if (B >= 2048) return 160;
  double best = 0.0;
  int rpt = 160;
  for (int mb = 1; mb <= 5; mb++) {
    const long long items = (long long)cdiv(B, 32 * mb) * n_col_tiles;
    const double cost = (double)((items + 255) / 256) * slab_us(mb);
    if (mb == 1 || cost <= best) {  // ties go to the larger tile: fewer re-reads of the weights
      best = cost;
      rpt = 32 * mb;
    }
  }
  return rpt;
}

static GemmParams dense_params(const bf16_t *A, const bf16_t *W, const float *bias, void *out, int B, int N, int K) {
  GemmParams g{};
  g.A = A;
  g.W = W;
  g.bias = bias;
  g.out = out;
  g.tiles = nullptr;
  g.dense_rows = B;
  g.N = N;
  g.K = K;
  g.n_col_tiles = gemm_col_tiles(N);
  return g;
}

// C[B, N] = A[B, K] . W[N, K]^T (+ bias): the dense GEMMs of a step (QKV and output projections,
// classifier), with the kernel and row tile chosen from the batch size.
int dense_gemm(const bf16_t *A, const bf16_t *W, const float *bias, void *out, int epi, int B, int N,
               int K, hipStream_t s, float *amax_val, int *amax_idx, int *amax_tiles) {
  GemmParams g = dense_params(A, W, bias, out, B, N, K);
  g.amax_val = amax_val;
  g.amax_idx = amax_idx;
  int rpt = dense_rows_per_tile(B, g.n_col_tiles);
  if (B >= (epi == EPI_ARGMAX ? argmax_tall_min_rows() : dense_tall_min_rows()) && gemm_tall_applies(g, false, epi) &&
      gemm_tall_shape_ok(N, K, B))
    rpt = 256;
  if (epi == EPI_ARGMAX) {
    GPTOSS_REQUIRE(amax_tiles, GPTOSS_ERR_NULL, "dense_gemm: the arg-max form reports its pairs per row");
    *amax_tiles = rpt == 256 ? 2 * g.n_col_tiles : g.n_col_tiles;
  }
  return run_gemm_dense(g, epi, rpt, cdiv(B, rpt), s);
}

int dense_gemm_mixed(const bf16_t *A, const bf16_t *W, float *out, const GemmBf16Range *ranges, int n_ranges, int B,
                     int N, int K, hipStream_t s) {
  GPTOSS_REQUIRE(n_ranges >= 0 && n_ranges <= 2, GPTOSS_ERR_DIM, "dense_gemm_mixed: %d ranges", n_ranges);
  GemmParams g = dense_params(A, W, nullptr, out, B, N, K);
  for (int i = 0; i < n_ranges; i++) {
    g.range[i] = ranges[i];
    GPTOSS_REQUIRE(ranges[i].from % 32 == 0 && ranges[i].to % 32 == 0 && ranges[i].ld % 4 == 0 && aligned(ranges[i].out, 8),
                   GPTOSS_ERR_DIM, "dense_gemm_mixed: ranges are whole 32-column blocks of aligned rows");
  }
  int rpt = dense_rows_per_tile(B, g.n_col_tiles);
  if (B >= dense_tall_min_rows() && gemm_tall_applies(g, false, EPI_MIXED) && gemm_tall_shape_ok(N, K, B)) rpt = 256;
  return run_gemm_dense(g, EPI_MIXED, rpt, cdiv(B, rpt), s);
}

// Few rows and few columns leave most CUs without a work item while those that have one walk all of K.
// Cutting K makes more items; what it costs is a fixed part per item and the partial sums' way to memory
// and back.
int dense_gemm_partial(const bf16_t *A, const bf16_t *W, float *out, size_t max_elems, int *parts, int B, int N, int K,
                       hipStream_t s) {
  *parts = 1;
  GemmParams g = dense_params(A, W, nullptr, out, B, N, K);
  if (B >= dense_tall_min_rows()) return dense_gemm(A, W, nullptr, out, EPI_F32, B, N, K, s);
  const int nslab = K / 64;
  double best = 0.0;
  int rpt = 32, splits = 1, slabs = nslab;
  for (int mb = 1; mb <= 5; mb++) {
    if (mb > 1 && 32 * (mb - 1) >= B) break;
    for (int want = 1; want <= GEMM_MAX_PARTS; want++) {
      const int per = cdiv(nslab, want), n = cdiv(nslab, per);
      // (an item prefetches two slabs of the next one, so no part may have fewer)
      if (n != want || (n > 1 && (per < 4 || nslab - per * (n - 1) < 2 || (size_t)n * B * N > max_elems))) continue;
      const long long items = (long long)cdiv(B, 32 * mb) * g.n_col_tiles * n;
      const double cost = (double)((items + 255) / 256) * (per * slab_us(mb) + 5.0) + (n - 1) * (double)B * N * 8 / 5e6;
      if ((mb == 1 && n == 1) || cost < best) {
        best = cost;
        rpt = 32 * mb;
        splits = n;
        slabs = per;
      }
    }
  }
  if (splits == 1) return run_gemm_dense(g, EPI_F32, rpt, cdiv(B, rpt), s);
  g.k_splits = splits;
  g.split_slabs = slabs;
  *parts = splits;
  return run_gemm_dense(g, EPI_PARTIAL, rpt, cdiv(B, rpt), s);
}

}  // namespace gptoss

using namespace gptoss;

extern "C" size_t gptoss_packed_weight_bytes(int n_mat, int n_out, int n_in) {
  if (n_mat <= 0 || n_out <= 0 || n_in <= 0) return 0;
  return (size_t)n_mat * n_out * n_in * sizeof(bf16_t);
}

extern "C" int gptoss_pack_weight(const void *src, void *dst, int n_mat, int n_out, int n_in,
                                  int flags, void *stream) {
  GPTOSS_REQUIRE(src && dst, GPTOSS_ERR_NULL, "pack_weight: null pointer");
  const int glu = (flags & GPTOSS_PACK_GLU) ? 1 : 0;
  GPTOSS_REQUIRE(n_mat >= 1 && n_out > 0 && n_in > 0 && n_out % 32 == 0 && n_in % 64 == 0, GPTOSS_ERR_DIM,
                 "pack_weight: need n_out %% 32 == 0 and n_in %% 64 == 0 (n_out=%d n_in=%d)", n_out, n_in);
  GPTOSS_REQUIRE(aligned(src, 16) && aligned(dst, 16), GPTOSS_ERR_ALIGN,
                 "pack_weight: pointers must be 16-byte aligned");
  size_t threads = (size_t)(n_out / 32) * (n_in / 16) * 64;
  dim3 grid((unsigned)((threads + 255) / 256), n_mat);
  hipStream_t s = (hipStream_t)stream;
  if (flags & GPTOSS_PACK_SRC_FP32)
    pack_weight_kernel<float><<<grid, 256, 0, s>>>((const float *)src, (bf16_t *)dst, n_out, n_in, glu);
  else
    pack_weight_kernel<bf16_t><<<grid, 256, 0, s>>>((const bf16_t *)src, (bf16_t *)dst, n_out, n_in, glu);
  GPTOSS_LAUNCH_CHECK("pack_weight_kernel");
  return GPTOSS_OK;
}
