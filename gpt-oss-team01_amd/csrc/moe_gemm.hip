// Host side of the grouped GEMMs (kernel dispatch), the weighted combine kernel and the MXFP4
// repacking kernel.  The GEMM kernel itself is in gemm_kernel.hpp.
#include <stdlib.h>

#include <mutex>

#include "common.hpp"
#include "gemm.hpp"

namespace gptoss {

// A token's experts in ascending order: their rows of y2 and their weights.
template <int KMAX>
struct TokenExperts {
  int rows[KMAX];
  float w[KMAX];
  __device__ __forceinline__ void load(const float *__restrict__ topk_w, const int *__restrict__ inv_perm, int b, int k) {
#pragma unroll
    for (int s = 0; s < KMAX; s++) {
      rows[s] = (s < k) ? inv_perm[(size_t)b * k + s] : 0x7fffffff;
      w[s] = (s < k) ? topk_w[(size_t)b * k + s] : 0.f;
    }
    // sorted position grows with expert id, so ordering by row orders by expert
#pragma unroll
    for (int i = 0; i < KMAX; i++)
#pragma unroll
      for (int j = 0; j + 1 < KMAX - i; j++)
        if (rows[j] > rows[j + 1]) {
          int tr = rows[j]; rows[j] = rows[j + 1]; rows[j + 1] = tr;
          float tw = w[j]; w[j] = w[j + 1]; w[j + 1] = tw;
        }
  }
  __device__ __forceinline__ f32x4 sum(const float *__restrict__ y2, int H, int h, int k) const {
    f32x4 agg = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < KMAX; s++) {
      if (s < k) {
        const f32x4 v = *reinterpret_cast<const f32x4 *>(y2 + (size_t)rows[s] * H + h);
#pragma unroll
        for (int q = 0; q < 4; q++) agg[q] = __fadd_rn(agg[q], __fmul_rn(v[q], w[s]));
      }
    }
    return agg;
  }
};

// Weighted combine: out[b,:] (+)= sum over the token's k experts, in ascending expert order (the
// order of the reference CPU loop, run.cpp:642-704), of w * y2[row of that pair].  Products and
// sums are rounded separately, as that loop rounds them.
// KMAX: room for a token's experts.
template <int VPT, int KMAX = 8>  // float4 chunks per thread: rows of at most 1024 * VPT floats (0: any length, a loop)
__global__ __launch_bounds__(256) void combine_kernel(const float *__restrict__ y2,
                                                      const float *__restrict__ topk_w,
                                                      const int *__restrict__ inv_perm,
                                                      float *__restrict__ out, int H, int k,
                                                      int accumulate) {
  const int b = blockIdx.x;
  TokenExperts<KMAX> x;
  x.load(topk_w, inv_perm, b, k);
  auto chunk = [&](int h) {
    f32x4 agg = x.sum(y2, H, h, k);
    f32x4 *op = reinterpret_cast<f32x4 *>(out + (size_t)b * H + h);
    if (accumulate) {
      f32x4 prev = *op;
#pragma unroll
      for (int q = 0; q < 4; q++) agg[q] = __fadd_rn(prev[q], agg[q]);
    }
    *op = agg;
  };
  if constexpr (VPT > 0) {
    // unrolled: the loads of every chunk are in flight before the first sum needs one
#pragma unroll
    for (int i = 0; i < VPT; i++) {
      const int h = (threadIdx.x + 256 * i) * 4;
      if (h < H) chunk(h);
    }
  } else {
    for (int h = threadIdx.x * 4; h < H; h += 256 * 4) chunk(h);
  }
}

// The same combine followed by the RMSNorm of the updated row (the next block's input norm), for
// rows of at most 1024 * VPT floats: every thread keeps its elements in registers between the two
// steps.  Element-to-thread mapping, the double-precision sum of squares and the scaling are those
// of rmsnorm_rows_kernel (glue.hip), so the result equals running the two kernels one after the
// other bit for bit.
template <int VPT>
__global__ __launch_bounds__(256) void combine_norm_kernel(const float *__restrict__ y2,
                                                           const float *__restrict__ topk_w,
                                                           const int *__restrict__ inv_perm,
                                                           float *__restrict__ out, int H, int k,
                                                           const float *__restrict__ norm_w,
                                                           bf16_t *__restrict__ t_bf16) {
  __shared__ double red[4];
  const int b = blockIdx.x;
  TokenExperts<8> x;
  x.load(topk_w, inv_perm, b, k);
  f32x4 v[VPT];
  double ss = 0.0;
#pragma unroll
  for (int i = 0; i < VPT; i++) {
    const int h = (threadIdx.x + 256 * i) * 4;
    v[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (h < H) {
      const f32x4 agg = x.sum(y2, H, h, k);
      f32x4 *op = reinterpret_cast<f32x4 *>(out + (size_t)b * H + h);
      const f32x4 prev = *op;
#pragma unroll
      for (int q = 0; q < 4; q++) v[i][q] = __fadd_rn(prev[q], agg[q]);
      *op = v[i];
#pragma unroll
      for (int q = 0; q < 4; q++) ss += (double)__fmul_rn(v[i][q], v[i][q]);
    }
  }
  for (int m = 32; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, 64);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
  __syncthreads();
  ss = red[0] + red[1] + red[2] + red[3];
  ss /= H;
  ss += 1e-5f;
  const double inv = (double)(1.0f / sqrtf((float)ss));
#pragma unroll
  for (int i = 0; i < VPT; i++) {
    const int h = (threadIdx.x + 256 * i) * 4;
    if (h < H) {
      const f32x4 nw = *reinterpret_cast<const f32x4 *>(norm_w + h);
      f32x4 o;
#pragma unroll
      for (int q = 0; q < 4; q++) o[q] = (float)((double)nw[q] * (inv * (double)v[i][q]));
      *reinterpret_cast<u32x2 *>(t_bf16 + (size_t)b * H + h) =
          u32x2{pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3])};
    }
  }
}

// The combine into the residual stream followed by a dynamic tanh norm of the updated row, element by element.
template <int KMAX>
__global__ __launch_bounds__(256) void combine_tanh_norm_kernel(const float *__restrict__ y2,
                                                                const float *__restrict__ topk_w,
                                                                const int *__restrict__ inv_perm,
                                                                float *__restrict__ out, int H, int k, TanhNorm norm,
                                                                bf16_t *__restrict__ t_bf16) {
  const int b = blockIdx.x, h = (blockIdx.y * 256 + threadIdx.x) * 4;
  TokenExperts<KMAX> x;
  x.load(topk_w, inv_perm, b, k);
  if (h >= H) return;
  const f32x4 agg = x.sum(y2, H, h, k);
  f32x4 *op = reinterpret_cast<f32x4 *>(out + (size_t)b * H + h);
  const f32x4 prev = *op, w = *reinterpret_cast<const f32x4 *>(norm.weight + h),
              c = *reinterpret_cast<const f32x4 *>(norm.bias + h);
  f32x4 v, o;
#pragma unroll
  for (int q = 0; q < 4; q++) {
    v[q] = __fadd_rn(prev[q], agg[q]);
    o[q] = fmaf(tanhf(norm.alpha * v[q]), w[q], c[q]);
  }
  *op = v;
  *reinterpret_cast<u32x2 *>(t_bf16 + (size_t)b * H + h) = u32x2{pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3])};
}

// MXFP4 repack: blocks [n_out, n_in/2] (low nibble = even element) and e8m0 scales [n_out, n_in/32]
// -> per (32-column block, 64-k slab): 64 lanes x 16 bytes of codes, then 32 x 2 scale bytes.
__global__ __launch_bounds__(256) void pack_mxfp4_kernel(const unsigned char *__restrict__ blocks,
                                                         const unsigned char *__restrict__ scales,
                                                         unsigned char *__restrict__ dst, int n_out,
                                                         int n_in, int glu) {
  const int nslab = n_in / 64;
  const size_t items = (size_t)(n_out / 32) * nslab;          // (column block, slab)
  const size_t gid = (size_t)blockIdx.x * 256 + threadIdx.x;  // one (item, lane) per thread
  const size_t item = gid >> 6;
  const int lane = (int)(gid & 63);
  const int mat = blockIdx.y;
  if (item >= items) return;
  const int nb = (int)(item / nslab), slab = (int)(item - (size_t)nb * nslab);
  int v = nb * 32 + (lane & 31);
  int row = v;
  if (glu) row = 2 * ((v >> 5) * 16 + (v & 15)) + ((v >> 4) & 1);
  const size_t mat_bytes = (size_t)n_out * n_in / 2 + (size_t)n_out * n_in / 32;
  const unsigned char *brow = blocks + ((size_t)mat * n_out + row) * (n_in / 2);
  const unsigned char *srow = scales + ((size_t)mat * n_out + row) * (n_in / 32);
  unsigned char *md = dst + (size_t)mat * mat_bytes;
  uint32_t w[4];
#pragma unroll
  for (int kk = 0; kk < 4; kk++) {
    const int k0 = (slab * 4 + kk) * 16 + (lane >> 5) * 8;  // the lane's 8 consecutive k
    w[kk] = *reinterpret_cast<const uint32_t *>(brow + k0 / 2);  // nibble j = element k0+j
  }
  *reinterpret_cast<u32x4 *>(md + (item * 64 + lane) * 16) = u32x4{w[0], w[1], w[2], w[3]};
  if (lane < 32) {
    unsigned char *sd = md + (size_t)n_out * n_in / 2 + (item * 32 + lane) * 2;
    sd[0] = srow[slab * 2];
    sd[1] = srow[slab * 2 + 1];
  }
}

// Host-side dispatcher used by the MoE layer.  rows_per_tile selects the kernel.
template <int MBMAX, bool GATHER, int EPI, bool FP4>
int launch_gemm(const GemmParams &p, int max_tiles, hipStream_t s);  // gemm_gather_bf16.hip

int (*run_gemm_mxfp4)(const GemmParams &p, bool gather, int epi, int rows_per_tile, int max_tiles, hipStream_t s) = nullptr;

template <bool GATHER, int EPI>
static int dispatch_rows(const GemmParams &p, int rows_per_tile, int max_tiles, hipStream_t s) {
  switch (rows_per_tile) {
    case 32: return launch_gemm<1, GATHER, EPI, false>(p, max_tiles, s);
    case 64: return launch_gemm<2, GATHER, EPI, false>(p, max_tiles, s);
    case 96: return launch_gemm<3, GATHER, EPI, false>(p, max_tiles, s);
    case 128: return launch_gemm<4, GATHER, EPI, false>(p, max_tiles, s);
    case 160: return launch_gemm<5, GATHER, EPI, false>(p, max_tiles, s);
  }
  return fail(GPTOSS_ERR_DIM, "run_gemm: unsupported rows_per_tile %d", rows_per_tile);
}

hipError_t gemm_set_attrs_gather_bf16();  // gemm_gather_bf16.hip

// Raises the dynamic-LDS limit of every grouped GEMM kernel on the calling thread's current device, the
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
    GPTOSS_HIP(gemm_set_attrs_gather_bf16());
    done[dev] = true;
  }
  return GPTOSS_OK;
}

int run_gemm(const GemmParams &p, bool gather, int epi, int rows_per_tile, int max_tiles,
             hipStream_t s) {
  if (!gather && !p.w_mxfp4) return run_gemm_dense(p, epi, rows_per_tile, max_tiles, s);
  // output and operand offsets inside the kernels are 32-bit element counts
  const long long max_rows = p.tiles ? (long long)max_tiles * rows_per_tile : p.dense_rows;
  GPTOSS_REQUIRE(max_rows * p.N < (1ll << 32) && max_rows * p.K < (1ll << 32), GPTOSS_ERR_DIM,
                 "run_gemm: rows x columns must stay below 2^32 elements (rows<=%lld N=%d K=%d)", max_rows, p.N, p.K);
  if (rows_per_tile == 256) {
    GPTOSS_REQUIRE(gather && epi == EPI_SWIGLU, GPTOSS_ERR_DIM, "run_gemm: no 256-row tiles for this form (epi=%d)", epi);
    return run_gemm_tall_gather(p, max_tiles, max_rows, s);
  }
  if (p.w_mxfp4) {
    GPTOSS_REQUIRE(run_gemm_mxfp4, GPTOSS_ERR_STATE, "run_gemm: this library was linked without the MXFP4 kernels");
    return run_gemm_mxfp4(p, gather, epi, rows_per_tile, max_tiles, s);
  }
  int prc = gemm_prepare_device();
  if (prc != GPTOSS_OK) return prc;
  if (gather && epi == EPI_SWIGLU) return dispatch_rows<true, EPI_SWIGLU>(p, rows_per_tile, max_tiles, s);
  return fail(GPTOSS_ERR_DIM, "run_gemm: unsupported combination (gather=%d epi=%d)", (int)gather, epi);
}

int run_combine(const float *y2, const float *topk_w, const int *inv_perm, float *out, int B, int H,
                int k, int accumulate, const float *norm_w, bf16_t *norm_out, hipStream_t s,
                const TanhNorm *tanh_norm) {
  if (B == 0) return GPTOSS_OK;
  if (tanh_norm && tanh_norm->weight) {
    GPTOSS_REQUIRE(accumulate && norm_out && H % 4 == 0, GPTOSS_ERR_DIM, "combine: the tanh norm follows an accumulation");
    TraceScope ts("combine_tanh_norm", s);
    const dim3 grid(B, cdiv(H, 1024));
    if (k <= 8) combine_tanh_norm_kernel<8><<<grid, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, *tanh_norm, norm_out);
    else combine_tanh_norm_kernel<MOE_MAX_TOP><<<grid, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, *tanh_norm, norm_out);
    GPTOSS_LAUNCH_CHECK("combine_tanh_norm_kernel");
    return GPTOSS_OK;
  }
  // out += combine, then norm_out = RMSNorm(out) * norm_w in the same kernel, when asked for
  if (norm_w && norm_out && accumulate && k <= 8 && H % 4 == 0 && H <= 4096 && aligned(norm_w, 16) && aligned(norm_out, 8)) {
    TraceScope ts("combine_rmsnorm", s);
    if (H <= 1024) combine_norm_kernel<1><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, norm_w, norm_out);
    else if (H <= 2048) combine_norm_kernel<2><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, norm_w, norm_out);
    else if (H <= 3072) combine_norm_kernel<3><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, norm_w, norm_out);
    else combine_norm_kernel<4><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, norm_w, norm_out);
    GPTOSS_LAUNCH_CHECK("combine_norm_kernel");
    return GPTOSS_OK;
  }
  {
    TraceScope ts("combine", s);
    if (k > 8) combine_kernel<0, MOE_MAX_TOP><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, accumulate);
    else if (H <= 3072 && H > 2048) combine_kernel<3><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, accumulate);
    else if (H <= 1024) combine_kernel<1><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, accumulate);
    else combine_kernel<0><<<B, 256, 0, s>>>(y2, topk_w, inv_perm, out, H, k, accumulate);
  }
  GPTOSS_LAUNCH_CHECK("combine_kernel");
  return GPTOSS_OK;
}

}  // namespace gptoss

using namespace gptoss;

extern "C" size_t gptoss_packed_mxfp4_bytes(int n_mat, int n_out, int n_in) {
  if (n_mat <= 0 || n_out <= 0 || n_in <= 0) return 0;
  return (size_t)n_mat * ((size_t)n_out * n_in / 2 + (size_t)n_out * n_in / 32);
}

extern "C" int gptoss_pack_mxfp4(const void *blocks, const void *scales, void *dst, int n_mat,
                                 int n_out, int n_in, int flags, void *stream) {
  GPTOSS_REQUIRE(blocks && scales && dst, GPTOSS_ERR_NULL, "pack_mxfp4: null pointer");
  const int glu = (flags & GPTOSS_PACK_GLU) ? 1 : 0;
  GPTOSS_REQUIRE(n_mat >= 1 && n_out > 0 && n_in > 0 && n_out % 32 == 0 && n_in % 64 == 0, GPTOSS_ERR_DIM,
                 "pack_mxfp4: need n_out %% 32 == 0 and n_in %% 64 == 0 (n_out=%d n_in=%d)", n_out, n_in);
  GPTOSS_REQUIRE(aligned(blocks, 4) && aligned(dst, 16), GPTOSS_ERR_ALIGN,
                 "pack_mxfp4: blocks must be 4-byte and dst 16-byte aligned");
  size_t threads = (size_t)(n_out / 32) * (n_in / 64) * 64;
  dim3 grid((unsigned)((threads + 255) / 256), n_mat);
  pack_mxfp4_kernel<<<grid, 256, 0, (hipStream_t)stream>>>((const unsigned char *)blocks,
                                                          (const unsigned char *)scales,
                                                          (unsigned char *)dst, n_out, n_in, glu);
  GPTOSS_LAUNCH_CHECK("pack_mxfp4_kernel");
  return GPTOSS_OK;
}
