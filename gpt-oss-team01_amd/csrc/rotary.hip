// Rotary positions over the rows of a step.
#include <math.h>

#include <algorithm>

#include "rotary.hpp"

namespace gptoss {

std::vector<float> rotary_table(const RotarySpec &r, int positions) {
  const int half = r.dims / 2;
  const bool scaled = r.factor > 0.0;
  std::vector<double> freq(half);
  double gain = 1.0, lo = 0.0, width = 1.0;
  if (scaled) {
    // the (fractional) pair index at which a pair makes `turns` turns in `original` positions
    auto place = [&](double turns) { return r.dims * log(r.original / (2.0 * M_PI * turns)) / (2.0 * log(r.base)); };
    lo = std::max(floor(place(r.fast)), 0.0);
    width = std::max(std::min(ceil(place(r.slow)), r.dims - 1.0) - lo, 0.001);
    gain = 0.1 * log(r.factor) + 1.0;
  }
  for (int i = 0; i < half; i++) {
    freq[i] = pow(r.base, -2.0 * i / r.dims);
    if (scaled) {
      const double ramp = std::min(std::max((i - lo) / width, 0.0), 1.0);
      freq[i] = freq[i] / r.factor * ramp + freq[i] * (1.0 - ramp);
    }
  }
  std::vector<float> t((size_t)positions * half * 2);
  for (int p = 0; p < positions; p++)
    for (int i = 0; i < half; i++) {
      const double a = p * freq[i];
      t[((size_t)p * half + i) * 2] = (float)(gain * cos(a));
      t[((size_t)p * half + i) * 2 + 1] = (float)(gain * sin(a));
    }
  return t;
}

// One thread per pair of a row.
__global__ __launch_bounds__(256) void rotary_kernel(Rotary r, float *__restrict__ x, int ld, int col, int dim, int pairs,
                                                     const int *__restrict__ lens) {
  const int half = r.dims >> 1, row = blockIdx.y, p = blockIdx.x * 256 + threadIdx.x;
  if (p >= pairs) return;
  const int head = p / half, i = p - head * half;
  const float2 cs = reinterpret_cast<const float2 *>(r.table)[(size_t)(lens[row] - 1) * half + i];
  float *h = x + (size_t)row * ld + col + head * dim;
  float *a = h + (r.interleaved ? 2 * i : i), *b = h + (r.interleaved ? 2 * i + 1 : i + half);
  const float u = *a, v = *b;
  *a = u * cs.x - v * cs.y;
  *b = v * cs.x + u * cs.y;
}

int run_rotary(const Rotary &r, float *x, int ld, int col, int heads, int dim, const int *lens, int n, hipStream_t s) {
  GPTOSS_REQUIRE(r.table && r.dims >= 2 && r.dims % 2 == 0 && r.dims <= dim, GPTOSS_ERR_DIM,
                 "rotary: %d of %d dimensions (an even number)", r.dims, dim);
  TraceScope ts("rotary", s);
  const int pairs = heads * (r.dims / 2);
  rotary_kernel<<<dim3(cdiv(pairs, 256), n), 256, 0, s>>>(r, x, ld, col, dim, pairs, lens);
  GPTOSS_LAUNCH_CHECK("rotary_kernel");
  return GPTOSS_OK;
}

}  // namespace gptoss
