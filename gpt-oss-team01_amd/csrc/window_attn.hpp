// Internal interface of the attention over a bounded stretch of the past, for the rows of a step
// (window_attn.hip).
#pragma once
#include "engine.hpp"
#include "rotary.hpp"

namespace gptoss {

// Causal attention inside a sliding window, or inside chunks of the sequence: with `chunked` a position sees
// those from the last multiple of `window` on.  Queries and keys are normed per head, or (whole_norm) over
// all heads' values at once, and then rotated where `rot` has a table; values may be the columns of the keys
// (v_col == k_col), as projected.
// The K/V of a sequence live in a ring of `cap` slots (position p in slot p % cap), which must hold what the
// first row of a stretch sees as well as the stretch: cap >= window - 1 + rows.
struct WindowAttn {
  int heads = 0, kv_heads = 0, dim = 0, vdim = 0, window = 0, cap = 0;
  float scale = 1.f, eps = 1e-5f, out_scale = 1.f;
  int chunked = 0, whole_norm = 0;
  const float *q_norm = nullptr, *k_norm = nullptr;   // [dim]; whole_norm: [heads * dim], [kv_heads * dim]
  Rotary rot;                                         // with whole_norm only
  // columns of the projected rows
  const float *in = nullptr;
  int ld_in = 0, q_col = 0, k_col = 0, v_col = 0;
  float *q = nullptr;          // scratch [n, heads, dim_pad]
  bf16_t *kv = nullptr;        // [slots, kv_heads, cap / 64] blocks (common.hpp), keys and values padded
  float *k32 = nullptr, *v32 = nullptr;   // instead, fp32: [slots, cap, kv_heads, dim] and [.., vdim]
  void *out = nullptr;         // bf16 (fp32 with k32) [n, ld_out], heads x vdim from column out_col
  int ld_out = 0, out_col = 0;
  int tiles = 0;               // index of its piece size in StepRows::tiles
  // first position that `pos` sees
  __host__ __device__ int first(int pos) const {
    const int lo = chunked ? pos / window * window : pos - window + 1;
    return lo > 0 ? lo : 0;
  }
  __host__ __device__ int dim_pad() const { return (dim + 31) / 32 * 32; }
  __host__ __device__ int vdim_pad() const { return (vdim + 31) / 32 * 32; }
  __host__ __device__ size_t block_elems() const { return (size_t)KV_BLOCK * (dim_pad() + vdim_pad()); }
};
constexpr int WINDOW_ATTN_MAX_DIM = 256;
// rows of a sequence that share a workgroup of the prompt kernel
inline int window_attn_tile_rows(int heads, int kv_heads) { return std::max(1, 128 / (heads / kv_heads)); }
// Norm of q and k, K/V into the ring, attention of every row up to its own position.
int run_window_attn(const WindowAttn &a, const StepRows &r, hipStream_t s);

}  // namespace gptoss
