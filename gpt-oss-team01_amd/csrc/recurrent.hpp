// Internal interface of the recurrent mixers (recurrent.hip): short causal convolution, the gated
// delta rules, the state-space recurrence and retention, and their gated output norms.
#pragma once
#include "engine.hpp"
#include "rotary.hpp"

namespace gptoss {

// A causal convolution per channel followed by silu, over `channels` consecutive columns of the
// projected rows; some of its heads are then made unit vectors.
struct ShortConv {
  int col = 0, channels = 0, taps = 1;  // taps - 1 earlier inputs per channel are state
  const float *weight = nullptr;        // [channels, taps], newest tap last
  const float *bias = nullptr;          // [channels] or nullptr
  // the first n_unit * 2 heads of unit_dim channels are unit vectors; the first n_unit of them are
  // also scaled by unit_scale (queries, then keys); the remaining channels are taken as they are
  int n_unit = 0, unit_dim = 0;
  float unit_scale = 1.f;
};
// rows `in` [n, ld_in] -> out [n, ld_out]; state [slots, taps - 1, channels] is read, not written
int run_short_conv(const ShortConv &c, const StepRows &r, const float *in, int ld_in, const float *state,
                   float *out, int ld_out, hipStream_t s);

enum ScanKind { SCAN_DELTA = 0, SCAN_CHANNEL_DELTA = 1, SCAN_STATE_SPACE = 2, SCAN_RETENTION = 3 };
constexpr int SCAN_MAX_KEY = 256;   // largest key (state) dimension
constexpr int RETENTION_CHUNK = 64; // most tokens of a chunk (retention.hip)
constexpr int RETENTION_FEW = 8;    // stretches of up to so many rows are taken token by token

// One recurrence over the rows of a step, per sequence and head.  The state of a head is K x V
// (keys x values), kept in fp32 as [slots, heads, V, key_pad(K)].
struct Scan {
  ScanKind kind = SCAN_DELTA;
  int heads = 0, key_heads = 0, K = 0, V = 0;
  // columns of the convolved rows (retention: of rows that no convolution precedes): queries and keys (C and B)
  // per key head, values (x) per head
  const float *conv = nullptr;
  int ld_conv = 0, q_col = 0, k_col = 0, v_col = 0;
  // columns of the projected rows: write strength (delta rules) and decay (step size)
  const float *in = nullptr;
  int ld_in = 0, beta_col = 0, decay_col = 0;
  const float *channel_decay = nullptr;  // [n, ld_decay]: heads x K (SCAN_CHANNEL_DELTA)
  int ld_decay = 0;
  const float *a_log = nullptr, *dt_bias = nullptr, *d_skip = nullptr;
  const float *head_decay = nullptr;     // [heads] (SCAN_RETENTION): the decay itself
  const float *decay_powers = nullptr;   // [heads, RETENTION_CHUNK + 1]: its powers from the 0th on
  float value_scale = 1.f;               // of what is written (SCAN_RETENTION)
  Rotary rot;                            // of queries and keys (SCAN_RETENTION; run_scan: steps of one row per sequence)
  float *state = nullptr;
  float *out = nullptr;   // [n, ld_out]: heads x V
  int ld_out = 0;
  // the convolution's state is brought up to date by the same launch
  ShortConv conv_desc;
  float *conv_state = nullptr;
  int vec = 0;            // the launch's choice of loads (retention chunks: of stores), 16 bytes at a time
};
inline int scan_key_pad(int K) { return (K + 31) / 32 * 32; }
inline size_t scan_state_elems(int heads, int K, int V) { return (size_t)heads * V * scan_key_pad(K); }
// rows may be read 16 bytes at a time
inline bool scan_reads_wide(const Scan &p) {
  return p.K % 4 == 0 && p.V % 4 == 0 && p.ld_conv % 4 == 0 && p.k_col % 4 == 0 && p.q_col % 4 == 0 && p.v_col % 4 == 0 &&
         aligned(p.conv, 16) &&
         (p.kind != SCAN_CHANNEL_DELTA || (p.ld_decay % 4 == 0 && aligned(p.channel_decay, 16)));
}
int run_scan(const Scan &p, const StepRows &r, hipStream_t s);
// Retention: rotation of the rows' queries and keys, and the recurrence (retention.hip).  Stretches of more than
// RETENTION_FEW rows go through the matrix cores chunk by chunk, unless tokens_only; everything else is run_scan's,
// for which `rows` (p.conv) may be rotated in place.
int run_retention(const Scan &p, const StepRows &r, bool tokens_only, float *rows, hipStream_t s);

// Output of a recurrence -> one range of the output projection's input rows.
struct GatedNorm {
  const float *y = nullptr;      // [n, ld_y]: groups x size
  int ld_y = 0, groups = 0, size = 0;
  const float *gate = nullptr;   // [n, ld_gate]: groups x size
  int ld_gate = 0;
  int gate_first = 0;            // 1: y * silu(gate), then the norm; 0: the norm, then the gate
  int sigmoid_gate = 0;          // gate behind the norm: sigmoid instead of silu
  const float *weight = nullptr; // [size], or [groups * size] with weight_per_group; nullptr: ones
  int weight_per_group = 0;
  float scale = 1.f, eps = 1e-5f;
  void *out = nullptr;           // bf16 (or fp32 with out_f32) [n, ld_out], from column out_col
  int ld_out = 0, out_col = 0, out_f32 = 0;
};
int run_gated_norm(const GatedNorm &g, int n, hipStream_t s);

// out[:, i] = f(in[:, col + i]), i < width; f: the square of relu, or the identity (what EPI_MIXED does in
// the bf16 GEMM, for fp32 rows)
int run_column_map(const float *in, int ld_in, int col, int width, bool relu_squared, float *out, int ld_out, int n,
                   hipStream_t s);

}  // namespace gptoss
