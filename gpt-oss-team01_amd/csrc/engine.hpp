// What every model served by the engine shares: device memory, the rows of a step, sampling, cache
// slots, and the interface the scheduler drives a model through.  A model (model_*.cpp) derives from
// gptoss_engine, owns its weights and per-slot caches or states, and implements forward_rows.
#pragma once
#include <string.h>

#include <algorithm>
#include <vector>

#include "common.hpp"
#include "gemm.hpp"
#include "glue.hpp"
#include "precise.hpp"

namespace gptoss {

// Consecutive rows of a step that belong to one sequence.
struct RowSeg {
  int row0, n, slot, pos0;
};

// The rows of one step, as uploaded: row i feeds tokens[i] at position lens[i] - 1 of cache slot
// slots[i].  Host-side segment list beside the device arrays, for launch shapes.
struct StepRows {
  int n = 0, n_seg = 0, max_len = 1;
  const int *tokens = nullptr, *slots = nullptr, *lens = nullptr;
  const int *offset = nullptr;     // rows of the same sequence in front of row i in this step
  const RowSeg *segs = nullptr;    // [n_seg], device
  const int *sample = nullptr;     // rows whose next id (or logits) is wanted
  const RowSeg *singles = nullptr; // the segments of one row
  int n_singles = 0, longest = 1;
  struct Tiles {                   // the segments of several rows, cut into pieces of at most `rows` rows
    int rows = 0, n = 0;
    const RowSeg *tiles = nullptr;
  };
  std::vector<Tiles> tiles;        // one list per entry of gptoss_engine::tile_rows
};

}  // namespace gptoss

struct gptoss_engine {
  int max_batch = 0, max_seq = 0, flags = 0;
  hipStream_t stream = nullptr;
  std::vector<void *> allocs;
  size_t device_bytes = 0;
  // geometry of the residual stream and of the classifier
  int hidden = 0;        // row stride of the residual stream (a multiple of 64)
  int hidden_real = 0;   // its real width: what a mean is taken over; columns from there on are zero
  int vocab = 0;
  int vocab_rows = 0;    // vocabulary padded for the classifier: the row stride of the logits
  int n_layers = 0;
  float norm_eps = 1e-5f;
  std::vector<int> stop_ids;
  // final norm and classifier (bf16 packed, or fp32 row-major with GPTOSS_ENGINE_PRECISE)
  float *final_norm = nullptr;
  gptoss::bf16_t *unembedding = nullptr;
  float *unembedding_f32 = nullptr;
  float *class_bias = nullptr;   // [vocab_rows]: 0, and a large negative value in the padding; or nullptr
  float logit_softcap = 0.f;     // > 0: logits become softcap * tanh(logits / softcap) (their order stays)
  // run state
  int *d_next = nullptr;
  int *h_next = nullptr;         // pinned
  float *x = nullptr;            // [max_batch, hidden]: sampled rows (lock-step models: the whole batch)
  gptoss::bf16_t *t = nullptr;   // [max_batch, hidden]
  float *t_f32 = nullptr;        // likewise, GPTOSS_ENGINE_PRECISE
  float *logits = nullptr;       // [max_batch, vocab_rows], only with GPTOSS_ENGINE_LOGITS
  float *amax_val = nullptr;     // [max_batch, column tiles of the classifier]: fused arg-max partials
  int *amax_idx = nullptr;
  // rows of a step
  int rows = 0;                  // most rows of a pass; 0: the model has no step over rows
  float *rows_x = nullptr;       // [rows, hidden] residual stream, left by forward_rows
  int *d_rows = nullptr, *h_rows = nullptr;   // one uploaded block; h_rows is pinned
  size_t row_ints = 0;
  std::vector<int> tile_rows;    // piece sizes the model's kernels want (StepRows::tiles)
  std::vector<gptoss::RowSeg> seg_scratch;
  // cache slots handed out to callers that keep sequences of their own
  std::vector<char> slot_used;
  std::vector<int> lengths;      // models with states: positions every slot's states hold (continue_slots)

  virtual ~gptoss_engine();
  bool precise() const { return (flags & GPTOSS_ENGINE_PRECISE) != 0; }

  // Embedding and all layers for the rows of a step: leaves the residual stream in rows_x.
  virtual int forward_rows(const gptoss::StepRows &r) = 0;
  // Consecutive rows of one sequence that one pass may hold from position pos on (at least 1).
  virtual int max_stretch(int pos) const = 0;
  // Model-specific checks of a row list, before anything is launched.
  virtual int check_segments(const std::vector<gptoss::RowSeg> &) { return GPTOSS_OK; }
  // One position of sequences 0..B-1 (host_pos == nullptr: all at pos).
  virtual int step(const int *host_tokens, int pos, const int *host_pos, int B, int *host_next);
  // Positions 0..T-1 of sequences 0..B-1.
  virtual int prefill(const int *host_tokens, int B, int T, int *host_next);
  virtual bool reference_schedule() const { return false; }
  // x (m sampled rows) -> t (and t_f32): the norm in front of the classifier.
  virtual int norm_sampled(int m);
  virtual int tensor_view(int tensor, int layer, void **ptr, size_t *bytes);

  // check_segments of models with states: a state knows only its own position, so a sequence goes on where it
  // stopped, or starts over.
  int continue_slots(const std::vector<gptoss::RowSeg> &segs);

  // Validate, upload and run a row list; then next ids (host_next) or logits (host_logits) of the
  // sampled rows.  n <= rows; n_sample <= max_batch for ids.
  int run_rows(int n, const int *tok, const int *slot, const int *pos, int n_sample, const int *sample,
               int *host_next, float *host_logits);
  int validate_rows(int n, const int *slot, const int *pos, const char *who);

  // Allocation of the shared run state (the dimensions above, tile_rows and the flags must be set):
  // the rows of a step, and what sampling needs.
  int create_rows(int rows_cap);
  int create_sampling();
  int device_alloc(void **p, size_t bytes);

 private:
  int upload_rows(int n, const int *tok, const int *slot, const int *pos, int n_sample, const int *sample,
                  gptoss::StepRows *out);
  int class_gemm(int row0, int count, float *out);
  int sample_rows(const gptoss::StepRows &r, const int *sample, const int *slot, int first, int count);
};

namespace gptoss {

// most rows (sequences x positions) one pass works on
constexpr long long PREFILL_ROWS = 8192;

#define GPTOSS_STEP(call)                      \
  do {                                         \
    const int rc__ = (call);                   \
    if (rc__ != GPTOSS_OK) return rc__;        \
  } while (0)

}  // namespace gptoss
