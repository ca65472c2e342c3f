// The model-independent part of the engine: rows of a step, sampling, cache slots, and greedy
// generation: the reference's lock-step batches (getp-csrc/submit/getp_run_submit.cpp:13-96) or, by
// default, the same requests over a fixed set of slots that are refilled as sequences end.
#include "engine.hpp"

using namespace gptoss;


gptoss_engine::~gptoss_engine() {
  for (void *p : allocs) (void)hipFree(p);
  if (h_next) (void)hipHostFree(h_next);
  if (h_rows) (void)hipHostFree(h_rows);
  if (stream) (void)hipStreamDestroy(stream);
}

int gptoss_engine::device_alloc(void **p, size_t bytes) {
  bytes = align_up(std::max<size_t>(bytes, 1), 256);
  hipError_t err = hipMalloc(p, bytes);
  GPTOSS_REQUIRE(err == hipSuccess, GPTOSS_ERR_HIP, "engine: hipMalloc of %zu bytes failed: %s", bytes,
                 hipGetErrorString(err));
  allocs.push_back(*p);
  device_bytes += bytes;
  return GPTOSS_OK;
}

int gptoss_engine::create_rows(int rows_cap) {
  const size_t R = rows_cap, S = std::min(rows_cap, max_batch);
  row_ints = 4 * R + 8 * S + tile_rows.size() * 4 * (R + S) + std::max<size_t>(R, max_batch) + 4 * (8 + tile_rows.size());
  GPTOSS_STEP(device_alloc((void **)&d_rows, row_ints * sizeof(int)));
  GPTOSS_HIP(hipHostMalloc((void **)&h_rows, row_ints * sizeof(int), hipHostMallocDefault));
  GPTOSS_STEP(device_alloc((void **)&rows_x, R * hidden * sizeof(float)));
  rows = rows_cap;
  return GPTOSS_OK;
}

int gptoss_engine::create_sampling() {
  const size_t B = max_batch;
  GPTOSS_STEP(device_alloc((void **)&d_next, B * sizeof(int)));
  GPTOSS_HIP(hipHostMalloc((void **)&h_next, B * sizeof(int), hipHostMallocDefault));
  GPTOSS_STEP(device_alloc((void **)&x, B * hidden * sizeof(float)));
  GPTOSS_STEP(device_alloc((void **)&t, B * hidden * sizeof(bf16_t)));
  if (precise()) GPTOSS_STEP(device_alloc((void **)&t_f32, B * hidden * sizeof(float)));
  if (precise() || (flags & GPTOSS_ENGINE_LOGITS)) {
    GPTOSS_STEP(device_alloc((void **)&logits, B * vocab_rows * sizeof(float)));
  } else {
    const size_t pairs = B * gemm_argmax_tiles(vocab_rows);
    GPTOSS_STEP(device_alloc((void **)&amax_val, pairs * sizeof(float)));
    GPTOSS_STEP(device_alloc((void **)&amax_idx, pairs * sizeof(int)));
  }
  return GPTOSS_OK;
}

// One copy carries everything the kernels need to know about the rows of a step.
int gptoss_engine::upload_rows(int n, const int *tok, const int *slot, const int *pos, int n_sample,
                               const int *sample, StepRows *out) {
  size_t used = 0;
  auto take = [&](size_t ints) {
    const size_t o = used;
    used += align_up(ints, 4);   // every array starts 16-byte aligned
    return o;
  };
  StepRows &r = *out;
  r.n = n;
  const size_t o_tok = take(n), o_slot = take(n), o_len = take(n), o_off = take(n);
  seg_scratch.clear();
  for (int i = 0; i < n; i++) {
    if (i > 0 && slot[i] == slot[i - 1]) seg_scratch.back().n++;
    else seg_scratch.push_back({i, 1, slot[i], pos[i]});
    h_rows[o_tok + i] = tok[i];
    h_rows[o_slot + i] = slot[i];
    h_rows[o_len + i] = pos[i] + 1;
    h_rows[o_off + i] = i - seg_scratch.back().row0;
    r.max_len = std::max(r.max_len, pos[i] + 1);
  }
  GPTOSS_STEP(check_segments(seg_scratch));
  r.n_seg = (int)seg_scratch.size();
  const size_t o_seg = take(4 * (size_t)r.n_seg);
  memcpy(h_rows + o_seg, seg_scratch.data(), sizeof(RowSeg) * r.n_seg);
  r.longest = 1;
  for (const RowSeg &s : seg_scratch) {
    r.n_singles += s.n == 1;
    r.longest = std::max(r.longest, s.n);
  }
  size_t o_single = o_seg;   // all decoding: the two lists are one
  if (r.n_singles && r.n_singles < r.n_seg) {
    o_single = take(4 * (size_t)r.n_singles);
    RowSeg *d = (RowSeg *)(h_rows + o_single);
    for (const RowSeg &s : seg_scratch)
      if (s.n == 1) *d++ = s;
  }
  std::vector<size_t> o_tiles;
  for (int tr : tile_rows) {
    StepRows::Tiles t;
    t.rows = tr;
    const size_t o = used;
    RowSeg *d = (RowSeg *)(h_rows + o);
    for (const RowSeg &s : seg_scratch)
      if (s.n > 1)
        for (int i = 0; i < s.n; i += tr) d[t.n++] = {s.row0 + i, std::min(tr, s.n - i), s.slot, s.pos0 + i};
    take(4 * (size_t)t.n);
    o_tiles.push_back(o);
    r.tiles.push_back(t);
  }
  const size_t o_smp = take(n_sample);
  if (n_sample) memcpy(h_rows + o_smp, sample, sizeof(int) * n_sample);
  GPTOSS_REQUIRE(used <= row_ints, GPTOSS_ERR_STATE, "engine: row block of %zu ints exceeds %zu", used, row_ints);
  GPTOSS_HIP(hipMemcpyAsync(d_rows, h_rows, sizeof(int) * used, hipMemcpyHostToDevice, stream));
  r.tokens = d_rows + o_tok;
  r.slots = d_rows + o_slot;
  r.lens = d_rows + o_len;
  r.offset = d_rows + o_off;
  r.segs = (const RowSeg *)(d_rows + o_seg);
  r.singles = (const RowSeg *)(d_rows + o_single);
  r.sample = d_rows + o_smp;
  for (size_t i = 0; i < o_tiles.size(); i++) r.tiles[i].tiles = (const RowSeg *)(d_rows + o_tiles[i]);
  return GPTOSS_OK;
}

int gptoss_engine::class_gemm(int row0, int count, float *out) {
  if (precise())
    return precise_matmul(out, t_f32 + (size_t)row0 * hidden, unembedding_f32, class_bias, nullptr, count, hidden,
                          vocab_rows, 1, stream);
  return dense_gemm(t + (size_t)row0 * hidden, unembedding, class_bias, out, EPI_F32, count, vocab_rows, hidden, stream);
}

int gptoss_engine::norm_sampled(int m) {
  return run_rmsnorm(x, nullptr, final_norm, t, t_f32, m, hidden, stream, norm_eps, hidden_real);
}

// Next ids of normed sampled rows first .. first + count - 1 (count <= max_batch); with the
// logits kept, those of a sequence's row stay in its slot's place.
int gptoss_engine::sample_rows(const StepRows &r, const int *sample, const int *slot, int first, int count) {
  if (logits) {
    const int s0 = slot[sample[first]];
    bool adjacent = true;
    for (int j = 0; j < count; j++) adjacent = adjacent && slot[sample[first + j]] == s0 + j;
    for (int j = 0; j < count; j += adjacent ? count : 1) {
      const int m = adjacent ? count : 1;
      float *lg = logits + (size_t)slot[sample[first + j]] * vocab_rows;
      GPTOSS_STEP(class_gemm(j, m, lg));
      GPTOSS_STEP(run_argmax(lg, d_next + j, m, vocab_rows, stream));
      if (logit_softcap > 0.f) GPTOSS_STEP(run_softcap(lg, (size_t)m * vocab_rows, logit_softcap, stream));
    }
    return GPTOSS_OK;
  }
  int pairs = 0;
  GPTOSS_STEP(dense_gemm(t, unembedding, class_bias, nullptr, EPI_ARGMAX, count, vocab_rows, hidden, stream, amax_val,
                         amax_idx, &pairs));
  return run_argmax_tiles(amax_val, amax_idx, d_next, count, pairs, stream);
}

// One step over n arbitrary rows: row i feeds token tok[i] at position pos[i] of the sequence in
// cache slot slot[i].  The rows share every weight pass of the step, so the prompt of a request
// that has just been admitted costs a few more rows in the GEMMs of a step that runs anyway.
int gptoss_engine::run_rows(int n, const int *tok, const int *slot, const int *pos, int n_sample, const int *sample,
                            int *host_next, float *host_logits) {
  GPTOSS_REQUIRE(n >= 1 && n <= rows && n_sample >= 0 && n_sample <= (host_logits ? n : max_batch), GPTOSS_ERR_DIM,
                 "step_rows: %d rows (at most %d), %d sampled", n, rows, n_sample);
  GPTOSS_REQUIRE(!host_logits || logits, GPTOSS_ERR_STATE, "step_rows: logits need an engine with GPTOSS_ENGINE_LOGITS");
  StepRows r;
  GPTOSS_STEP(upload_rows(n, tok, slot, pos, n_sample, sample, &r));
  GPTOSS_STEP(forward_rows(r));
  for (int first = 0; first < n_sample; first += max_batch) {
    const int m = std::min(max_batch, n_sample - first);
    GPTOSS_STEP(run_gather_rows_idx(rows_x, x, r.sample + first, m, hidden, stream));
    GPTOSS_STEP(norm_sampled(m));
    if (host_logits) {
      GPTOSS_STEP(class_gemm(0, m, logits));
      if (logit_softcap > 0.f) GPTOSS_STEP(run_softcap(logits, (size_t)m * vocab_rows, logit_softcap, stream));
      GPTOSS_HIP(hipMemcpy2DAsync(host_logits + (size_t)first * vocab, sizeof(float) * vocab, logits,
                                  sizeof(float) * vocab_rows, sizeof(float) * vocab, m, hipMemcpyDeviceToHost, stream));
      GPTOSS_HIP(hipStreamSynchronize(stream));   // the buffer is reused by the next portion
    } else {
      GPTOSS_STEP(sample_rows(r, sample, slot, first, m));
      GPTOSS_HIP(hipMemcpyAsync(h_next, d_next, sizeof(int) * m, hipMemcpyDeviceToHost, stream));
    }
  }
  GPTOSS_HIP(hipStreamSynchronize(stream));
  if (host_next && !host_logits) memcpy(host_next, h_next, sizeof(int) * n_sample);
  return GPTOSS_OK;
}

int gptoss_engine::continue_slots(const std::vector<RowSeg> &segs) {
  for (const RowSeg &s : segs)
    GPTOSS_REQUIRE(s.pos0 == 0 || s.pos0 == lengths[s.slot], GPTOSS_ERR_STATE,
                   "step: slot %d holds %d positions and cannot continue at position %d", s.slot, lengths[s.slot], s.pos0);
  for (const RowSeg &s : segs) lengths[s.slot] = s.pos0 + s.n;
  return GPTOSS_OK;
}

int gptoss_engine::validate_rows(int n, const int *slot, const int *pos, const char *who) {
  std::vector<char> seen(max_batch, 0);
  for (int i = 0; i < n; i++) {
    GPTOSS_REQUIRE(slot[i] >= 0 && slot[i] < max_batch && pos[i] >= 0 && pos[i] < max_seq, GPTOSS_ERR_STATE,
                   "%s: row %d names slot %d, position %d (slots 0..%d, positions 0..%d)", who, i, slot[i], pos[i],
                   max_batch - 1, max_seq - 1);
    // several rows of one sequence: adjacent, consecutive, ascending
    if (i > 0 && slot[i] == slot[i - 1]) {
      GPTOSS_REQUIRE(pos[i] == pos[i - 1] + 1, GPTOSS_ERR_STATE,
                     "%s: rows %d and %d of slot %d must be consecutive positions (got %d, %d)", who, i - 1, i, slot[i],
                     pos[i - 1], pos[i]);
    } else {
      GPTOSS_REQUIRE(!seen[slot[i]], GPTOSS_ERR_STATE, "%s: the rows of slot %d must be adjacent", who, slot[i]);
      seen[slot[i]] = 1;
    }
  }
  return GPTOSS_OK;
}

// ---- defaults of the interface, over step rows -------------------------------------------------
int gptoss_engine::step(const int *host_tokens, int pos, const int *host_pos, int B, int *host_next) {
  std::vector<int> slot(B), at(B), sample(B);
  for (int i = 0; i < B; i++) {
    slot[i] = i;
    at[i] = host_pos ? host_pos[i] : pos;
  }
  for (int i0 = 0; i0 < B; i0 += rows) {
    const int m = std::min(rows, B - i0);
    for (int j = 0; j < m; j++) sample[j] = j;
    GPTOSS_STEP(run_rows(m, host_tokens + i0, &slot[i0], &at[i0], m, sample.data(), host_next + i0, nullptr));
  }
  return GPTOSS_OK;
}

int gptoss_engine::prefill(const int *host_tokens, int B, int T, int *host_next) {
  std::vector<int> tok, slot, pos, sample, owner, next(max_batch), done(B, 0);
  for (int lo = 0; lo < B;) {
    tok.clear(), slot.clear(), pos.clear(), sample.clear(), owner.clear();
    for (int i = lo; i < B && (int)tok.size() < rows; i++) {
      const int m = std::min({T - done[i], max_stretch(done[i]), rows - (int)tok.size()});
      for (int j = 0; j < m; j++) {
        tok.push_back(host_tokens[(size_t)i * T + done[i] + j]);
        slot.push_back(i);
        pos.push_back(done[i] + j);
      }
      done[i] += m;
      if (done[i] == T) {
        sample.push_back((int)tok.size() - 1);
        owner.push_back(i);
      }
    }
    GPTOSS_STEP(run_rows((int)tok.size(), tok.data(), slot.data(), pos.data(), (int)sample.size(), sample.data(),
                         next.data(), nullptr));
    for (size_t j = 0; j < owner.size(); j++) host_next[owner[j]] = next[j];
    while (lo < B && done[lo] == T) lo++;
  }
  return GPTOSS_OK;
}

int gptoss_engine::tensor_view(int, int, void **, size_t *) {
  return fail(GPTOSS_ERR_STATE, "engine_tensor_view: not available for this model");
}

static bool is_stop(const gptoss_engine *e, int id) {
  return std::find(e->stop_ids.begin(), e->stop_ids.end(), id) != e->stop_ids.end();
}
// The reference's schedule: requests in batches of max_batch, every batch in lock step until its
// last sequence ends (getp_run_submit.cpp:13-87).
static int generate_lockstep(gptoss_engine *e, const int *host_prompts, const int *host_n_prompt,
                             int prompt_stride, int n_req, int max_seq_len, int *host_out,
                             long long *n_generated) {
  long long total = 0;
  // requests are served in batches of max_batch, all sequences of a batch in lock step
  // (getp_run_submit.cpp:13-87)
  for (int r0 = 0; r0 < n_req; r0 += e->max_batch) {
    const int B = std::min(e->max_batch, n_req - r0);
    std::vector<int> cur_tok(B), cur_pos(B, 0), next(B);
    std::vector<char> active(B, 1);
    int active_count = B;
    for (int i = 0; i < B; i++) cur_tok[i] = host_prompts[(size_t)(r0 + i) * prompt_stride];
    // The prompt positions every sequence of the batch has in common go through one prefill pass
    // instead of one lock-step step each (the reference feeds prompts token by token,
    // getp_run_submit.cpp:60-72).  The pass stops before a prompt's own stop token, which ends
    // that sequence in the lock-step loop, and before the last position the loop may visit.
    int first_pos = 0;
    if (e->rows > 0 && !(e->flags & GPTOSS_ENGINE_PRECISE)) {
      int T = std::min(max_seq_len - 1, e->rows);
      for (int i = 0; i < B; i++) {
        const int *pt = host_prompts + (size_t)(r0 + i) * prompt_stride;
        const int np = host_n_prompt[r0 + i];
        T = std::min(T, np);
        for (int j = 1; j < T; j++)
          if (is_stop(e, pt[j])) T = j;
      }
      if (T >= 2) {
        std::vector<int> toks((size_t)B * T);
        for (int i = 0; i < B; i++)
          memcpy(&toks[(size_t)i * T], host_prompts + (size_t)(r0 + i) * prompt_stride, sizeof(int) * T);
        int rc = gptoss_engine_prefill(e, toks.data(), B, T, next.data());
        if (rc != GPTOSS_OK) return rc;
        first_pos = T;
        for (int i = 0; i < B; i++) cur_pos[i] = T - 1;  // the loop body below finishes position T-1
      }
    }
    for (int pos = first_pos > 0 ? first_pos - 1 : 0; pos < max_seq_len - 1 && active_count > 0; pos++) {
      if (pos >= first_pos) {
        int rc = gptoss_engine_step(e, cur_tok.data(), pos, B, next.data());
        if (rc != GPTOSS_OK) return rc;
      }
      for (int i = 0; i < B; i++) {
        if (!active[i]) continue;
        const int *pt = host_prompts + (size_t)(r0 + i) * prompt_stride;
        const int np = host_n_prompt[r0 + i];
        int *o = host_out + (size_t)(r0 + i) * (max_seq_len + 1);
        int nt = next[i];
        if (cur_pos[i] < np - 1) nt = pt[cur_pos[i] + 1];
        else o[cur_pos[i] - (np - 1)] = nt;
        if (is_stop(e, nt)) {
          active[i] = 0;
          active_count--;
        }
        cur_tok[i] = nt;
        cur_pos[i]++;
      }
    }
    for (int i = 0; i < B; i++) {
      int generated_len = cur_pos[i] - host_n_prompt[r0 + i];
      if (generated_len < 0) generated_len = 0;
      host_out[(size_t)(r0 + i) * (max_seq_len + 1) + generated_len + 1] = -1;
      total += generated_len + 1;
    }
  }
  if (n_generated) *n_generated = total;
  return GPTOSS_OK;
}

// Continuous batching: max_batch slots; a slot whose sequence ended (stop id or its length limit)
// takes the next waiting request at once, while the other slots carry on at their own positions.
// Every request sees the arithmetic it would see alone, so its output is the one the lock-step
// schedule gives; only the order of the work changes.  host_max_len (optional) limits request r
// to host_max_len[r] positions in all (prompt included) instead of max_seq_len.
//
// Prompts are not forced one token per step (getp_run_submit.cpp:67-72 does that).  The positions
// the first max_batch requests share go through one prompt pass; after that every step is a step
// over rows (step_rows): one row for each sequence that is decoding, and for a request that has
// just been admitted all the prompt positions it has left, as consecutive rows of the same step.
// Those rows ride along in the weight passes the step makes anyway, so a prompt costs its slot
// one step instead of one step per token.  On the sliding-window layers the rows of one step must
// stay inside the first lap of the ring, so prompt positions from the ring's capacity on are
// forced one per step as before; and a step never has more rows than the prompt buffers hold.
static int generate_continuous(gptoss_engine *e, const int *host_prompts, const int *host_n_prompt,
                               int prompt_stride, int n_req, int max_seq_len, const int *host_max_len,
                               int *host_out, long long *n_generated) {
  long long total = 0;
  const int B = std::min(e->max_batch, n_req);
  if (B == 0) {
    if (n_generated) *n_generated = 0;
    return GPTOSS_OK;
  }
  std::vector<int> req(B, -1), cur_tok(B, 0), cur_pos(B, 0), next(B), prefix(B, 0);
  int next_req = 0, active_count = 0;
  const bool rows_path = e->rows > 0;
  auto limit = [&](int r) { return host_max_len ? std::min(host_max_len[r], max_seq_len) : max_seq_len; };
  // prompt positions of request r that may be run without looking at a result: a prompt's own stop
  // token ends the sequence when it is fed, and the loop visits limit - 1 positions at most
  auto forced_prefix = [&](int r) {
    const int *pt = host_prompts + (size_t)r * prompt_stride;
    int T = std::min(host_n_prompt[r], limit(r) - 1);
    for (int j = 1; j < T; j++)
      if (is_stop(e, pt[j])) T = j;
    return T;
  };
  auto finish = [&](int i) {
    const int r = req[i];
    int generated_len = cur_pos[i] - host_n_prompt[r];
    if (generated_len < 0) generated_len = 0;
    host_out[(size_t)r * (max_seq_len + 1) + generated_len + 1] = -1;
    total += generated_len + 1;
    req[i] = -1;
    active_count--;
  };
  auto admit = [&](int i) {
    // requests that may not even take one step are closed as the lock-step loop closes them
    while (next_req < n_req) {
      const int r = next_req++;
      req[i] = r;
      cur_tok[i] = host_prompts[(size_t)r * prompt_stride];
      cur_pos[i] = 0;
      active_count++;
      if (limit(r) - 1 > 0) {
        prefix[i] = forced_prefix(r);
        return;
      }
      finish(i);
    }
    cur_tok[i] = 0;
    cur_pos[i] = 0;
  };
  // what the loop of getp_run_submit.cpp:60-96 does with the id the forward call of position
  // cur_pos returned
  auto advance = [&](int i, int next_id) {
    const int r = req[i];
    const int *pt = host_prompts + (size_t)r * prompt_stride;
    const int np = host_n_prompt[r];
    int *o = host_out + (size_t)r * (max_seq_len + 1);
    int nt = next_id;
    if (cur_pos[i] < np - 1) nt = pt[cur_pos[i] + 1];
    else o[cur_pos[i] - (np - 1)] = nt;
    cur_tok[i] = nt;
    cur_pos[i]++;
    if (is_stop(e, nt) || cur_pos[i] >= limit(r) - 1) {
      finish(i);
      admit(i);
    }
  };
  for (int i = 0; i < B; i++) admit(i);

  // the prompt positions the first B requests share go through one prompt pass
  bool first_wave = rows_path;
  for (int i = 0; i < B; i++) first_wave = first_wave && req[i] == i;
  if (first_wave) {
    int T = e->rows;
    for (int i = 0; i < B; i++) T = std::min(T, prefix[i]);
    if (T >= 2) {
      std::vector<int> toks((size_t)B * T);
      for (int i = 0; i < B; i++)
        memcpy(&toks[(size_t)i * T], host_prompts + (size_t)i * prompt_stride, sizeof(int) * T);
      int rc = gptoss_engine_prefill(e, toks.data(), B, T, next.data());
      if (rc != GPTOSS_OK) return rc;
      for (int i = 0; i < B; i++) cur_pos[i] = T - 1;  // advance() finishes position T-1
      for (int i = 0; i < B; i++) advance(i, next[i]);
    }
  }
  if (!rows_path) {
    while (active_count > 0) {
      int rc = gptoss_engine_step_ragged(e, cur_tok.data(), cur_pos.data(), B, next.data());
      if (rc != GPTOSS_OK) return rc;
      for (int i = 0; i < B; i++)
        if (req[i] >= 0) advance(i, next[i]);
    }
    if (n_generated) *n_generated = total;
    return GPTOSS_OK;
  }
  std::vector<int> r_tok, r_slot, r_pos, sample, owner, count(B);
  while (active_count > 0) {
    // rows of this step: one per running sequence, plus what fits of the prompt stretches
    int extra = e->rows - active_count;
    r_tok.clear();
    r_slot.clear();
    r_pos.clear();
    sample.clear();
    owner.clear();
    for (int i = 0; i < B; i++) {
      count[i] = 0;
      if (req[i] < 0) continue;
      // positions cur_pos .. cur_pos + m - 1 are prompt positions whose inputs are known
      const int m = std::max(1, std::min({prefix[i] - cur_pos[i], e->max_stretch(cur_pos[i]), 1 + std::max(0, extra)}));
      extra -= m - 1;
      const int *pt = host_prompts + (size_t)req[i] * prompt_stride;
      for (int j = 0; j < m; j++) {
        r_tok.push_back(j == 0 ? cur_tok[i] : pt[cur_pos[i] + j]);
        r_slot.push_back(i);
        r_pos.push_back(cur_pos[i] + j);
      }
      count[i] = m;
      sample.push_back((int)r_tok.size() - 1);
      owner.push_back(i);
    }
    int rc = e->run_rows((int)r_tok.size(), r_tok.data(), r_slot.data(), r_pos.data(), (int)sample.size(),
                         sample.data(), next.data(), nullptr);
    if (rc != GPTOSS_OK) return rc;
    for (size_t j = 0; j < owner.size(); j++) {
      const int i = owner[j];
      cur_pos[i] += count[i] - 1;  // advance() finishes the stretch's last position
      advance(i, next[j]);
    }
  }
  if (n_generated) *n_generated = total;
  return GPTOSS_OK;
}

extern "C" int gptoss_engine_generate_ragged(gptoss_engine *e, const int *host_prompts, const int *host_n_prompt,
                                             int prompt_stride, int n_req, int max_seq_len,
                                             const int *host_max_len, int *host_out, long long *n_generated) {
  GPTOSS_REQUIRE(e && host_prompts && host_n_prompt && host_out, GPTOSS_ERR_NULL, "engine_generate: null pointer");
  GPTOSS_REQUIRE(n_req >= 0 && prompt_stride >= 1 && max_seq_len >= 1 && max_seq_len <= e->max_seq + 1,
                 GPTOSS_ERR_DIM, "engine_generate: max_seq_len %d needs an engine with max_seq >= %d",
                 max_seq_len, max_seq_len - 1);
  for (int r = 0; r < n_req; r++)
    GPTOSS_REQUIRE(host_n_prompt[r] >= 1 && host_n_prompt[r] <= prompt_stride, GPTOSS_ERR_DIM,
                   "engine_generate: request %d has %d prompt tokens", r, host_n_prompt[r]);
  if (host_max_len)
    for (int r = 0; r < n_req; r++)
      GPTOSS_REQUIRE(host_max_len[r] >= 1, GPTOSS_ERR_DIM, "engine_generate: request %d has length limit %d", r,
                     host_max_len[r]);
  for (int i = 0; i < std::min(n_req, e->max_batch); i++)
    GPTOSS_REQUIRE(!e->slot_used[i], GPTOSS_ERR_STATE, "engine_generate: cache slot %d is held by a sequence", i);
  if (e->reference_schedule()) {
    GPTOSS_REQUIRE(!host_max_len, GPTOSS_ERR_STATE,
                   "engine_generate: per-request length limits need the continuous schedule "
                   "(not GPTOSS_ENGINE_PRECISE / GPTOSS_ENGINE_NO_PREFILL)");
    return generate_lockstep(e, host_prompts, host_n_prompt, prompt_stride, n_req, max_seq_len, host_out, n_generated);
  }
  return generate_continuous(e, host_prompts, host_n_prompt, prompt_stride, n_req, max_seq_len, host_max_len,
                             host_out, n_generated);
}

extern "C" int gptoss_engine_generate(gptoss_engine *e, const int *host_prompts, const int *host_n_prompt,
                                      int prompt_stride, int n_req, int max_seq_len, int *host_out,
                                      long long *n_generated) {
  return gptoss_engine_generate_ragged(e, host_prompts, host_n_prompt, prompt_stride, n_req, max_seq_len, nullptr,
                                       host_out, n_generated);
}

// ---- C ABI ---------------------------------------------------------------------------------------
extern "C" void gptoss_engine_destroy(gptoss_engine *e) { delete e; }

extern "C" int gptoss_engine_step(gptoss_engine *e, const int *host_tokens, int pos, int B, int *host_next) {
  GPTOSS_REQUIRE(e && host_tokens && host_next, GPTOSS_ERR_NULL, "engine_step: null pointer");
  GPTOSS_REQUIRE(B >= 1 && B <= e->max_batch, GPTOSS_ERR_DIM, "engine_step: batch %d outside 1..%d", B, e->max_batch);
  GPTOSS_REQUIRE(pos >= 0 && pos < e->max_seq, GPTOSS_ERR_STATE, "engine_step: position %d outside 0..%d", pos, e->max_seq - 1);
  return e->step(host_tokens, pos, nullptr, B, host_next);
}

extern "C" int gptoss_engine_step_ragged(gptoss_engine *e, const int *host_tokens, const int *host_pos, int B,
                                         int *host_next) {
  GPTOSS_REQUIRE(e && host_tokens && host_pos && host_next, GPTOSS_ERR_NULL, "engine_step_ragged: null pointer");
  GPTOSS_REQUIRE(B >= 1 && B <= e->max_batch, GPTOSS_ERR_DIM, "engine_step_ragged: batch %d outside 1..%d", B,
                 e->max_batch);
  GPTOSS_REQUIRE(!(e->precise() && e->rows == 0), GPTOSS_ERR_STATE,
                 "engine_step_ragged: not available with GPTOSS_ENGINE_PRECISE");
  int max_pos = 0;
  for (int i = 0; i < B; i++) {
    GPTOSS_REQUIRE(host_pos[i] >= 0 && host_pos[i] < e->max_seq, GPTOSS_ERR_STATE,
                   "engine_step_ragged: sequence %d at position %d outside 0..%d", i, host_pos[i], e->max_seq - 1);
    max_pos = std::max(max_pos, host_pos[i]);
  }
  return e->step(host_tokens, max_pos, host_pos, B, host_next);
}

extern "C" int gptoss_engine_prefill(gptoss_engine *e, const int *host_tokens, int B, int T, int *host_next) {
  GPTOSS_REQUIRE(e && host_tokens && host_next, GPTOSS_ERR_NULL, "engine_prefill: null pointer");
  GPTOSS_REQUIRE(e->rows > 0, GPTOSS_ERR_STATE,
                 "engine_prefill: not available (GPTOSS_ENGINE_PRECISE or GPTOSS_ENGINE_NO_PREFILL)");
  GPTOSS_REQUIRE(B >= 1 && B <= e->max_batch, GPTOSS_ERR_DIM, "engine_prefill: batch %d outside 1..%d", B, e->max_batch);
  GPTOSS_REQUIRE(T >= 1 && T <= e->max_seq && T <= e->rows, GPTOSS_ERR_DIM,
                 "engine_prefill: %d positions outside 1..%d", T, std::min(e->max_seq, e->rows));
  return e->prefill(host_tokens, B, T, host_next);
}

extern "C" int gptoss_engine_step_rows(gptoss_engine *e, int n_rows, const int *host_tokens, const int *host_slots,
                                       const int *host_pos, int n_sample, const int *host_sample, int *host_next) {
  GPTOSS_REQUIRE(e && host_tokens && host_slots && host_pos && host_sample && host_next, GPTOSS_ERR_NULL,
                 "engine_step_rows: null pointer");
  GPTOSS_REQUIRE(e->rows > 0, GPTOSS_ERR_STATE,
                 "engine_step_rows: not available (GPTOSS_ENGINE_PRECISE or GPTOSS_ENGINE_NO_PREFILL)");
  GPTOSS_REQUIRE(n_rows >= 1 && n_rows <= e->rows && n_sample >= 1 && n_sample <= e->max_batch, GPTOSS_ERR_DIM,
                 "engine_step_rows: %d rows outside 1..%d or %d sampled rows outside 1..%d", n_rows, e->rows, n_sample,
                 e->max_batch);
  GPTOSS_STEP(e->validate_rows(n_rows, host_slots, host_pos, "engine_step_rows"));
  for (int j = 0; j < n_sample; j++)
    GPTOSS_REQUIRE(host_sample[j] >= 0 && host_sample[j] < n_rows, GPTOSS_ERR_DIM,
                   "engine_step_rows: sampled row %d outside 0..%d", host_sample[j], n_rows - 1);
  return e->run_rows(n_rows, host_tokens, host_slots, host_pos, n_sample, host_sample, host_next, nullptr);
}

extern "C" int gptoss_engine_step_logits(gptoss_engine *e, int n_rows, const int *host_tokens, const int *host_slots,
                                         const int *host_pos, int n_want, const int *host_want, float *host_logits) {
  GPTOSS_REQUIRE(e && host_tokens && host_slots && host_pos && (n_want == 0 || (host_want && host_logits)),
                 GPTOSS_ERR_NULL, "engine_step_logits: null pointer");
  GPTOSS_REQUIRE(e->rows > 0, GPTOSS_ERR_STATE,
                 "engine_step_logits: not available (GPTOSS_ENGINE_PRECISE or GPTOSS_ENGINE_NO_PREFILL)");
  GPTOSS_REQUIRE(n_rows >= 1 && n_want >= 0, GPTOSS_ERR_DIM, "engine_step_logits: %d rows, %d wanted", n_rows, n_want);
  GPTOSS_STEP(e->validate_rows(n_rows, host_slots, host_pos, "engine_step_logits"));
  for (int j = 0; j < n_want; j++)
    GPTOSS_REQUIRE(host_want[j] >= 0 && host_want[j] < n_rows && (j == 0 || host_want[j] > host_want[j - 1]),
                   GPTOSS_ERR_DIM, "engine_step_logits: wanted rows must ascend within 0..%d", n_rows - 1);
  // passes of at most e->rows rows, a sequence's rows at most max_stretch() per pass
  std::vector<int> want;
  int w = 0;
  for (int lo = 0; lo < n_rows;) {
    int hi = lo, seg = lo;
    while (hi < n_rows && hi - lo < e->rows) {
      if (hi == lo || host_slots[hi] != host_slots[hi - 1]) seg = hi;
      if (hi - seg >= e->max_stretch(host_pos[seg])) break;
      hi++;
    }
    const int w0 = w;
    want.clear();
    while (w < n_want && host_want[w] < hi) want.push_back(host_want[w++] - lo);
    GPTOSS_STEP(e->run_rows(hi - lo, host_tokens + lo, host_slots + lo, host_pos + lo, (int)want.size(), want.data(),
                            nullptr, want.empty() ? nullptr : host_logits + (size_t)w0 * e->vocab));
    lo = hi;
  }
  return GPTOSS_OK;
}

extern "C" int gptoss_engine_slot_acquire(gptoss_engine *e, int *slot) {
  GPTOSS_REQUIRE(e && slot, GPTOSS_ERR_NULL, "engine_slot_acquire: null pointer");
  for (int i = 0; i < e->max_batch; i++)
    if (!e->slot_used[i]) {
      e->slot_used[i] = 1;
      *slot = i;
      return GPTOSS_OK;
    }
  return fail(GPTOSS_ERR_STATE, "engine_slot_acquire: all %d cache slots are held", e->max_batch);
}

extern "C" int gptoss_engine_slot_release(gptoss_engine *e, int slot) {
  GPTOSS_REQUIRE(e, GPTOSS_ERR_NULL, "engine_slot_release: null engine");
  GPTOSS_REQUIRE(slot >= 0 && slot < e->max_batch && e->slot_used[slot], GPTOSS_ERR_STATE,
                 "engine_slot_release: slot %d is not held", slot);
  e->slot_used[slot] = 0;
  return GPTOSS_OK;
}

extern "C" int gptoss_engine_info(gptoss_engine *e, gptoss_model_info *info) {
  GPTOSS_REQUIRE(e && info, GPTOSS_ERR_NULL, "engine_info: null pointer");
  *info = {e->vocab, e->vocab_rows, e->hidden_real, e->hidden, e->n_layers, e->max_batch, e->max_seq, e->rows};
  return GPTOSS_OK;
}

// Device view of one weight tensor in the layout the kernels read.
extern "C" int gptoss_engine_tensor_view(gptoss_engine *e, int tensor, int layer, void **ptr, size_t *bytes) {
  GPTOSS_REQUIRE(e && ptr && bytes, GPTOSS_ERR_NULL, "engine_tensor_view: null pointer");
  return e->tensor_view(tensor, layer, ptr, bytes);
}

// Device views for tests and tracing: logits of the last step [B,V] and the residual stream.
extern "C" int gptoss_engine_debug_views(gptoss_engine *e, float **logits, float **x, size_t *device_bytes) {
  GPTOSS_REQUIRE(e, GPTOSS_ERR_NULL, "engine_debug_views: null engine");
  if (logits) *logits = e->logits;
  if (x) *x = e->x;
  if (device_bytes) *device_bytes = e->device_bytes;
  return GPTOSS_OK;
}
