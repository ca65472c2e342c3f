// Nezavik: decoder layers with one norm whose output feeds a mixer and a feed-forward side by side; the
// mixer is a gated delta rule ("delta": one decay per head, "channel_delta": one per key channel) or
// sliding-window attention next to a state-space recurrence ("parallel"); what a layer passes on is a
// learned average over the embedding output and all layer results so far.
//
// Per layer the step runs
//   one GEMM for everything that reads the norm's output (mixer projections and the feed-forward's
//   up projection, rows of one packed matrix), the mixer's kernels (recurrent.hip, window_attn.hip),
//   one GEMM for everything that adds into the residual stream (mixer output and down projection,
//   columns of one packed matrix), and the depth average with the next layer's norm.
// Every size and constant comes from config.json or a tensor's shape.  With GPTOSS_ENGINE_PRECISE
// weights, activations and the K/V ring are fp32 and so is every product.
#include "model_loader.hpp"
#include "recurrent.hpp"
#include "window_attn.hpp"

namespace gptoss {

namespace {

// rows of one sequence in a pass: the window rings hold the window in front of such a stretch as well
constexpr int NEZAVIK_STRETCH = 2048;

struct NezavikLayer {
  enum Type { DELTA, CHANNEL_DELTA, PARALLEL } type = DELTA;
  float *norm = nullptr, *average = nullptr;   // [hidden], [layer + 2]
  Matrix in, low_rank, out;
  // the recurrence and what surrounds it; pointers to activations are filled in per step
  ShortConv conv;
  Scan scan;
  GatedNorm gated;
  int gate_col = 0;        // gate in the projected rows, or in the low-rank outputs
  int low_col = 0, low_width = 0, low_out = 0;   // channel_delta: [a1 | g1] columns; low_out: columns of the outputs
  WindowAttn attn;
  int up_col = 0, ff = 0;  // feed-forward (ff == 0: none); its activations are columns 0.. of the output's input
};

struct Shapes {
  int in = 0, conv = 0, y = 0, low = 0, low_out = 0, act = 0, q = 0;   // widest rows over the layers
};

}  // namespace

struct Nezavik final : gptoss_engine {
  bf16_t *embedding = nullptr, *positions = nullptr;
  float *embedding_f32 = nullptr, *positions_f32 = nullptr;
  int n_positions = 0;
  std::vector<NezavikLayer> layers;
  // activations of a pass
  Shapes wide;
  float *in_rows = nullptr, *conv_rows = nullptr, *y_rows = nullptr, *low_out_rows = nullptr, *q_rows = nullptr;
  float *branch = nullptr, *history = nullptr;   // partial sums of [rows, hidden], [layers + 1][rows, hidden]
  size_t branch_elems = 0;
  bf16_t *t_rows = nullptr;
  float *t_rows_f32 = nullptr;
  void *act_rows = nullptr, *low_rows = nullptr;

  int max_stretch(int) const override { return NEZAVIK_STRETCH; }
  int check_segments(const std::vector<RowSeg> &segs) override { return continue_slots(segs); }
  int forward_rows(const StepRows &r) override;

  int project_in(const NezavikLayer &w, int n);
  int gemm(const Matrix &m, const bf16_t *a, const float *a_f32, float *out, int n) {
    if (precise()) return precise_matmul(out, a_f32, m.f32, nullptr, nullptr, n, m.n_in, m.n_out, 1, stream);
    return dense_gemm(a, m.packed, nullptr, out, EPI_F32, n, m.n_out, m.n_in, stream);
  }
};

// Everything that reads the norm's output: mixer projections in fp32; the feed-forward's activations and
// the inner ends of the low-rank pairs go where the next products read them.
int Nezavik::project_in(const NezavikLayer &w, int n) {
  const int ld_in = w.in.n_out, ld_act = w.out.n_in, ld_low = w.low_rank.n_in;
  if (precise()) {
    GPTOSS_STEP(gemm(w.in, nullptr, t_rows_f32, in_rows, n));
    if (w.ff) GPTOSS_STEP(run_column_map(in_rows, ld_in, w.up_col, w.ff, true, (float *)act_rows, ld_act, n, stream));
    if (w.low_width)
      GPTOSS_STEP(run_column_map(in_rows, ld_in, w.low_col, w.low_width, false, (float *)low_rows, ld_low, n, stream));
    return GPTOSS_OK;
  }
  GemmBf16Range ranges[2];
  int k = 0;
  if (w.ff) ranges[k++] = {w.up_col, ld_in, (bf16_t *)act_rows, ld_act, 1};   // the last columns
  if (w.low_width) ranges[k++] = {w.low_col, w.low_col + (w.low_width + 31) / 32 * 32, (bf16_t *)low_rows, ld_low, 0};
  return dense_gemm_mixed(t_rows, w.in.packed, in_rows, ranges, k, n, ld_in, w.in.n_in, stream);
}

int Nezavik::forward_rows(const StepRows &r) {
  const int n = r.n, f32 = precise();
  hipStream_t s = stream;
  const size_t plane = (size_t)rows * hidden;
  if (f32)
    GPTOSS_STEP(run_embedding_position_f32(embedding_f32, positions_f32, r.tokens, r.lens, rows_x, history, n, hidden_real,
                                           hidden, vocab, n_positions, s));
  else
    GPTOSS_STEP(run_embedding_position(embedding, positions, r.tokens, r.lens, rows_x, history, n, hidden_real, hidden,
                                       vocab, n_positions, s));
  GPTOSS_STEP(run_rmsnorm(rows_x, nullptr, layers[0].norm, t_rows, t_rows_f32, n, hidden, s, norm_eps, hidden_real));
  for (int l = 0; l < n_layers; l++) {
    NezavikLayer &w = layers[l];
    const int ld_in = w.in.n_out, ld_act = w.out.n_in;
    GPTOSS_STEP(project_in(w, n));
    if (w.type == NezavikLayer::PARALLEL) {
      WindowAttn a = w.attn;
      a.in = in_rows;
      a.ld_in = ld_in;
      a.q = q_rows;
      a.out = act_rows;
      a.ld_out = ld_act;
      GPTOSS_STEP(run_window_attn(a, r, s));
    }
    if (w.type == NezavikLayer::CHANNEL_DELTA) {
      GPTOSS_STEP(gemm(w.low_rank, (const bf16_t *)low_rows, (const float *)low_rows, low_out_rows, n));
    }
    GPTOSS_STEP(run_short_conv(w.conv, r, in_rows, ld_in, w.scan.conv_state, conv_rows, w.conv.channels, s));
    Scan sc = w.scan;
    sc.conv = conv_rows;
    sc.ld_conv = w.conv.channels;
    sc.in = in_rows;
    sc.ld_in = ld_in;
    sc.channel_decay = low_out_rows;
    sc.ld_decay = w.low_rank.n_out;
    sc.out = y_rows;
    sc.ld_out = sc.heads * sc.V;
    sc.conv_desc = w.conv;
    GPTOSS_STEP(run_scan(sc, r, s));
    GatedNorm g = w.gated;
    g.y = y_rows;
    g.ld_y = sc.ld_out;
    g.gate = w.type == NezavikLayer::CHANNEL_DELTA ? low_out_rows + w.gate_col : in_rows + w.gate_col;
    g.ld_gate = w.type == NezavikLayer::CHANNEL_DELTA ? w.low_rank.n_out : ld_in;
    g.out = act_rows;
    g.ld_out = ld_act;
    g.out_f32 = f32;
    GPTOSS_STEP(run_gated_norm(g, n, s));
    int parts = 1;
    if (f32) GPTOSS_STEP(gemm(w.out, nullptr, (const float *)act_rows, branch, n));
    else
      GPTOSS_STEP(dense_gemm_partial((const bf16_t *)act_rows, w.out.packed, branch, branch_elems, &parts, n, w.out.n_out,
                                     w.out.n_in, s));
    const float *next_norm = l + 1 < n_layers ? layers[l + 1].norm : nullptr;   // the sampled rows are normed later
    GPTOSS_STEP(run_depth_average_norm(rows_x, branch, parts, history, plane, w.average, l, next_norm, t_rows, t_rows_f32, n,
                                       hidden, norm_eps, hidden_real, s));
  }
  return GPTOSS_OK;
}

namespace {

using Part = Loader::Part;

void check_scan(const Scan &s, const ShortConv &c, int i) {
  require(s.heads % s.key_heads == 0, "heads must be a multiple of kv_heads (or groups)", i);
  require(s.K <= SCAN_MAX_KEY, "key or state dimensions above 256 are not supported", i);
  require(s.heads < 65535 && c.taps <= 64, "too many heads or convolution taps", i);
}

void scan_state(Loader &ld, NezavikLayer &w, const std::string &p) {
  gptoss_engine *e = ld.e;
  Scan &s = w.scan;
  s.state = ld.zeros((size_t)e->max_batch * scan_state_elems(s.heads, s.K, s.V));
  s.conv_state = ld.zeros((size_t)e->max_batch * (w.conv.taps - 1) * w.conv.channels);
  // e.g. random weights: decays exp(-exp(A_log) softplus(dt)) of the order of 0.9
  s.a_log = ld.vec(p + ".A_log", {s.heads}, -2.f, 0.5f);
  const int n_dt = s.kind == SCAN_CHANNEL_DELTA ? s.heads * s.K : s.heads;
  s.dt_bias = ld.vec(p + ".dt_bias", {n_dt}, 0.f, 0.5f);
}

// q, k, v with their short convolutions, unit vectors, write strength and output norm of the delta rules
void load_delta(Loader &ld, NezavikLayer &w, const Json &mix, const std::string &p, int i, Columns &cols,
                std::vector<Part> &parts) {
  Scan &s = w.scan;
  const int W = ld.e->hidden_real;
  s.kind = w.type == NezavikLayer::DELTA ? SCAN_DELTA : SCAN_CHANNEL_DELTA;
  s.heads = size_of(mix, "heads");
  s.key_heads = size_of(mix, "kv_heads");
  s.K = size_of(mix, "dim");
  s.V = size_of(mix, "vdim");
  const int nk = s.key_heads * s.K, nv = s.heads * s.V;
  w.conv.taps = size_of(mix, "conv");
  w.conv.channels = 2 * nk + nv;
  w.conv.n_unit = s.key_heads;
  w.conv.unit_dim = s.K;
  w.conv.unit_scale = 1.f / sqrtf((float)s.K);
  check_scan(s, w.conv, i);
  w.conv.col = cols.take(w.conv.channels);
  parts.push_back({p + ".q", nk, W, w.conv.col, 0});
  parts.push_back({p + ".k", nk, W, w.conv.col + nk, 0});
  parts.push_back({p + ".v", nv, W, w.conv.col + 2 * nk, 0});
  s.q_col = 0;
  s.k_col = nk;
  s.v_col = 2 * nk;
  if (ld.st) {
    std::vector<float> taps;
    for (const auto &part : {std::make_pair(".q.conv", nk), std::make_pair(".k.conv", nk), std::make_pair(".v.conv", nv)}) {
      const std::vector<float> v = ld.host(p + part.first, {part.second, w.conv.taps});
      taps.insert(taps.end(), v.begin(), v.end());
    }
    w.conv.weight = ld.b.upload_f32(taps.data(), taps.size(), 0, 0, 0);
  } else {
    w.conv.weight = ld.vec("", {w.conv.channels, w.conv.taps}, 0.f, 0.5f);
  }
  s.beta_col = cols.take(s.heads);
  parts.push_back({p + ".b", s.heads, W, s.beta_col, 0});
  scan_state(ld, w, p);
  w.gated.groups = s.heads;
  w.gated.size = s.V;
  w.gated.weight = ld.vec(p + ".norm", {s.V}, 1.f, 0.02f);
  w.gated.eps = ld.e->norm_eps;
}

void load_state_space(Loader &ld, NezavikLayer &w, const Json &mix, const std::string &p, int i, Columns &cols,
                      std::vector<Part> &parts) {
  Scan &s = w.scan;
  s.kind = SCAN_STATE_SPACE;
  s.heads = size_of(mix, "heads");
  s.key_heads = size_of(mix, "groups");
  s.K = size_of(mix, "state");
  s.V = size_of(mix, "vdim");
  const int inner = s.heads * s.V, gn = s.key_heads * s.K;
  w.conv.taps = size_of(mix, "conv");
  w.conv.channels = inner + 2 * gn;
  check_scan(s, w.conv, i);
  const int norm_groups = size_of(mix, "norm_groups");
  require(inner % norm_groups == 0, "norm_groups must divide heads * vdim", i);
  const int all = 2 * inner + 2 * gn + s.heads, base = cols.take(all);
  parts.push_back({p + ".in", all, ld.e->hidden_real, base, 0});
  w.gate_col = base;
  w.conv.col = base + inner;
  s.v_col = 0;          // columns of the convolved rows: x, B, C
  s.k_col = inner;
  s.q_col = inner + gn;
  s.decay_col = base + 2 * inner + 2 * gn;
  w.conv.weight = ld.vec(p + ".conv", {w.conv.channels, w.conv.taps}, 0.f, 0.5f);
  w.conv.bias = ld.vec(p + ".conv.b", {w.conv.channels}, 0.f, 0.1f);
  s.d_skip = ld.vec(p + ".D", {s.heads}, 1.f, 0.1f);
  scan_state(ld, w, p);
  w.gated.groups = norm_groups;
  w.gated.size = inner / norm_groups;
  w.gated.weight = ld.vec(p + ".norm", {inner}, 1.f, 0.02f);
  w.gated.weight_per_group = 1;
  w.gated.gate_first = 1;
  w.gated.eps = ld.e->norm_eps;
}

void load_window(Loader &ld, NezavikLayer &w, const Json &mix, const std::string &p, int i, Columns &cols,
                 std::vector<Part> &parts) {
  gptoss_engine *e = ld.e;
  WindowAttn &a = w.attn;
  a.heads = size_of(mix, "heads");
  a.kv_heads = size_of(mix, "kv_heads");
  a.dim = size_of(mix, "dim");
  a.vdim = size_of(mix, "vdim");
  a.scale = (float)number(mix, "scale");
  a.window = size_of(field(mix, "mask", Json::OBJECT), "size");
  a.eps = e->norm_eps;
  require(a.heads % a.kv_heads == 0, "heads must be a multiple of kv_heads", i);
  require(a.dim <= WINDOW_ATTN_MAX_DIM && a.vdim <= WINDOW_ATTN_MAX_DIM, "head sizes above 256 are not supported", i);
  a.q_col = cols.take(a.heads * a.dim);
  a.k_col = cols.take(a.kv_heads * a.dim);
  a.v_col = cols.take(a.kv_heads * a.vdim);
  parts.push_back({p + ".q", a.heads * a.dim, e->hidden_real, a.q_col, 0});
  parts.push_back({p + ".k", a.kv_heads * a.dim, e->hidden_real, a.k_col, 0});
  parts.push_back({p + ".v", a.kv_heads * a.vdim, e->hidden_real, a.v_col, 0});
  a.q_norm = ld.vec(p + ".q.norm", {a.dim}, 1.f, 0.02f);
  a.k_norm = ld.vec(p + ".k.norm", {a.dim}, 1.f, 0.02f);
  window_attn_cache(ld, a, NEZAVIK_STRETCH);
}

void load_layer(Loader &ld, NezavikLayer &w, const Json &j, int i) {
  Nezavik *e = static_cast<Nezavik *>(ld.e);
  const int W = e->hidden_real;
  const std::string l = "l" + std::to_string(i), p = l + ".mix";
  const std::string &type = field(j, "type", Json::STRING).text;
  const Json &mix = field(j, "mixer", Json::OBJECT);
  const Json *mlp = j.find("mlp");
  if (mlp && mlp->is(Json::NUL)) mlp = nullptr;
  if (mlp) {
    require(mlp->is(Json::OBJECT) && field(*mlp, "kind", Json::STRING).text == "dense", "unknown kind of feed-forward", i);
    w.ff = size_of(*mlp, "ff");
  }
  w.norm = ld.scalar_norm(l + ".norm1");
  w.average = ld.vec(l + ".dwa", {i + 2}, 1.f / (i + 2), 0.02f);
  Columns cols;                    // of the projected rows
  std::vector<Part> in_parts, out_parts;
  Columns act;                     // of the output projection's input rows
  if (w.ff) {
    out_parts.push_back({l + ".mlp.down", W, w.ff, 0, act.take(w.ff)});
    act.align();
  }
  auto mixer_out = [&](const std::string &name, int width) {
    const int c = act.take(width);
    out_parts.push_back({name, W, width, 0, c});
    act.used = (act.used + 3) / 4 * 4;
    return c;
  };
  if (type == "delta") {
    w.type = NezavikLayer::DELTA;
    load_delta(ld, w, mix, p, i, cols, in_parts);
    w.scan.decay_col = cols.take(w.scan.heads);
    in_parts.push_back({p + ".a", w.scan.heads, W, w.scan.decay_col, 0});
    w.gate_col = cols.take(w.scan.heads * w.scan.V);
    in_parts.push_back({p + ".g", w.scan.heads * w.scan.V, W, w.gate_col, 0});
    w.gated.out_col = mixer_out(p + ".o", w.scan.heads * w.scan.V);
  } else if (type == "channel_delta") {
    w.type = NezavikLayer::CHANNEL_DELTA;
    load_delta(ld, w, mix, p, i, cols, in_parts);
    w.gated.sigmoid_gate = 1;
    // decays and gates go through low-rank pairs; both second halves are one block-diagonal matrix
    const int nk = w.scan.heads * w.scan.K, nv = w.scan.heads * w.scan.V;
    int ra = std::min(W, 128), rg = ra;
    if (ld.st) {
      const SafeTensors::Tensor *a1 = ld.st->find(p + ".a1"), *g1 = ld.st->find(p + ".g1");
      require(a1 && g1 && a1->shape.size() == 2 && g1->shape.size() == 2, "the low-rank projections a1 and g1 are missing", i);
      ra = (int)a1->shape[0];
      rg = (int)g1->shape[0];
    }
    cols.align();
    w.low_width = ra + rg;
    w.low_col = cols.take(w.low_width);
    in_parts.push_back({p + ".a1", ra, W, w.low_col, 0});
    in_parts.push_back({p + ".g1", rg, W, w.low_col + ra, 0});
    w.gate_col = (nk + 3) / 4 * 4;
    w.low_rank = ld.matrix(up32(w.gate_col + nv), up64(w.low_width),
                           {{p + ".a2", nk, ra, 0, 0}, {p + ".g2", nv, rg, w.gate_col, ra}});
    w.gated.out_col = mixer_out(p + ".o", nv);
  } else if (type == "parallel") {
    w.type = NezavikLayer::PARALLEL;
    const Json &left = field(mix, "left", Json::OBJECT), &right = field(mix, "right", Json::OBJECT);
    load_window(ld, w, left, p + ".left", i, cols, in_parts);
    load_state_space(ld, w, right, p + ".right", i, cols, in_parts);
    // both scales are applied to the output projections' inputs
    w.attn.out_scale = (float)number(mix, "left_scale");
    w.gated.scale = (float)number(mix, "right_scale");
    w.attn.out_col = mixer_out(p + ".left.o", w.attn.heads * w.attn.vdim);
    w.gated.out_col = mixer_out(p + ".right.o", w.scan.heads * w.scan.V);
  } else {
    throw ConfigError{fail(GPTOSS_ERR_IO, "config.json: layer %d has the unknown type \"%s\"", i, type.c_str())};
  }
  cols.align();
  if (w.ff) {
    w.up_col = cols.take(w.ff);
    in_parts.push_back({l + ".mlp.up", w.ff, W, w.up_col, 0});
    cols.align();
  }
  w.in = ld.matrix(cols.used, e->hidden, in_parts);
  w.out = ld.matrix(e->hidden, up64(act.used), out_parts);
  Shapes &x = e->wide;
  x.in = std::max(x.in, w.in.n_out);
  x.conv = std::max(x.conv, w.conv.channels);
  x.y = std::max(x.y, w.scan.heads * w.scan.V);
  x.low = std::max(x.low, w.low_rank.n_in);
  x.low_out = std::max(x.low_out, w.low_rank.n_out);
  x.act = std::max(x.act, w.out.n_in);
  x.q = std::max(x.q, w.attn.heads * w.attn.dim_pad());
}

void load_model(Nezavik *e, Builder &b, const ModelSource &src, uint64_t seed) {
  const Json &cfg = *src.config;
  Loader ld{e, b, src.weights, seed * 1000003ull + 29};
  const Json &list = field(cfg, "layers", Json::ARRAY);
  const int V = e->vocab, W = e->hidden_real;
  ld.table("embed", V, W, W, 1.f, &e->embedding, &e->embedding_f32);
  ld.table("pos", e->n_positions, W, W, 1.f, &e->positions, &e->positions_f32);
  e->layers.resize(list.items.size());
  for (size_t i = 0; i < list.items.size() && b.ok(); i++) load_layer(ld, e->layers[i], list.items[i], (int)i);
  e->final_norm = ld.scalar_norm("final.norm");
  const Matrix head = ld.matrix(e->vocab_rows, e->hidden, {{"head", V, W, 0, 0}});
  e->unembedding = head.packed;
  e->unembedding_f32 = head.f32;
  e->class_bias = ld.class_bias();
}

// largest matrix of the model in elements (the staging buffers hold one), from the configuration alone
size_t staging_elems(const Json &cfg, int hidden, int vocab_rows) {
  double widest = vocab_rows;
  for (const Json &l : field(cfg, "layers", Json::ARRAY).items) {
    double sum = 256;
    auto add = [&](const Json &m) {
      auto v = [&](const char *k) {
        const Json *x = m.find(k);
        return x && x->is(Json::NUMBER) ? x->number : 0.0;
      };
      sum += (v("heads") + v("kv_heads")) * (2 * v("dim") + 3 * v("vdim") + 2) + 2 * v("groups") * v("state") + v("ff");
      return v("heads") * (v("dim") + v("vdim")) + v("ff");
    };
    for (const char *k : {"mixer", "mlp"})
      if (const Json *m = l.find(k)) {
        add(*m);
        for (const char *side : {"left", "right"})
          if (const Json *x = m->find(side)) add(*x);
      }
    sum += 2.0 * hidden;   // the low-rank pairs
    widest = std::max(widest, sum);
  }
  // low-rank matrices are [heads * (dim + vdim), rank]: their rank is bounded by the width
  return std::max<size_t>((size_t)1 << 20, (size_t)(widest + 128) * hidden);
}

int open_nezavik(const ModelSource &src, const OpenOptions &o, gptoss_engine **out) {
  const bool synthetic = src.weights == nullptr;
  GPTOSS_REQUIRE(!(o.flags & (GPTOSS_ENGINE_NO_PREFILL | GPTOSS_ENGINE_MXFP4_EXPERTS)), GPTOSS_ERR_STATE,
                 "Nezavik: GPTOSS_ENGINE_NO_PREFILL and GPTOSS_ENGINE_MXFP4_EXPERTS do not apply");
  GPTOSS_REQUIRE(!(synthetic && (o.flags & GPTOSS_ENGINE_PRECISE)), GPTOSS_ERR_STATE,
                 "Nezavik: GPTOSS_ENGINE_PRECISE needs weights");
  Nezavik *e = new Nezavik();
  Builder b;
  b.e = e;
  try {
    const Json &cfg = *src.config;
    e->vocab = size_of(cfg, "vocab");
    e->vocab_rows = up64(e->vocab);
    e->hidden_real = size_of(cfg, "width");
    e->hidden = up64(e->hidden_real);
    e->n_positions = size_of(cfg, "max_positions");
    e->norm_eps = (float)number(field(cfg, "norm", Json::OBJECT), "eps");
    e->n_layers = (int)field(cfg, "layers", Json::ARRAY).items.size();
    if (e->n_layers < 1) throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: no layers")};
    if (e->hidden > 16384) throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: widths above 16384 are not supported")};
    e->max_batch = o.max_batch;
    e->max_seq = o.max_seq > 0 ? std::min(o.max_seq, e->n_positions) : e->n_positions;
    e->flags = o.flags;
    e->slot_used.assign(o.max_batch, 0);
    e->lengths.assign(o.max_batch, 0);
    b.hip(hipStreamCreate(&e->stream), "hipStreamCreate");
    b.stage_elems = staging_elems(cfg, e->hidden, e->vocab_rows);
    if (!synthetic) b.stager_create(b.stage_elems);
    else b.hip(hipMalloc((void **)&b.stage_bf16, b.stage_elems * sizeof(bf16_t)), "staging hipMalloc");
    if (b.ok()) load_model(e, b, src, o.seed);
  } catch (const ConfigError &err) {
    b.rc = err.rc;
  }
  if (e->stream) (void)hipStreamSynchronize(e->stream);
  b.stager_destroy();
  if (b.stage_bf16) (void)hipFree(b.stage_bf16);
  if (b.ok()) {
    const int R = (int)std::min<long long>((long long)o.max_batch * e->max_seq, PREFILL_ROWS);
    const size_t elem = e->precise() ? sizeof(float) : sizeof(bf16_t);
    b.check(e->create_rows(R));
    if (b.ok()) b.check(e->create_sampling());
    e->in_rows = b.alloc<float>((size_t)R * e->wide.in);
    e->conv_rows = b.alloc<float>((size_t)R * e->wide.conv);
    e->y_rows = b.alloc<float>((size_t)R * e->wide.y);
    e->low_out_rows = b.alloc<float>((size_t)R * e->wide.low_out);
    e->q_rows = b.alloc<float>((size_t)R * e->wide.q);
    // room for every part of the output projection's sum while the rows are few
    e->branch_elems = std::max((size_t)R * e->hidden, std::min<size_t>((size_t)R * e->hidden * GEMM_MAX_PARTS, (size_t)32 << 20));
    e->branch = b.alloc<float>(e->branch_elems);
    e->history = b.alloc<float>((size_t)R * e->hidden * (e->n_layers + 1));
    e->t_rows = b.alloc<bf16_t>((size_t)R * e->hidden);
    if (e->precise()) e->t_rows_f32 = b.alloc<float>((size_t)R * e->hidden);
    e->low_rows = b.alloc<unsigned char>((size_t)R * e->wide.low * elem);
    e->act_rows = b.alloc<unsigned char>((size_t)R * e->wide.act * elem);
    // padding columns are multiplied by zero weights, but must hold finite values
    if (b.ok()) b.hip(hipMemsetAsync(e->low_rows, 0, (size_t)R * e->wide.low * elem, e->stream), "memset");
    if (b.ok()) b.hip(hipMemsetAsync(e->act_rows, 0, (size_t)R * e->wide.act * elem, e->stream), "memset");
    if (b.ok()) b.hip(hipStreamSynchronize(e->stream), "sync");
  }
  if (!b.ok()) {
    delete e;
    return b.rc;
  }
  *out = e;
  return GPTOSS_OK;
}

const ModelClass nezavik_class("Nezavik", open_nezavik);

}  // namespace

}  // namespace gptoss
