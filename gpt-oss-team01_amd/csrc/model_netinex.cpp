// Netinex: pre-norm decoder layers whose mixer is retention (linear attention with a fixed decay per head) or
// chunked attention whose values are its keys as projected, each followed by a mixture of experts; norms are
// dynamic tanh, positions rotary, the classifier is the embedding table and its logits are soft-capped.
//
// Per layer the step runs
//   one GEMM for the mixer's projections (rows of one packed matrix), the mixer's kernels (retention.hip,
//   recurrent.hip / window_attn.hip), the output GEMM, the residual sum with the feed-forward's norm, the
//   MoE block (moe_layer.cpp), whose combine adds into the residual stream and norms it for the next layer.
// Every size and constant comes from config.json.  With GPTOSS_ENGINE_PRECISE weights, activations and the
// K/V ring are fp32 and so is every product.
#include "model_loader.hpp"
#include "recurrent.hpp"
#include "rotary.hpp"
#include "window_attn.hpp"

namespace gptoss {

namespace {

// rows of one sequence in a pass: the rings hold the chunk in front of such a stretch as well
constexpr int NETINEX_STRETCH = 2048;
// positions of a sequence where the caller names no limit (the design has none; the rotary tables do)
constexpr int NETINEX_POSITIONS = 8192;

struct NetinexLayer {
  enum Type { RETENTION, ATTENTION } type = RETENTION;
  TanhNorm norm1, norm2;
  Matrix in, out;
  // retention; pointers to activations are filled in per step
  Scan scan;
  GatedNorm gated;
  int gate_col = 0;
  WindowAttn attn;
  // mixture of experts (moe.n_experts == 0: no feed-forward); fp32 weights with GPTOSS_ENGINE_PRECISE
  gptoss_moe_weights moe = {};
  const float *router_f32 = nullptr, *w1_f32 = nullptr, *w2_f32 = nullptr;
};

struct Shapes {
  int in = 0, y = 0, act = 0, q = 0;              // widest rows over the layers
  size_t moe = 0, logits = 0, pairs_i = 0, pairs_h = 0, pairs = 0;   // of a pass of `rows` rows
};

}  // namespace

struct Netinex final : gptoss_engine {
  bf16_t *embedding = nullptr;
  float *embedding_f32 = nullptr;
  std::vector<NetinexLayer> layers;
  TanhNorm last_norm;
  std::vector<std::pair<RotarySpec, const float *>> tables;   // rotary tables, shared by layers of one spec
  // activations of a pass
  Shapes wide;
  float *in_rows = nullptr, *y_rows = nullptr, *q_rows = nullptr, *branch = nullptr;
  size_t branch_elems = 0;
  bf16_t *t_rows = nullptr;
  float *t_rows_f32 = nullptr;
  void *act_rows = nullptr, *moe_ws = nullptr;
  struct {   // GPTOSS_ENGINE_PRECISE
    float *logits = nullptr, *topk_w = nullptr, *up = nullptr, *act = nullptr, *down = nullptr;
    int *topk_i = nullptr;
  } pr;

  int max_stretch(int) const override { return NETINEX_STRETCH; }
  int check_segments(const std::vector<RowSeg> &segs) override { return continue_slots(segs); }
  int forward_rows(const StepRows &r) override;
  int norm_sampled(int m) override { return run_residual_tanh_norm(x, nullptr, 0, last_norm, t, t_f32, m, hidden, stream); }

  int mix(NetinexLayer &w, const StepRows &r);
  int feed_forward(const NetinexLayer &w, const TanhNorm &next, int n);
};

// Projected rows -> input rows of the output projection.
int Netinex::mix(NetinexLayer &w, const StepRows &r) {
  const int ld_in = w.in.n_out, ld_act = w.out.n_in;
  if (w.type == NetinexLayer::ATTENTION) {
    WindowAttn a = w.attn;
    a.in = in_rows;
    a.ld_in = ld_in;
    a.q = q_rows;
    a.out = act_rows;
    a.ld_out = ld_act;
    return run_window_attn(a, r, stream);
  }
  Scan sc = w.scan;
  sc.conv = sc.in = in_rows;
  sc.ld_conv = sc.ld_in = ld_in;
  sc.out = y_rows;
  sc.ld_out = sc.heads * sc.V;
  GPTOSS_STEP(run_retention(sc, r, precise(), in_rows, stream));
  GatedNorm g = w.gated;
  g.y = y_rows;
  g.ld_y = sc.ld_out;
  g.gate = in_rows + w.gate_col;
  g.ld_gate = ld_in;
  g.out = act_rows;
  g.ld_out = ld_act;
  g.out_f32 = precise();
  return run_gated_norm(g, r.n, stream);
}

// rows_x += experts(t_rows); t_rows = next(rows_x) where there is a next norm.
int Netinex::feed_forward(const NetinexLayer &w, const TanhNorm &next, int n) {
  const GluForm silu{1.f, 0.f, INFINITY};
  if (!precise()) return moe_forward_glu(&w.moe, silu, t_rows, n, rows_x, moe_ws, wide.moe, stream, next, t_rows);
  const int E = w.moe.n_experts, k = w.moe.top_k, I = w.moe.intermediate, pairs = n * k;
  GPTOSS_STEP(precise_matmul(pr.logits, t_rows_f32, w.router_f32, w.moe.b_router, nullptr, n, hidden, E, 1, stream));
  GPTOSS_STEP(run_topk_softmax(pr.logits, n, E, k, pr.topk_w, pr.topk_i, stream));
  GPTOSS_STEP(precise_matmul(pr.up, t_rows_f32, w.w1_f32, nullptr, pr.topk_i, pairs, hidden, 2 * I, k, stream));
  GPTOSS_STEP(precise_swiglu(pr.up, pr.act, pairs, I, silu, stream));
  GPTOSS_STEP(precise_matmul(pr.down, pr.act, w.w2_f32, nullptr, pr.topk_i, pairs, I, hidden, 1, stream));
  GPTOSS_STEP(precise_moe_agg(pr.down, pr.topk_w, pr.topk_i, rows_x, n, hidden, k, stream));
  return next.weight ? run_residual_tanh_norm(rows_x, nullptr, 0, next, t_rows, t_rows_f32, n, hidden, stream) : GPTOSS_OK;
}

int Netinex::forward_rows(const StepRows &r) {
  const int n = r.n;
  hipStream_t s = stream;
  if (precise())
    GPTOSS_STEP(run_embedding_position_f32(embedding_f32, nullptr, r.tokens, r.lens, rows_x, nullptr, n, hidden_real, hidden,
                                           vocab, 1, s));
  else
    GPTOSS_STEP(run_embedding_position(embedding, nullptr, r.tokens, r.lens, rows_x, nullptr, n, hidden_real, hidden, vocab, 1, s));
  GPTOSS_STEP(run_residual_tanh_norm(rows_x, nullptr, 0, layers[0].norm1, t_rows, t_rows_f32, n, hidden, s));
  for (int l = 0; l < n_layers; l++) {
    NetinexLayer &w = layers[l];
    if (precise()) GPTOSS_STEP(precise_matmul(in_rows, t_rows_f32, w.in.f32, nullptr, nullptr, n, w.in.n_in, w.in.n_out, 1, s));
    else GPTOSS_STEP(dense_gemm(t_rows, w.in.packed, nullptr, in_rows, EPI_F32, n, w.in.n_out, w.in.n_in, s));
    GPTOSS_STEP(mix(w, r));
    int parts = 1;
    if (precise())
      GPTOSS_STEP(precise_matmul(branch, (const float *)act_rows, w.out.f32, nullptr, nullptr, n, w.out.n_in, w.out.n_out, 1, s));
    else
      GPTOSS_STEP(dense_gemm_partial((const bf16_t *)act_rows, w.out.packed, branch, branch_elems, &parts, n, w.out.n_out,
                                     w.out.n_in, s));
    // the sampled rows are normed later
    const TanhNorm next = l + 1 < n_layers ? layers[l + 1].norm1 : TanhNorm();
    const bool ff = w.moe.n_experts > 0;
    GPTOSS_STEP(run_residual_tanh_norm(rows_x, branch, parts, ff ? w.norm2 : next, t_rows, t_rows_f32, n, hidden, s));
    if (ff) GPTOSS_STEP(feed_forward(w, next, n));
  }
  return GPTOSS_OK;
}

namespace {

using Part = Loader::Part;

TanhNorm load_norm(Loader &ld, const std::string &name) {
  TanhNorm n;
  n.weight = ld.column_vec(name, 1.f);
  n.bias = ld.column_vec(name + ".b", 0.f);
  n.alpha = ld.scalar(name + ".alpha", 0.5f);
  return n;
}

Rotary load_rotary(Loader &ld, const Json &mix, int dim, bool interleaved, int i) {
  Netinex *e = static_cast<Netinex *>(ld.e);
  const Json &rot = field(mix, "rot", Json::OBJECT);
  RotarySpec spec;
  spec.dims = size_of(rot, "dims");
  spec.base = number(rot, "base");
  require(spec.dims % 2 == 0 && spec.dims <= dim && spec.base > 1.0, "rotary positions need an even number of dimensions within the head", i);
  const Json *sc = rot.find("scaling");
  if (sc && !sc->is(Json::NUL)) {
    require(sc->is(Json::OBJECT), "\"scaling\" must be an object", i);
    spec.factor = number(*sc, "factor");
    spec.original = number(*sc, "original");
    spec.fast = number(*sc, "fast");
    spec.slow = number(*sc, "slow");
    require(spec.factor > 0 && spec.original > 0 && spec.fast > 0 && spec.slow > 0, "constants of the scaling must be positive", i);
  }
  Rotary r;
  r.dims = spec.dims;
  r.interleaved = interleaved;
  for (const auto &t : e->tables)
    if (t.first == spec) r.table = t.second;
  if (!r.table) {
    r.table = ld.put(rotary_table(spec, e->max_seq));
    e->tables.push_back({spec, r.table});
  }
  return r;
}

void load_retention(Loader &ld, NetinexLayer &w, const Json &mix, const std::string &p, int i) {
  gptoss_engine *e = ld.e;
  const int W = e->hidden_real;
  Scan &s = w.scan;
  s.kind = SCAN_RETENTION;
  s.heads = s.key_heads = size_of(mix, "heads");
  s.K = size_of(mix, "dim");
  s.V = size_of(mix, "vdim");
  require(s.K <= SCAN_MAX_KEY, "key dimensions above 256 are not supported", i);
  s.rot = load_rotary(ld, mix, s.K, false, i);
  s.value_scale = 1.f / sqrtf((float)s.K);   // of the keys; what is written is linear in both
  const int nk = s.heads * s.K, nv = s.heads * s.V;
  const Json &decay = field(mix, "decay", Json::ARRAY);
  require((int)decay.items.size() == s.heads, "\"decay\" must name one number per head", i);
  std::vector<float> d;
  for (const Json &x : decay.items) {
    require(x.is(Json::NUMBER), "\"decay\" must name one number per head", i);
    d.push_back((float)x.number);
  }
  s.head_decay = ld.put(d);
  std::vector<float> powers;
  for (float x : d) {
    double power = 1.0;
    for (int t = 0; t <= RETENTION_CHUNK; t++, power *= x) powers.push_back((float)power);
  }
  s.decay_powers = ld.put(powers);
  Columns cols;
  s.q_col = cols.take(nk);
  s.k_col = cols.take(nk);
  cols.align(4);
  s.v_col = cols.take(nv);
  cols.align(4);
  w.gate_col = cols.take(nv);
  cols.align();
  w.in = ld.matrix(cols.used, e->hidden,
                   {{p + ".q", nk, W, s.q_col, 0}, {p + ".k", nk, W, s.k_col, 0}, {p + ".v", nv, W, s.v_col, 0},
                    {p + ".g", nv, W, w.gate_col, 0}});
  w.out = ld.matrix(e->hidden, up64(nv), {{p + ".o", W, nv, 0, 0}});
  s.state = ld.zeros((size_t)e->max_batch * scan_state_elems(s.heads, s.K, s.V));
  w.gated.groups = s.heads;
  w.gated.size = s.V;
  w.gated.eps = e->norm_eps;
}

void load_attention(Loader &ld, NetinexLayer &w, const Json &mix, const std::string &p, int i) {
  gptoss_engine *e = ld.e;
  const int W = e->hidden_real;
  WindowAttn &a = w.attn;
  a.heads = size_of(mix, "heads");
  a.kv_heads = size_of(mix, "kv_heads");
  a.dim = size_of(mix, "dim");
  a.vdim = size_of(mix, "vdim");
  a.scale = (float)number(mix, "scale");
  a.window = size_of(field(mix, "mask", Json::OBJECT), "size");
  a.chunked = a.whole_norm = 1;
  a.eps = e->norm_eps;
  require(a.heads % a.kv_heads == 0, "heads must be a multiple of kv_heads", i);
  require(a.dim <= WINDOW_ATTN_MAX_DIM, "head sizes above 256 are not supported", i);
  require(a.dim == a.vdim, "the values are the keys: dim and vdim must be equal", i);
  a.rot = load_rotary(ld, mix, a.dim, true, i);
  const int nq = a.heads * a.dim, nk = a.kv_heads * a.dim;
  Columns cols;
  a.q_col = cols.take(nq);
  cols.align(4);
  a.k_col = a.v_col = cols.take(nk);
  cols.align();
  w.in = ld.matrix(cols.used, e->hidden, {{p + ".q", nq, W, a.q_col, 0}, {p + ".k", nk, W, a.k_col, 0}});
  w.out = ld.matrix(e->hidden, up64(nq), {{p + ".o", W, nq, 0, 0}});
  a.q_norm = ld.vec(p + ".q.norm", {nq}, 1.f, 0.02f);
  a.k_norm = ld.vec(p + ".k.norm", {nk}, 1.f, 0.02f);
  window_attn_cache(ld, a, NETINEX_STRETCH);
}

void load_experts(Loader &ld, NetinexLayer &w, const Json &mlp, const std::string &p, int i) {
  gptoss_engine *e = ld.e;
  const int W = e->hidden_real;
  require(field(mlp, "kind", Json::STRING).text == "moe", "unknown kind of feed-forward", i);
  const Json &router = field(mlp, "router", Json::OBJECT);
  const int E = size_of(router, "experts"), k = size_of(router, "top"), ff = size_of(field(mlp, "expert", Json::OBJECT), "ff");
  require(E <= 256 && k <= E && k <= MOE_MAX_TOP, "at most 256 experts, of which a token uses at most 32", i);
  const int I = up64(ff);
  gptoss_moe_weights &m = w.moe;
  m.n_experts = E;
  m.top_k = k;
  m.hidden = e->hidden;
  m.intermediate = I;
  m.swiglu_limit = INFINITY;
  std::vector<std::vector<Part>> first, second;   // gate and up rows in turn; padding gives silu(0) * 0
  for (int x = 0; x < E; x++) {
    const std::string ex = p + ".e" + std::to_string(x);
    first.push_back({{ex + ".gate", ff, W, 0, 0, 2}, {ex + ".up", ff, W, 1, 0, 2}});
    second.push_back({{ex + ".down", W, ff, 0, 0}});
  }
  const Matrix w1 = ld.matrices(2 * I, e->hidden, first, GPTOSS_PACK_GLU), w2 = ld.matrices(e->hidden, I, second, 0);
  bf16_t *r16 = nullptr;
  float *r32 = nullptr;
  ld.table(p + ".router", E, W, e->hidden, 1.f / sqrtf((float)W), &r16, &r32);
  m.w_router = r16;
  m.b_router = ld.vec(p + ".router.b", {E}, 0.f, 0.02f);
  m.w1 = w1.packed;
  m.w2 = w2.packed;
  w.router_f32 = r32;
  w.w1_f32 = w1.f32;
  w.w2_f32 = w2.f32;
}

void load_layer(Loader &ld, NetinexLayer &w, const Json &j, int i) {
  Netinex *e = static_cast<Netinex *>(ld.e);
  const std::string l = "l" + std::to_string(i), p = l + ".mix";
  const std::string &type = field(j, "type", Json::STRING).text;
  const Json &mix = field(j, "mixer", Json::OBJECT);
  w.norm1 = load_norm(ld, l + ".norm1");
  if (type == "retention") {
    w.type = NetinexLayer::RETENTION;
    load_retention(ld, w, mix, p, i);
  } else if (type == "attention") {
    w.type = NetinexLayer::ATTENTION;
    load_attention(ld, w, mix, p, i);
  } else {
    throw ConfigError{fail(GPTOSS_ERR_IO, "config.json: layer %d has the unknown type \"%s\"", i, type.c_str())};
  }
  const Json *mlp = j.find("mlp");
  if (mlp && !mlp->is(Json::NUL)) {
    require(mlp->is(Json::OBJECT), "\"mlp\" must be an object or null", i);
    w.norm2 = load_norm(ld, l + ".norm2");
    load_experts(ld, w, *mlp, l + ".mlp", i);
  }
  Shapes &x = e->wide;
  x.in = std::max(x.in, w.in.n_out);
  x.y = std::max(x.y, w.scan.heads * w.scan.V);
  x.act = std::max(x.act, w.out.n_in);
  x.q = std::max(x.q, w.attn.heads * w.attn.dim_pad());
}

void load_model(Netinex *e, Builder &b, const ModelSource &src, uint64_t seed) {
  const Json &list = field(*src.config, "layers", Json::ARRAY);
  Loader ld{e, b, src.weights, seed * 1000003ull + 31};
  ld.table("embed", e->vocab, e->hidden_real, e->hidden_real, 1.f, &e->embedding, &e->embedding_f32);
  e->layers.resize(list.items.size());
  for (size_t i = 0; i < list.items.size() && b.ok(); i++) load_layer(ld, e->layers[i], list.items[i], (int)i);
  e->last_norm = load_norm(ld, "final.norm");
  const Matrix head = ld.matrix(e->vocab_rows, e->hidden, {{"embed", e->vocab, e->hidden_real, 0, 0}});
  e->unembedding = head.packed;
  e->unembedding_f32 = head.f32;
  e->class_bias = ld.class_bias();
}

// largest matrix of the model in elements (the staging buffers hold one), from the configuration alone
size_t staging_elems(const Json &cfg, int hidden, int vocab_rows) {
  double widest = vocab_rows;
  for (const Json &l : field(cfg, "layers", Json::ARRAY).items) {
    auto v = [](const Json *m, const char *k) {
      const Json *x = m ? m->find(k) : nullptr;
      return x && x->is(Json::NUMBER) ? x->number : 0.0;
    };
    const Json *mix = l.find("mixer"), *mlp = l.find("mlp");
    widest = std::max(widest, (v(mix, "heads") + v(mix, "kv_heads")) * 2 * (v(mix, "dim") + v(mix, "vdim")));
    if (mlp) widest = std::max(widest, 2 * v(mlp->find("expert"), "ff"));
  }
  return std::max<size_t>((size_t)1 << 20, (size_t)(widest + 256) * hidden);
}

// Activations of a pass of R rows.
void create_pass(Netinex *e, Builder &b, int R) {
  const size_t elem = e->precise() ? sizeof(float) : sizeof(bf16_t), H = e->hidden;
  Shapes &x = e->wide;
  for (const NetinexLayer &w : e->layers) {
    const gptoss_moe_weights &m = w.moe;
    if (!m.n_experts) continue;
    const size_t pairs = (size_t)R * m.top_k;
    x.moe = std::max(x.moe, gptoss_moe_workspace_bytes(R, m.n_experts, m.top_k, m.hidden, m.intermediate));
    x.logits = std::max(x.logits, (size_t)R * m.n_experts);
    x.pairs = std::max(x.pairs, pairs);
    x.pairs_i = std::max(x.pairs_i, pairs * m.intermediate);
    x.pairs_h = std::max(x.pairs_h, pairs * m.hidden);
  }
  e->in_rows = b.alloc<float>((size_t)R * x.in);
  e->y_rows = b.alloc<float>((size_t)R * x.y);
  e->q_rows = b.alloc<float>((size_t)R * x.q);
  // room for every part of the output projection's sum while the rows are few
  e->branch_elems = std::max((size_t)R * H, std::min<size_t>((size_t)R * H * GEMM_MAX_PARTS, (size_t)32 << 20));
  e->branch = b.alloc<float>(e->branch_elems);
  e->t_rows = b.alloc<bf16_t>((size_t)R * H);
  e->act_rows = b.alloc<unsigned char>((size_t)R * x.act * elem);
  // padding columns are multiplied by zero weights, but must hold finite values
  if (b.ok()) b.hip(hipMemsetAsync(e->act_rows, 0, (size_t)R * x.act * elem, e->stream), "memset");
  if (e->precise()) {
    e->t_rows_f32 = b.alloc<float>((size_t)R * H);
    e->pr.logits = b.alloc<float>(x.logits);
    e->pr.topk_w = b.alloc<float>(x.pairs);
    e->pr.topk_i = b.alloc<int>(x.pairs);
    e->pr.up = b.alloc<float>(2 * x.pairs_i);
    e->pr.act = b.alloc<float>(x.pairs_i);
    e->pr.down = b.alloc<float>(x.pairs_h);
  } else {
    e->moe_ws = b.alloc<unsigned char>(x.moe);
  }
  if (b.ok()) b.hip(hipStreamSynchronize(e->stream), "sync");
}

int open_netinex(const ModelSource &src, const OpenOptions &o, gptoss_engine **out) {
  const bool synthetic = src.weights == nullptr;
  GPTOSS_REQUIRE(!(o.flags & (GPTOSS_ENGINE_NO_PREFILL | GPTOSS_ENGINE_MXFP4_EXPERTS)), GPTOSS_ERR_STATE,
                 "Netinex: GPTOSS_ENGINE_NO_PREFILL and GPTOSS_ENGINE_MXFP4_EXPERTS do not apply");
  GPTOSS_REQUIRE(!(synthetic && (o.flags & GPTOSS_ENGINE_PRECISE)), GPTOSS_ERR_STATE,
                 "Netinex: GPTOSS_ENGINE_PRECISE needs weights");
  Netinex *e = new Netinex();
  Builder b;
  b.e = e;
  try {
    const Json &cfg = *src.config;
    e->vocab = size_of(cfg, "vocab");
    e->vocab_rows = up64(e->vocab);
    e->hidden_real = size_of(cfg, "width");
    e->hidden = up64(e->hidden_real);
    e->norm_eps = (float)number(field(cfg, "norm", Json::OBJECT), "eps");
    const Json *cap = cfg.find("logit_softcap");
    if (cap && !cap->is(Json::NUL)) e->logit_softcap = (float)number(cfg, "logit_softcap");
    if (!(e->logit_softcap >= 0.f)) throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: \"logit_softcap\" must not be negative")};
    e->n_layers = (int)field(cfg, "layers", Json::ARRAY).items.size();
    if (e->n_layers < 1) throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: no layers")};
    if (e->hidden > 16384) throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: widths above 16384 are not supported")};
    e->max_batch = o.max_batch;
    e->max_seq = o.max_seq > 0 ? o.max_seq : NETINEX_POSITIONS;
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
    b.check(e->create_rows(R));
    if (b.ok()) b.check(e->create_sampling());
    if (b.ok()) create_pass(e, b, R);
  }
  if (!b.ok()) {
    delete e;
    return b.rc;
  }
  *out = e;
  return GPTOSS_OK;
}

const ModelClass netinex_class("Netinex", open_netinex);

}  // namespace

}  // namespace gptoss
