// What the classes that open config.json + model.safetensors share: typed access to the configuration, and
// matrices assembled from tensors for the kernels' layouts.
#pragma once
#include <math.h>

#include "builder.hpp"
#include "model_registry.hpp"
#include "window_attn.hpp"

namespace gptoss {

// ---- config.json ---------------------------------------------------------------------------------
struct ConfigError {
  int rc;
};

inline const Json &field(const Json &j, const char *key, Json::Type type) {
  const Json *v = j.find(key);
  if (!v || !v->is(type)) throw ConfigError{fail(GPTOSS_ERR_IO, "config.json: \"%s\" is missing or of the wrong type", key)};
  return *v;
}
inline double number(const Json &j, const char *key) { return field(j, key, Json::NUMBER).number; }
inline int size_of(const Json &j, const char *key) {
  const double v = number(j, key);
  if (!(v >= 1 && v <= (1 << 30) && v == floor(v)))
    throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: \"%s\" must be a positive integer", key)};
  return (int)v;
}
inline void require(bool ok, const char *what, int layer) {
  if (!ok) throw ConfigError{fail(GPTOSS_ERR_DIM, "config.json: layer %d: %s", layer, what)};
}

inline int up32(int n) { return (n + 31) / 32 * 32; }
inline int up64(int n) { return (n + 63) / 64 * 64; }

// ---- weights -------------------------------------------------------------------------------------
struct Matrix {   // bf16 packed, or fp32 row-major
  bf16_t *packed = nullptr;
  float *f32 = nullptr;
  int n_out = 0, n_in = 0;
};

// Tensors of a checkpoint on their way to the device.  A matrix is assembled on the host from several tensors,
// its unused rows and columns zero.
struct Loader {
  gptoss_engine *e;
  Builder &b;
  const SafeTensors *st;   // nullptr: random weights
  uint64_t seed;
  uint64_t next_seed() { return seed += 0x9E3779B97F4A7C15ull; }

  std::vector<float> host(const std::string &name, const std::vector<long long> &shape) {
    std::vector<float> v;
    const int rc = st->read(name, shape, &v);
    if (rc != GPTOSS_OK) throw ConfigError{rc};
    return v;
  }
  // host values -> fp32 on the device, as they are
  float *put(const std::vector<float> &v) {
    float *d = b.alloc<float>(v.size());
    if (b.ok()) b.hip(hipMemcpy(d, v.data(), sizeof(float) * v.size(), hipMemcpyHostToDevice), "H2D");
    return d;
  }
  // fp32 vector on the device; random: N(mean, std)
  float *vec(const std::string &name, const std::vector<long long> &shape, float mean, float std) {
    size_t n = 1;
    for (long long d : shape) n *= d;
    if (!st) return b.upload_f32(nullptr, n, next_seed(), mean, std);
    return b.upload_f32(host(name, shape).data(), n, 0, 0, 0);
  }
  // a vector over the residual stream's columns, zero in the padding; random: all `value`
  float *column_vec(const std::string &name, float value) {
    std::vector<float> v(e->hidden_real, value);
    if (st) v = host(name, {e->hidden_real});
    v.resize(e->hidden, 0.f);
    return put(v);
  }
  // a single value; random: `value`
  float scalar(const std::string &name, float value) { return st ? host(name, {})[0] : value; }
  // a norm whose gain is a scalar, as the vector the norm kernels take (zero in the padding)
  float *scalar_norm(const std::string &name) {
    std::vector<float> v(e->hidden_real, scalar(name, 1.f));
    v.resize(e->hidden, 0.f);
    return put(v);
  }
  struct Part {
    std::string name;
    int rows, cols, row0, col0;
    int row_step = 1;   // rows of the matrix from one row of the tensor to the next
  };
  // n_mat matrices of one shape, one list of parts each
  Matrix matrices(int n_out, int n_in, const std::vector<std::vector<Part>> &lists, int pack_flags) {
    Matrix m;
    m.n_out = n_out;
    m.n_in = n_in;
    const size_t per = (size_t)n_out * n_in;
    std::vector<float> full;
    if (st) {
      full.assign(per * lists.size(), 0.f);
      for (size_t i = 0; i < lists.size(); i++)
        for (const Part &p : lists[i]) {
          const std::vector<float> v = host(p.name, {p.rows, p.cols});
          for (int r = 0; r < p.rows; r++)
            memcpy(&full[per * i + (size_t)(p.row0 + r * p.row_step) * n_in + p.col0], &v[(size_t)r * p.cols],
                   sizeof(float) * p.cols);
        }
    }
    if (e->precise()) m.f32 = b.upload_f32(full.data(), full.size(), 0, 0, 0);
    else
      m.packed = b.upload_matrices(st ? full.data() : nullptr, (int)lists.size(), n_out, n_in, true, pack_flags, next_seed(),
                                   1.f / sqrtf((float)n_in));
    return m;
  }
  Matrix matrix(int n_out, int n_in, const std::vector<Part> &parts) { return matrices(n_out, n_in, {parts}, 0); }
  // a row-major table of `ld` columns (the tensor's `cols`, then zeros), not packed: rows that are gathered or read in place
  void table(const std::string &name, int n_rows, int cols, int ld, float std, bf16_t **t, float **t_f32) {
    std::vector<float> v;
    if (st) {
      v = host(name, {n_rows, cols});
      if (ld != cols) {
        std::vector<float> wide((size_t)n_rows * ld, 0.f);
        for (int r = 0; r < n_rows; r++) memcpy(&wide[(size_t)r * ld], &v[(size_t)r * cols], sizeof(float) * cols);
        v.swap(wide);
      }
    }
    if (e->precise()) {
      *t_f32 = b.upload_f32(v.data(), v.size(), 0, 0, 0);
      return;
    }
    const size_t n = (size_t)n_rows * ld;
    *t = b.alloc<bf16_t>(n);
    if (!st) {
      if (b.ok()) b.check(run_synth_bf16(*t, n, next_seed(), 0.f, std, e->stream));
      return;
    }
    for (size_t o = 0; o < n && b.ok(); o += b.st.elems) {
      const size_t c = std::min(b.st.elems, n - o);
      int slot;
      const float *src = b.stage_in(v.data() + o, c, &slot);
      if (!b.ok()) break;
      b.check(run_f32_to_bf16(src, *t + o, c, e->stream));
      b.release(slot);
    }
  }
  float *zeros(size_t n) {
    float *d = b.alloc<float>(n);
    if (b.ok()) b.hip(hipMemsetAsync(d, 0, n * sizeof(float), e->stream), "memset");
    return d;
  }
  // 0 for the vocabulary, a large negative value for its padding (never the arg-max); nullptr without padding
  float *class_bias() {
    if (e->vocab_rows == e->vocab) return nullptr;
    std::vector<float> bias(e->vocab, 0.f);
    bias.resize(e->vocab_rows, -3.0e38f);
    return put(bias);
  }
};

// The K/V ring of an attention layer whose passes hold up to `most` rows of a sequence, and its piece size among
// the step's tiles.
inline void window_attn_cache(Loader &ld, WindowAttn &a, int most) {
  gptoss_engine *e = ld.e;
  const long long stretch = std::min(e->max_seq, most);
  a.cap = (int)std::min<long long>((e->max_seq + 63) / 64 * 64, (a.window - 1 + stretch + 63) / 64 * 64);
  const size_t slots = (size_t)e->max_batch * a.cap * a.kv_heads;
  if (e->precise()) {
    a.k32 = ld.zeros(slots * a.dim);
    a.v32 = ld.zeros(slots * a.vdim);
  } else {
    // slots that were never written are masked, but must hold finite values
    a.kv = (bf16_t *)ld.zeros(slots / KV_BLOCK * a.block_elems() / 2);
  }
  const int tr = window_attn_tile_rows(a.heads, a.kv_heads);
  auto at = std::find(e->tile_rows.begin(), e->tile_rows.end(), tr);
  a.tiles = (int)(at - e->tile_rows.begin());
  if (at == e->tile_rows.end()) e->tile_rows.push_back(tr);
}

// Columns of assembled rows are handed out in the order they are asked for.
struct Columns {
  int used = 0;
  int take(int n) {
    const int o = used;
    used += n;
    return o;
  }
  void align(int to = 32) { used = (used + to - 1) / to * to; }
};

}  // namespace gptoss
