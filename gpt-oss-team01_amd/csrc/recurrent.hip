// Recurrent mixers for gfx950: gated delta rules (one decay per head, or one per key channel), the
// state-space recurrence and retention (a fixed decay per head, plain writes), with the short
// convolutions in front of them and the gated norms behind.
//
// The recurrence of a head acts on a K x V state whose V columns are independent of each other, so a
// column lives in 8 lanes of a wave (K / 8 rows each, in registers) and a wave owns 16 columns (8 where
// there is little to share out): for a step of one token the launch streams every state once through
// the chip, 16 bytes per lane and request; for a stretch of a prompt the state stays in registers while
// the tokens go by, their keys, queries and gates staged in LDS and shared by the workgroup's columns.
// Everything is fp32, and the tokens are taken one after the other, so a sequence's results are bit for
// bit the same however it is cut into steps.  Long stretches of retention run in retention.hip instead.
#include <type_traits>

#include "recurrent.hpp"

namespace gptoss {

// On the hardware's exp2, log2 and reciprocal (about one unit in the last place each), which keeps these
// within a few units: the argument of an exponential that matters is small.
__device__ __forceinline__ float exp_f(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.f + exp_f(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
// max(z, 0) + log(1 + e), e = exp(-|z|).  With u = 1 + e rounded, log(u) e / (u - 1) is log(1 + e) to a few
// units in the last place however small e is (W. Kahan's form of log1p).
__device__ __forceinline__ float softplus_f(float z) {
  const float e = exp_f(-fabsf(z)), u = 1.f + e, d = u - 1.f;
  const float l = __builtin_amdgcn_logf(u) * 0.6931471805599453f * e * __builtin_amdgcn_rcpf(d);
  return fmaxf(z, 0.f) + (d == 0.f ? e : l);
}

__device__ __forceinline__ float wave_sum_f(float v) {
#pragma unroll
  for (int m = 32; m >= 1; m >>= 1) v += __shfl_xor(v, m, 64);
  return v;
}

// sum over 8 consecutive lanes: two exchanges inside a quad, then the mirrored half row
template <int CTRL>
__device__ __forceinline__ float dpp_add(float v) {
  return v + __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float sum8(float v) {
  v = dpp_add<0xB1>(v);    // quad_perm [1,0,3,2]
  v = dpp_add<0x4E>(v);    // quad_perm [2,3,0,1]
  return dpp_add<0x141>(v);  // row_half_mirror
}

// ---- short convolution ---------------------------------------------------------------------------
// Input of channel c, j tokens before row r (offset `off` in its sequence's stretch, position `pos`).
__device__ __forceinline__ float conv_input(const ShortConv &c, const float *in, int ld_in, const float *state,
                                            int row, int off, int pos, int slot, int ch, int j) {
  if (j > pos) return 0.f;
  if (j <= off) return in[(size_t)(row - j) * ld_in + c.col + ch];
  // state[taps - 2] is the input right before the stretch
  return state[((size_t)slot * (c.taps - 1) + (c.taps - 1 + off - j)) * c.channels + ch];
}

// One wave per (rows, head): heads of unit_dim channels that become unit vectors first, then the remaining
// channels in pieces of 64.  A wave takes RT consecutive rows, whose inputs it requests together and
// slides the taps over (TAPS 0: any number of taps, inputs read tap by tap).
template <int TAPS, int RT>
__global__ __launch_bounds__(256) void short_conv_kernel(ShortConv c, const int *__restrict__ slots,
                                                         const int *__restrict__ lens,
                                                         const int *__restrict__ offset,
                                                         const float *__restrict__ in, int ld_in,
                                                         const float *__restrict__ state, float *__restrict__ out,
                                                         int ld_out, int units, int n) {
  constexpr int PIECES = SCAN_MAX_KEY / 64;
  const int row0 = blockIdx.y * RT, lane = threadIdx.x & 63;
  const int unit = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (unit >= units) return;
  const bool norm = unit < 2 * c.n_unit;
  const int unit_ch = 2 * c.n_unit * c.unit_dim;
  const int ch0 = norm ? unit * c.unit_dim : unit_ch + (unit - 2 * c.n_unit) * 64;
  const int width = norm ? c.unit_dim : min(64, c.channels - ch0);
  const int live = min(RT, n - row0);
  int off[RT], pos[RT], slot[RT];
#pragma unroll
  for (int r = 0; r < RT; r++) {
    const int row = row0 + min(r, live - 1);
    off[r] = offset[row];
    pos[r] = lens[row] - 1;
    slot[r] = slots[row];
  }
  float v[PIECES][RT], ss[RT];
#pragma unroll
  for (int r = 0; r < RT; r++) ss[r] = 0.f;
#pragma unroll
  for (int i = 0; i < PIECES; i++) {
    if (64 * i >= width) break;
    const int d = lane + 64 * i, ch = ch0 + min(d, width - 1);
    const float bias = c.bias ? c.bias[ch] : 0.f;
    if constexpr (TAPS > 0) {
      float w[TAPS], x[RT], past[TAPS];   // past[j]: the input j + 1 tokens back
#pragma unroll
      for (int j = 0; j < TAPS; j++) w[j] = c.weight[(size_t)ch * TAPS + (TAPS - 1 - j)];
#pragma unroll
      for (int r = 0; r < RT; r++) x[r] = in[(size_t)(row0 + min(r, live - 1)) * ld_in + c.col + ch];
#pragma unroll
      for (int r = 0; r < RT; r++) {
        if (r == 0 || off[r] == 0) {   // wave-uniform: the first row here, or of its sequence in this step
#pragma unroll
          for (int j = 0; j + 1 < TAPS; j++)
            past[j] = conv_input(c, in, ld_in, state, row0 + min(r, live - 1), off[r], pos[r], slot[r], ch, j + 1);
        }
        float a = bias;
#pragma unroll
        for (int j = TAPS - 1; j >= 1; j--) a = fmaf(w[j], past[j - 1], a);
        a = fmaf(w[0], x[r], a);
#pragma unroll
        for (int j = TAPS - 2; j >= 1; j--) past[j] = past[j - 1];
        if (TAPS > 1) past[0] = x[r];
        v[i][r] = d < width ? silu_f(a) : 0.f;
        ss[r] = fmaf(v[i][r], v[i][r], ss[r]);
      }
    } else {
#pragma unroll
      for (int r = 0; r < RT; r++) {
        float a = bias;
        for (int j = c.taps - 1; j >= 0; j--)
          a = fmaf(c.weight[(size_t)ch * c.taps + (c.taps - 1 - j)],
                   conv_input(c, in, ld_in, state, row0 + min(r, live - 1), off[r], pos[r], slot[r], ch, j), a);
        v[i][r] = d < width ? silu_f(a) : 0.f;
        ss[r] = fmaf(v[i][r], v[i][r], ss[r]);
      }
    }
  }
  float scale[RT];
#pragma unroll
  for (int r = 0; r < RT; r++) scale[r] = 1.f;
  if (norm) {
#pragma unroll
    for (int r = 0; r < RT; r++)
      scale[r] = (unit < c.n_unit ? c.unit_scale : 1.f) / sqrtf(wave_sum_f(ss[r]) + 1e-6f);
  }
#pragma unroll
  for (int i = 0; i < PIECES; i++) {
    if (64 * i >= width) break;
    const int d = lane + 64 * i;
#pragma unroll
    for (int r = 0; r < RT; r++)
      if (r < live && d < width) out[(size_t)(row0 + r) * ld_out + ch0 + d] = v[i][r] * scale[r];
  }
}

// ---- recurrence ----------------------------------------------------------------------------------
constexpr int SCAN_TOKENS = 16;   // tokens staged at a time

// The convolution's last taps - 1 inputs after the stretch; one thread owns a channel.
__device__ __forceinline__ void advance_conv_state(const Scan &p, const RowSeg &seg, int part, int parts) {
  const ShortConv &c = p.conv_desc;
  const int keep = c.taps - 1;
  for (int ch = part * 256 + threadIdx.x; ch < c.channels; ch += parts * 256) {
    float *st = p.conv_state + (size_t)seg.slot * keep * c.channels + ch;
    for (int i = 0; i < keep; i++) {
      const int t = seg.n - keep + i;   // row of the stretch whose input belongs here; negative: an older one
      float v = 0.f;
      if (t >= 0) v = p.in[(size_t)(seg.row0 + t) * p.ld_in + c.col + ch];
      else if (seg.pos0 + t >= 0) v = st[(size_t)(i + seg.n) * c.channels];
      st[(size_t)i * c.channels] = v;
    }
  }
}

// What a lane needs of one token.
template <int NI, bool CHANNEL, int CPL>
struct ScanToken {
  f32x4 k[NI], q[NI], g[CHANNEL ? NI : 1];
  float v[CPL], decay, beta;
};

// CPL: columns per lane; a workgroup has 4 waves x 8 lane groups x CPL columns.  Two share the reads of a
// token's keys and queries; one gives twice the workgroups, where there are few heads and sequences.
// ONE: every sequence has one row (decoding); the launch is then a stream of states through the chip.
template <int NI, int KIND, bool ONE, int CPL>
__global__ __launch_bounds__(256) void scan_kernel(Scan p, const RowSeg *__restrict__ segs, int n_seg) {
  constexpr int KP = 32 * NI, TC = ONE ? 1 : SCAN_TOKENS;
  constexpr bool CHANNEL = KIND == SCAN_CHANNEL_DELTA, SSM = KIND == SCAN_STATE_SPACE, RET = KIND == SCAN_RETENTION;
  constexpr int COLS = 32 * CPL;
  constexpr int PIECES = (TC * KP / 4 + 255) / 256, VPIECES = (TC * COLS / 4 + 255) / 256;
  // one token more than is staged: the loop reads a token ahead
  __shared__ __attribute__((aligned(16))) float sk[TC + 1][KP], sq[TC + 1][KP], sg[CHANNEL ? TC + 1 : 1][KP];
  __shared__ __attribute__((aligned(16))) float sv[TC + 1][COLS];
  __shared__ float s_decay[TC + 1], s_beta[TC + 1];
  // workgroups in order of (head, column block, sequence); those of the convolutions' states come last
  const int blocks = (p.V + COLS - 1) / COLS;
  const int seg_id = blockIdx.x % n_seg, unit = blockIdx.x / n_seg;
  const RowSeg seg = segs[seg_id];
  if (unit >= p.heads * blocks) {
    advance_conv_state(p, seg, unit - p.heads * blocks, blocks);
    return;
  }
  const int h = unit / blocks;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int j = lane & 7;
  const int c0 = (unit - h * blocks) * COLS, cw = (wave * 8 + (lane >> 3)) * CPL;   // this lane's first column is c0 + cw
  const bool busy = c0 + wave * 8 * CPL < p.V;   // wave-uniform
  const int kh = h / (p.heads / p.key_heads);
  const float rate = RET ? 0.f : expf(p.a_log[h]);
  const float bias = CHANNEL || RET ? 0.f : p.dt_bias[h];
  const float fixed = RET ? p.head_decay[h] : 0.f;
  const float skip = SSM ? p.d_skip[h] : 0.f;

  f32x4 S[CPL][NI];
  float *st = p.state + (((size_t)seg.slot * p.heads + h) * p.V + c0 + cw) * KP + 4 * j;
#pragma unroll
  for (int c = 0; c < CPL; c++)
#pragma unroll
    for (int i = 0; i < NI; i++) {
      S[c][i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (seg.pos0 > 0 && c0 + cw + c < p.V)
        S[c][i] = __builtin_nontemporal_load(reinterpret_cast<const f32x4 *>(st + c * KP + 32 * i));
    }

  // the next tokens' inputs travel through registers, four values at a time, while the current ones are
  // worked on; rows and columns outside the problem are read from inside it and replaced by zero
  f32x4 rk[PIECES], rq[PIECES], rg[CHANNEL ? PIECES : 1], rv[VPIECES];
  float r_beta = 0.f, r_decay = 0.f;
  const float *k_src = p.conv + p.k_col + kh * p.K, *q_src = p.conv + p.q_col + kh * p.K;
  const float *v_src = p.conv + p.v_col + h * p.V, *g_src = p.channel_decay + h * p.K;
  auto load4 = [&](const float *row, int d, int limit) {
    f32x4 x;
    if (p.vec) {
      x = *reinterpret_cast<const f32x4 *>(row + min(d, limit - 4));
    } else {
#pragma unroll
      for (int e = 0; e < 4; e++) x[e] = row[min(d + e, limit - 1)];
    }
#pragma unroll
    for (int e = 0; e < 4; e++) x[e] = d + e < limit ? x[e] : 0.f;
    return x;
  };
  auto fetch = [&](int t0) {
    const int T = min(TC, seg.n - t0);
    const size_t first = seg.row0 + t0;
#pragma unroll
    for (int x = 0; x < PIECES; x++) {
      const int idx = tid + 256 * x, t = min(idx / (KP / 4), T - 1), d = idx % (KP / 4) * 4;
      const float *kr = k_src + (first + t) * p.ld_conv, *qr = q_src + (first + t) * p.ld_conv;
      rk[x] = load4(kr, d, p.K);
      rq[x] = load4(qr, d, p.K);
      if constexpr (RET && ONE) {
        const int half = p.rot.table ? p.rot.dims >> 1 : 0;
        if (d < 2 * half) {   // pairs (i, i + half)
          const bool second = d >= half;
          const int i = second ? d - half : d, partner = second ? i : i + half;
          const f32x4 ko = load4(kr, partner, p.K), qo = load4(qr, partner, p.K);
          const f32x4 *at = reinterpret_cast<const f32x4 *>(p.rot.table + ((size_t)seg.pos0 * half + i) * 2);
          const f32x4 cs[2] = {at[0], at[1]};
#pragma unroll
          for (int e = 0; e < 4; e++) {
            const float c = cs[e >> 1][2 * (e & 1)], s = (second ? 1.f : -1.f) * cs[e >> 1][2 * (e & 1) + 1];
            rk[x][e] = rk[x][e] * c + ko[e] * s;
            rq[x][e] = rq[x][e] * c + qo[e] * s;
          }
        }
      }
      if (CHANNEL) rg[x] = load4(g_src + (first + t) * p.ld_decay, d, p.K);
    }
#pragma unroll
    for (int x = 0; x < VPIECES; x++) {
      const int idx = tid + 256 * x, t = min(idx / (COLS / 4), T - 1), c = c0 + idx % (COLS / 4) * 4;
      rv[x] = load4(v_src + (first + t) * p.ld_conv, c, p.V);
    }
    if (RET) return;
    const float *ir = p.in + (first + min(tid, T - 1)) * p.ld_in + h;
    if (!SSM) r_beta = ir[p.beta_col];
    if (!CHANNEL) r_decay = ir[p.decay_col];
  };
  auto put = [&]() {
#pragma unroll
    for (int x = 0; x < PIECES; x++) {
      const int idx = tid + 256 * x, t = idx / (KP / 4), d = idx % (KP / 4) * 4;
      if (TC * KP / 4 % 256 == 0 || t < TC) {
        *reinterpret_cast<f32x4 *>(&sk[t][d]) = rk[x];
        *reinterpret_cast<f32x4 *>(&sq[t][d]) = rq[x];
        if (CHANNEL) {
          f32x4 g;
#pragma unroll
          for (int e = 0; e < 4; e++)
            g[e] = exp_f(-rate * softplus_f(rg[x][e] + p.dt_bias[h * p.K + min(d + e, p.K - 1)]));
          *reinterpret_cast<f32x4 *>(&sg[t][d]) = g;
        }
      }
    }
#pragma unroll
    for (int x = 0; x < VPIECES; x++) {
      const int idx = tid + 256 * x;
      if (TC * COLS / 4 % 256 == 0 || idx < TC * COLS / 4)
        *reinterpret_cast<f32x4 *>(&sv[0][0] + idx * 4) = rv[x];
    }
    if (!RET && tid < TC) {
      if (SSM) {
        const float dt = softplus_f(r_decay + bias);
        s_decay[tid] = exp_f(-rate * dt);
        s_beta[tid] = dt;
      } else {
        s_beta[tid] = sigmoid_f(r_beta);
        if (!CHANNEL) s_decay[tid] = exp_f(-rate * softplus_f(r_decay + bias));
      }
    }
  };
  using Token = ScanToken<NI, CHANNEL, CPL>;
  auto read = [&](Token &x, int t) {
#pragma unroll
    for (int i = 0; i < NI; i++) {
      x.k[i] = *reinterpret_cast<const f32x4 *>(&sk[t][32 * i + 4 * j]);
      x.q[i] = *reinterpret_cast<const f32x4 *>(&sq[t][32 * i + 4 * j]);
      if (CHANNEL) x.g[i] = *reinterpret_cast<const f32x4 *>(&sg[t][32 * i + 4 * j]);
    }
#pragma unroll
    for (int c = 0; c < CPL; c++) x.v[c] = sv[t][cw + c];
    if (!RET) x.beta = s_beta[t];
    if (!CHANNEL && !RET) x.decay = s_decay[t];
  };
  auto advance = [&](const Token &x, float (&o)[CPL]) {
#pragma unroll
    for (int c = 0; c < CPL; c++)
#pragma unroll
      for (int i = 0; i < NI; i++)
#pragma unroll
        for (int e = 0; e < 4; e++) S[c][i][e] *= CHANNEL ? x.g[CHANNEL ? i : 0][e] : RET ? fixed : x.decay;
    float u[CPL];
#pragma unroll
    for (int c = 0; c < CPL; c++) {
      if constexpr (RET) {
        u[c] = p.value_scale * x.v[c];
      } else if constexpr (SSM) {
        u[c] = x.beta * x.v[c];
      } else {
        float d0 = 0.f, d1 = 0.f;
#pragma unroll
        for (int i = 0; i < NI; i++) {
          d0 = fmaf(S[c][i][0], x.k[i][0], d0);
          d1 = fmaf(S[c][i][1], x.k[i][1], d1);
          d0 = fmaf(S[c][i][2], x.k[i][2], d0);
          d1 = fmaf(S[c][i][3], x.k[i][3], d1);
        }
        u[c] = x.beta * (x.v[c] - sum8(d0 + d1));
      }
    }
#pragma unroll
    for (int c = 0; c < CPL; c++) {
      float d0 = 0.f, d1 = 0.f;
#pragma unroll
      for (int i = 0; i < NI; i++) {
#pragma unroll
        for (int e = 0; e < 4; e++) S[c][i][e] = fmaf(x.k[i][e], u[c], S[c][i][e]);
        d0 = fmaf(S[c][i][0], x.q[i][0], d0);
        d1 = fmaf(S[c][i][1], x.q[i][1], d1);
        d0 = fmaf(S[c][i][2], x.q[i][2], d0);
        d1 = fmaf(S[c][i][3], x.q[i][3], d1);
      }
      o[c] = sum8(d0 + d1);
      if (SSM) o[c] = fmaf(skip, x.v[c], o[c]);
    }
  };
  // lane j of a group keeps the results of tokens t with t % 8 == j; they are stored eight at a time, those
  // of a piece's last tokens after the next piece has been staged (the wait for its loads would otherwise
  // be one for these stores)
  float keep[CPL];
  int kept = -1;   // first row of the tokens in keep; -1: stored
  auto flush = [&](int rows) {
    if (j < rows) {
      float *dst = p.out + (size_t)(kept + j) * p.ld_out + h * p.V + c0 + cw;
#pragma unroll
      for (int c = 0; c < CPL; c++)
        if (c0 + cw + c < p.V) dst[c] = keep[c];
    }
    kept = -1;
  };
  fetch(0);
  for (int t0 = 0; t0 < seg.n; t0 += TC) {
    const int T = min(TC, seg.n - t0);
    if (t0 > 0) __syncthreads();
    put();
    __syncthreads();
    if (!ONE && t0 + TC < seg.n) fetch(t0 + TC);
    if (!busy) continue;
    if (!ONE && kept >= 0) flush(8);   // a full piece came before
    auto emit = [&](int t, const float (&o)[CPL]) {
#pragma unroll
      for (int c = 0; c < CPL; c++) keep[c] = (t & 7) == j ? o[c] : keep[c];
      if ((t & 7) == 0) kept = seg.row0 + t0 + t;
      if ((t & 7) == 7 && t + 1 < TC) flush(8);
    };
    Token a;
    read(a, 0);
    if constexpr (ONE) {
      float o[CPL];
      advance(a, o);
      emit(0, o);
    } else if constexpr (NI <= 4) {
      // two tokens in registers: the next one's inputs are requested before the current one is worked on
      Token b;
      for (int t = 0; t < T; t += 2) {
        float o[CPL];
        read(b, t + 1);
        advance(a, o);
        emit(t, o);
        if (t + 1 >= T) break;
        read(a, t + 2);
        advance(b, o);
        emit(t + 1, o);
      }
    } else {
      for (int t = 0; t < T; t++) {
        float o[CPL];
        advance(a, o);
        emit(t, o);
        if (t + 1 < T) read(a, t + 1);
      }
    }
  }
  if (busy && kept >= 0) flush(seg.row0 + seg.n - kept);
#pragma unroll
  for (int c = 0; c < CPL; c++)
#pragma unroll
    for (int i = 0; i < NI; i++)
      if (c0 + cw + c < p.V)
        __builtin_nontemporal_store(S[c][i], reinterpret_cast<f32x4 *>(st + c * KP + 32 * i));
}

// ---- gated output norm ---------------------------------------------------------------------------
__device__ __forceinline__ float gated_value(const GatedNorm &g, float y, float gate) {
  return g.gate_first ? y * silu_f(gate) : y;
}

// One wave per (row, group), any size and alignment.
template <typename OUT>
__global__ __launch_bounds__(256) void gated_norm_kernel(GatedNorm g) {
  const int row = blockIdx.y, lane = threadIdx.x & 63;
  const int group = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (group >= g.groups) return;
  const float *y = g.y + (size_t)row * g.ld_y + group * g.size;
  const float *gate = g.gate + (size_t)row * g.ld_gate + group * g.size;
  const float *w = g.weight ? g.weight + (g.weight_per_group ? group * g.size : 0) : nullptr;
  float ss = 0.f;
  for (int d = lane; d < g.size; d += 64) {
    const float v = gated_value(g, y[d], gate[d]);
    ss += v * v;
  }
  const float inv = 1.f / sqrtf(wave_sum_f(ss) / g.size + g.eps);
  OUT *out = (OUT *)g.out + (size_t)row * g.ld_out + g.out_col + group * g.size;
  for (int d = lane; d < g.size; d += 64) {
    float v = gated_value(g, y[d], gate[d]) * inv * (w ? w[d] : 1.f);
    if (!g.gate_first) v *= g.sigmoid_gate ? sigmoid_f(gate[d]) : silu_f(gate[d]);
    v *= g.scale;
    if constexpr (sizeof(OUT) == 2) out[d] = f32_to_bf16(v);
    else out[d] = v;
  }
}

// Groups of at most 4 * LANES * VPT values whose rows are 16-byte aligned: LANES lanes hold a group in
// registers, a wave 64 / LANES groups.
template <typename OUT, int LANES, int VPT>
__global__ __launch_bounds__(256) void gated_norm_vec_kernel(GatedNorm g) {
  const int row = blockIdx.y, l = threadIdx.x % LANES;
  const int group = blockIdx.x * (256 / LANES) + threadIdx.x / LANES;
  const bool live = group < g.groups;
  const int at = (live ? group : 0) * g.size;
  const float *y = g.y + (size_t)row * g.ld_y + at, *gate = g.gate + (size_t)row * g.ld_gate + at;
  const float *w = g.weight ? g.weight + (g.weight_per_group ? at : 0) : nullptr;
  f32x4 v[VPT], z[VPT];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; i++) {
    const int d = (l + LANES * i) * 4;
    v[i] = z[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (d < g.size) {
      v[i] = *reinterpret_cast<const f32x4 *>(y + d);
      z[i] = *reinterpret_cast<const f32x4 *>(gate + d);
    }
  }
#pragma unroll
  for (int i = 0; i < VPT; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      v[i][e] = gated_value(g, v[i][e], z[i][e]);
      ss = fmaf(v[i][e], v[i][e], ss);
    }
#pragma unroll
  for (int m = LANES / 2; m >= 1; m >>= 1) ss += __shfl_xor(ss, m, 64);
  const float inv = 1.f / sqrtf(ss / g.size + g.eps);
  if (!live) return;
  OUT *out = (OUT *)g.out + (size_t)row * g.ld_out + g.out_col + at;
#pragma unroll
  for (int i = 0; i < VPT; i++) {
    const int d = (l + LANES * i) * 4;
    if (d < g.size) {
      const f32x4 wv = w ? *reinterpret_cast<const f32x4 *>(w + d) : f32x4{1.f, 1.f, 1.f, 1.f};
      f32x4 o;
#pragma unroll
      for (int e = 0; e < 4; e++) {
        o[e] = v[i][e] * inv * wv[e];
        if (!g.gate_first) o[e] *= g.sigmoid_gate ? sigmoid_f(z[i][e]) : silu_f(z[i][e]);
        o[e] *= g.scale;
      }
      if constexpr (sizeof(OUT) == 2)
        *reinterpret_cast<u32x2 *>(out + d) = u32x2{pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3])};
      else *reinterpret_cast<f32x4 *>(out + d) = o;
    }
  }
}

__global__ __launch_bounds__(256) void column_map_kernel(const float *__restrict__ in, int ld_in, int col, int width,
                                                         int relu_squared, float *__restrict__ out, int ld_out) {
  const int d = blockIdx.x * 256 + threadIdx.x;
  const size_t row = blockIdx.y;
  if (d >= width) return;
  float v = in[row * ld_in + col + d];
  if (relu_squared) {
    v = fmaxf(v, 0.f);
    v *= v;
  }
  out[row * ld_out + d] = v;
}

// ---- launches ------------------------------------------------------------------------------------
int run_short_conv(const ShortConv &c, const StepRows &r, const float *in, int ld_in, const float *state,
                   float *out, int ld_out, hipStream_t s) {
  GPTOSS_REQUIRE(c.unit_dim <= SCAN_MAX_KEY && c.taps >= 1, GPTOSS_ERR_DIM,
                 "short_conv: heads of at most %d channels, at least one tap (%d, %d)", SCAN_MAX_KEY, c.unit_dim, c.taps);
  const int plain = c.channels - 2 * c.n_unit * c.unit_dim;
  const int units = 2 * c.n_unit + cdiv(plain, 64);
  TraceScope ts("short_conv", s);
  auto go = [&](auto kern, int rt) {
    kern<<<dim3(cdiv(units, 4), cdiv(r.n, rt)), 256, 0, s>>>(c, r.slots, r.lens, r.offset, in, ld_in, state, out, ld_out,
                                                             units, r.n);
  };
  const bool many = r.longest > 1 && r.n >= 256;
  if (c.taps == 4) many ? go(short_conv_kernel<4, 8>, 8) : go(short_conv_kernel<4, 1>, 1);
  else if (c.taps == 3) many ? go(short_conv_kernel<3, 8>, 8) : go(short_conv_kernel<3, 1>, 1);
  else if (c.taps == 2) many ? go(short_conv_kernel<2, 8>, 8) : go(short_conv_kernel<2, 1>, 1);
  else go(short_conv_kernel<0, 1>, 1);
  GPTOSS_LAUNCH_CHECK("short_conv_kernel");
  return GPTOSS_OK;
}

template <int NI, int KIND>
static void launch_scan_kind(const Scan &p, const StepRows &r, hipStream_t s) {
  auto grid = [&](int cols) { return dim3((unsigned)(r.n_seg * (p.heads + (KIND == SCAN_RETENTION ? 0 : 1)) * cdiv(p.V, cols))); };
  // stretches of few heads and sequences: with two columns per lane half of the chip would be idle
  const bool few = (long long)r.n_seg * p.heads * cdiv(p.V, 64) <= 128;
  if (r.longest == 1) scan_kernel<NI, KIND, true, 2><<<grid(64), 256, 0, s>>>(p, r.segs, r.n_seg);
  else if (few) scan_kernel<NI, KIND, false, 1><<<grid(32), 256, 0, s>>>(p, r.segs, r.n_seg);
  else scan_kernel<NI, KIND, false, 2><<<grid(64), 256, 0, s>>>(p, r.segs, r.n_seg);
}

template <int NI>
static void launch_scan(const Scan &p, const StepRows &r, hipStream_t s) {
  switch (p.kind) {
    case SCAN_DELTA: launch_scan_kind<NI, SCAN_DELTA>(p, r, s); break;
    case SCAN_CHANNEL_DELTA: launch_scan_kind<NI, SCAN_CHANNEL_DELTA>(p, r, s); break;
    case SCAN_STATE_SPACE: launch_scan_kind<NI, SCAN_STATE_SPACE>(p, r, s); break;
    case SCAN_RETENTION: launch_scan_kind<NI, SCAN_RETENTION>(p, r, s); break;
  }
}

int run_scan(const Scan &scan, const StepRows &r, hipStream_t s) {
  Scan p = scan;
  p.vec = scan_reads_wide(p);
  GPTOSS_REQUIRE(!p.rot.table || (p.kind == SCAN_RETENTION && r.longest == 1 && p.vec && !p.rot.interleaved &&
                                  p.rot.dims % 8 == 0 && p.rot.dims <= p.K),
                 GPTOSS_ERR_DIM, "scan: only steps of one row per sequence rotate queries and keys, in groups of four dimensions");
  GPTOSS_REQUIRE(p.K >= 1 && p.K <= SCAN_MAX_KEY && p.V >= 1 && p.key_heads >= 1 && p.heads % p.key_heads == 0,
                 GPTOSS_ERR_DIM, "scan: key dimension %d (at most %d), %d heads over %d", p.K, SCAN_MAX_KEY, p.heads,
                 p.key_heads);
  GPTOSS_REQUIRE((long long)r.n_seg * (p.heads + 1) * cdiv(p.V, 32) < (1ll << 31), GPTOSS_ERR_DIM,
                 "scan: too many workgroups");
  static const char *names[] = {"scan_delta", "scan_channel_delta", "scan_state_space", "scan_retention"};
  TraceScope ts(names[p.kind], s);
  switch (scan_key_pad(p.K) / 32) {
    case 1: launch_scan<1>(p, r, s); break;
    case 2: launch_scan<2>(p, r, s); break;
    case 3: launch_scan<3>(p, r, s); break;
    case 4: launch_scan<4>(p, r, s); break;
    case 5: launch_scan<5>(p, r, s); break;
    case 6: launch_scan<6>(p, r, s); break;
    case 7: launch_scan<7>(p, r, s); break;
    default: launch_scan<8>(p, r, s); break;
  }
  GPTOSS_LAUNCH_CHECK("scan_kernel");
  return GPTOSS_OK;
}

template <typename OUT>
static void launch_gated_norm(const GatedNorm &g, int n, hipStream_t s) {
  const bool vec = g.size % 4 == 0 && g.ld_y % 4 == 0 && g.ld_gate % 4 == 0 && g.ld_out % 4 == 0 && g.out_col % 4 == 0 &&
                   aligned(g.y, 16) && aligned(g.gate, 16) && aligned(g.weight, 16) && aligned(g.out, 16);
  if (vec && g.size <= 64) gated_norm_vec_kernel<OUT, 16, 1><<<dim3(cdiv(g.groups, 16), n), 256, 0, s>>>(g);
  else if (vec && g.size <= 128) gated_norm_vec_kernel<OUT, 32, 1><<<dim3(cdiv(g.groups, 8), n), 256, 0, s>>>(g);
  else if (vec && g.size <= 256) gated_norm_vec_kernel<OUT, 64, 1><<<dim3(cdiv(g.groups, 4), n), 256, 0, s>>>(g);
  else if (vec && g.size <= 512) gated_norm_vec_kernel<OUT, 64, 2><<<dim3(cdiv(g.groups, 4), n), 256, 0, s>>>(g);
  else if (vec && g.size <= 1024) gated_norm_vec_kernel<OUT, 64, 4><<<dim3(cdiv(g.groups, 4), n), 256, 0, s>>>(g);
  else gated_norm_kernel<OUT><<<dim3(cdiv(g.groups, 4), n), 256, 0, s>>>(g);
}

int run_gated_norm(const GatedNorm &g, int n, hipStream_t s) {
  TraceScope ts("gated_norm", s);
  if (g.out_f32) launch_gated_norm<float>(g, n, s);
  else launch_gated_norm<bf16_t>(g, n, s);
  GPTOSS_LAUNCH_CHECK("gated_norm_kernel");
  return GPTOSS_OK;
}

int run_column_map(const float *in, int ld_in, int col, int width, bool relu_squared, float *out, int ld_out, int n,
                   hipStream_t s) {
  TraceScope ts(relu_squared ? "relu_squared" : "column_copy", s);
  column_map_kernel<<<dim3(cdiv(width, 256), n), 256, 0, s>>>(in, ld_in, col, width, relu_squared, out, ld_out);
  GPTOSS_LAUNCH_CHECK("column_map_kernel");
  return GPTOSS_OK;
}

}  // namespace gptoss
