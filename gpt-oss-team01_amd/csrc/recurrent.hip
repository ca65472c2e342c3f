// Recurrent mixers for gfx950: gated delta rules (one decay per head, or one per key channel) and the
// state-space recurrence, with the short convolutions in front of them and the gated norms behind.
//
// The recurrence of a head acts on a K x V state whose V columns are independent of each other, so a
// column lives in 8 lanes of a wave (K / 8 rows each, in registers) and a wave owns 16 columns: for a
// step of one token the launch streams every state once through the chip, 16 bytes per lane and
// request; for a stretch of a prompt the state stays in registers while the tokens go by, their keys,
// queries and gates staged in LDS and shared by the workgroup's 64 columns.  Everything is fp32, and
// the tokens are taken one after the other, so a sequence's results are bit for bit the same however
// it is cut into steps.
#include <type_traits>

#include "recurrent.hpp"

namespace gptoss {

__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

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

// One wave per (row, head): heads of unit_dim channels that become unit vectors first, then the
// remaining channels in pieces of 64.
__global__ __launch_bounds__(256) void short_conv_kernel(ShortConv c, const int *__restrict__ slots,
                                                         const int *__restrict__ lens,
                                                         const int *__restrict__ offset,
                                                         const float *__restrict__ in, int ld_in,
                                                         const float *__restrict__ state, float *__restrict__ out,
                                                         int ld_out, int units) {
  const int row = blockIdx.y, lane = threadIdx.x & 63;
  const int unit = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (unit >= units) return;
  const int off = offset[row], pos = lens[row] - 1, slot = slots[row];
  const bool norm = unit < 2 * c.n_unit;
  const int unit_ch = 2 * c.n_unit * c.unit_dim;
  const int ch0 = norm ? unit * c.unit_dim : unit_ch + (unit - 2 * c.n_unit) * 64;
  const int width = norm ? c.unit_dim : min(64, c.channels - ch0);
  float v[SCAN_MAX_KEY / 64], ss = 0.f;
#pragma unroll
  for (int i = 0; i < SCAN_MAX_KEY / 64; i++) {
    v[i] = 0.f;
    const int d = lane + 64 * i;
    if (d < width) {
      const int ch = ch0 + d;
      float a = c.bias ? c.bias[ch] : 0.f;
      for (int j = c.taps - 1; j >= 0; j--)
        a += c.weight[(size_t)ch * c.taps + (c.taps - 1 - j)] * conv_input(c, in, ld_in, state, row, off, pos, slot, ch, j);
      v[i] = silu_f(a);
      ss += v[i] * v[i];
    }
  }
  float scale = 1.f;
  if (norm) scale = (unit < c.n_unit ? c.unit_scale : 1.f) / sqrtf(wave_sum_f(ss) + 1e-6f);
#pragma unroll
  for (int i = 0; i < SCAN_MAX_KEY / 64; i++) {
    const int d = lane + 64 * i;
    if (d < width) out[(size_t)row * ld_out + ch0 + d] = v[i] * scale;
  }
}

// ---- recurrence ----------------------------------------------------------------------------------
constexpr int SCAN_TOKENS = 16;   // tokens staged at a time
constexpr int SCAN_COLS = 64;     // state columns of a workgroup: 4 waves x 8 lane groups x 2

// The convolution's last taps - 1 inputs after the stretch; one thread owns a channel.
__device__ __forceinline__ void advance_conv_state(const Scan &p, const RowSeg &seg) {
  const ShortConv &c = p.conv_desc;
  const int keep = c.taps - 1;
  for (int ch = blockIdx.z * 256 + threadIdx.x; ch < c.channels; ch += gridDim.z * 256) {
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

template <int NI, int KIND>
__global__ __launch_bounds__(256) void scan_kernel(Scan p, const RowSeg *__restrict__ segs) {
  constexpr int KP = 32 * NI, TC = SCAN_TOKENS;
  constexpr bool CHANNEL = KIND == SCAN_CHANNEL_DELTA, SSM = KIND == SCAN_STATE_SPACE;
  __shared__ __attribute__((aligned(16))) float sk[TC][KP], sq[TC][KP], sg[CHANNEL ? TC : 1][KP];
  __shared__ float sv[TC][SCAN_COLS], s_decay[TC], s_beta[TC];
  const RowSeg seg = segs[blockIdx.x];
  const int h = blockIdx.y;
  if (h == p.heads) {
    advance_conv_state(p, seg);
    return;
  }
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int j = lane & 7;
  const int c0 = blockIdx.z * SCAN_COLS, cw = wave * 16 + (lane >> 3) * 2;   // this lane's columns c0 + cw, + 1
  const int kh = h / (p.heads / p.key_heads);
  const float rate = expf(p.a_log[h]);
  const float bias = CHANNEL ? 0.f : p.dt_bias[h];
  const float skip = SSM ? p.d_skip[h] : 0.f;

  f32x4 S[2][NI];
  float *st = p.state + (((size_t)seg.slot * p.heads + h) * p.V + c0 + cw) * KP + 4 * j;
#pragma unroll
  for (int c = 0; c < 2; c++)
#pragma unroll
    for (int i = 0; i < NI; i++) {
      S[c][i] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (seg.pos0 > 0 && c0 + cw + c < p.V) S[c][i] = *reinterpret_cast<const f32x4 *>(st + c * KP + 32 * i);
    }

  for (int t0 = 0; t0 < seg.n; t0 += TC) {
    const int T = min(TC, seg.n - t0);
    if (t0 > 0) __syncthreads();
    for (int idx = tid; idx < T * KP; idx += 256) {
      const int t = idx / KP, d = idx - t * KP;
      const size_t row = seg.row0 + t0 + t;
      float k = 0.f, q = 0.f, g = 0.f;
      if (d < p.K) {
        const float *cr = p.conv + row * p.ld_conv + kh * p.K + d;
        k = cr[p.k_col];
        q = cr[p.q_col];
        if (CHANNEL)
          g = expf(-rate * softplus_f(p.channel_decay[row * p.ld_decay + h * p.K + d] + p.dt_bias[h * p.K + d]));
      }
      sk[t][d] = k;
      sq[t][d] = q;
      if (CHANNEL) sg[t][d] = g;
    }
    for (int idx = tid; idx < T * SCAN_COLS; idx += 256) {
      const int t = idx / SCAN_COLS, c = idx - t * SCAN_COLS;
      sv[t][c] = c0 + c < p.V ? p.conv[(size_t)(seg.row0 + t0 + t) * p.ld_conv + p.v_col + h * p.V + c0 + c] : 0.f;
    }
    if (tid < T) {
      const float *ir = p.in + (size_t)(seg.row0 + t0 + tid) * p.ld_in;
      if (SSM) {
        const float dt = softplus_f(ir[p.decay_col + h] + bias);
        s_decay[tid] = expf(-rate * dt);
        s_beta[tid] = dt;
      } else {
        s_beta[tid] = sigmoid_f(ir[p.beta_col + h]);
        if (!CHANNEL) s_decay[tid] = expf(-rate * softplus_f(ir[p.decay_col + h] + bias));
      }
    }
    __syncthreads();
    float keep[2] = {0.f, 0.f};
    for (int t = 0; t < T; t++) {
      f32x4 k[NI], q[NI];
#pragma unroll
      for (int i = 0; i < NI; i++) {
        k[i] = *reinterpret_cast<const f32x4 *>(&sk[t][32 * i + 4 * j]);
        q[i] = *reinterpret_cast<const f32x4 *>(&sq[t][32 * i + 4 * j]);
      }
      const float beta = s_beta[t];
      float v[2] = {sv[t][cw], sv[t][cw + 1]}, u[2], o[2];
      if constexpr (CHANNEL) {
#pragma unroll
        for (int i = 0; i < NI; i++) {
          const f32x4 g = *reinterpret_cast<const f32x4 *>(&sg[t][32 * i + 4 * j]);
#pragma unroll
          for (int c = 0; c < 2; c++)
#pragma unroll
            for (int e = 0; e < 4; e++) S[c][i][e] *= g[e];
        }
      } else {
        const float g = s_decay[t];
#pragma unroll
        for (int c = 0; c < 2; c++)
#pragma unroll
          for (int i = 0; i < NI; i++)
#pragma unroll
            for (int e = 0; e < 4; e++) S[c][i][e] *= g;
      }
#pragma unroll
      for (int c = 0; c < 2; c++) {
        if constexpr (SSM) {
          u[c] = beta * v[c];
        } else {
          float d0 = 0.f, d1 = 0.f;
#pragma unroll
          for (int i = 0; i < NI; i++) {
            d0 = fmaf(S[c][i][0], k[i][0], d0);
            d1 = fmaf(S[c][i][1], k[i][1], d1);
            d0 = fmaf(S[c][i][2], k[i][2], d0);
            d1 = fmaf(S[c][i][3], k[i][3], d1);
          }
          u[c] = beta * (v[c] - sum8(d0 + d1));
        }
      }
#pragma unroll
      for (int c = 0; c < 2; c++) {
        float d0 = 0.f, d1 = 0.f;
#pragma unroll
        for (int i = 0; i < NI; i++) {
#pragma unroll
          for (int e = 0; e < 4; e++) S[c][i][e] = fmaf(k[i][e], u[c], S[c][i][e]);
          d0 = fmaf(S[c][i][0], q[i][0], d0);
          d1 = fmaf(S[c][i][1], q[i][1], d1);
          d0 = fmaf(S[c][i][2], q[i][2], d0);
          d1 = fmaf(S[c][i][3], q[i][3], d1);
        }
        o[c] = sum8(d0 + d1);
        if (SSM) o[c] = fmaf(skip, v[c], o[c]);
      }
      // lane j of a group keeps the results of tokens t with t % 8 == j and stores them together
      if ((t & 7) == j) {
        keep[0] = o[0];
        keep[1] = o[1];
      }
      if ((t & 7) == 7 || t == T - 1) {
        const int tj = (t & ~7) + j;
        if (tj <= t) {
          float *dst = p.out + (size_t)(seg.row0 + t0 + tj) * p.ld_out + h * p.V + c0 + cw;
          if (c0 + cw < p.V) dst[0] = keep[0];
          if (c0 + cw + 1 < p.V) dst[1] = keep[1];
        }
      }
    }
  }
#pragma unroll
  for (int c = 0; c < 2; c++)
#pragma unroll
    for (int i = 0; i < NI; i++)
      if (c0 + cw + c < p.V) *reinterpret_cast<f32x4 *>(st + c * KP + 32 * i) = S[c][i];
}

// ---- gated output norm ---------------------------------------------------------------------------
// One wave per (row, group).
template <typename OUT>
__global__ __launch_bounds__(256) void gated_norm_kernel(GatedNorm g) {
  const int row = blockIdx.y, lane = threadIdx.x & 63;
  const int group = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  if (group >= g.groups) return;
  const float *y = g.y + (size_t)row * g.ld_y + group * g.size;
  const float *gate = g.gate + (size_t)row * g.ld_gate + group * g.size;
  const float *w = g.weight + (g.weight_per_group ? group * g.size : 0);
  float ss = 0.f;
  for (int d = lane; d < g.size; d += 64) {
    const float v = g.gate_first ? y[d] * silu_f(gate[d]) : y[d];
    ss += v * v;
  }
  const float inv = 1.f / sqrtf(wave_sum_f(ss) / g.size + g.eps);
  OUT *out = (OUT *)g.out + (size_t)row * g.ld_out + g.out_col + group * g.size;
  for (int d = lane; d < g.size; d += 64) {
    float v = g.gate_first ? y[d] * silu_f(gate[d]) : y[d];
    v = v * inv * w[d];
    if (!g.gate_first) v *= g.sigmoid_gate ? sigmoid_f(gate[d]) : silu_f(gate[d]);
    v *= g.scale;
    if constexpr (sizeof(OUT) == 2) out[d] = f32_to_bf16(v);
    else out[d] = v;
  }
}

template <typename OUT>
__global__ __launch_bounds__(256) void column_map_kernel(const float *__restrict__ in, int ld_in, int col, int width,
                                                         int relu_squared, OUT *__restrict__ out, int ld_out,
                                                         int out_col) {
  const int d = blockIdx.x * 256 + threadIdx.x;
  const size_t row = blockIdx.y;
  if (d >= width) return;
  float v = in[row * ld_in + col + d];
  if (relu_squared) {
    v = fmaxf(v, 0.f);
    v *= v;
  }
  if constexpr (sizeof(OUT) == 2) out[row * ld_out + out_col + d] = f32_to_bf16(v);
  else out[row * ld_out + out_col + d] = v;
}

// ---- launches ------------------------------------------------------------------------------------
int run_short_conv(const ShortConv &c, const StepRows &r, const float *in, int ld_in, const float *state,
                   float *out, int ld_out, hipStream_t s) {
  GPTOSS_REQUIRE(c.unit_dim <= SCAN_MAX_KEY && c.taps >= 1, GPTOSS_ERR_DIM,
                 "short_conv: heads of at most %d channels, at least one tap (%d, %d)", SCAN_MAX_KEY, c.unit_dim, c.taps);
  const int plain = c.channels - 2 * c.n_unit * c.unit_dim;
  const int units = 2 * c.n_unit + cdiv(plain, 64);
  TraceScope ts("short_conv", s);
  short_conv_kernel<<<dim3(cdiv(units, 4), r.n), 256, 0, s>>>(c, r.slots, r.lens, r.offset, in, ld_in, state, out,
                                                              ld_out, units);
  GPTOSS_LAUNCH_CHECK("short_conv_kernel");
  return GPTOSS_OK;
}

template <int NI>
static void launch_scan(const Scan &p, const StepRows &r, dim3 grid, hipStream_t s) {
  switch (p.kind) {
    case SCAN_DELTA: scan_kernel<NI, SCAN_DELTA><<<grid, 256, 0, s>>>(p, r.segs); break;
    case SCAN_CHANNEL_DELTA: scan_kernel<NI, SCAN_CHANNEL_DELTA><<<grid, 256, 0, s>>>(p, r.segs); break;
    case SCAN_STATE_SPACE: scan_kernel<NI, SCAN_STATE_SPACE><<<grid, 256, 0, s>>>(p, r.segs); break;
  }
}

int run_scan(const Scan &p, const StepRows &r, hipStream_t s) {
  GPTOSS_REQUIRE(p.K >= 1 && p.K <= SCAN_MAX_KEY && p.V >= 1 && p.key_heads >= 1 && p.heads % p.key_heads == 0,
                 GPTOSS_ERR_DIM, "scan: key dimension %d (at most %d), %d heads over %d", p.K, SCAN_MAX_KEY, p.heads,
                 p.key_heads);
  static const char *names[] = {"scan_delta", "scan_channel_delta", "scan_state_space"};
  TraceScope ts(names[p.kind], s);
  const dim3 grid(r.n_seg, p.heads + 1, cdiv(p.V, SCAN_COLS));   // y == heads: the convolution's state
  switch (scan_key_pad(p.K) / 32) {
    case 1: launch_scan<1>(p, r, grid, s); break;
    case 2: launch_scan<2>(p, r, grid, s); break;
    case 3: launch_scan<3>(p, r, grid, s); break;
    case 4: launch_scan<4>(p, r, grid, s); break;
    case 5: launch_scan<5>(p, r, grid, s); break;
    case 6: launch_scan<6>(p, r, grid, s); break;
    case 7: launch_scan<7>(p, r, grid, s); break;
    default: launch_scan<8>(p, r, grid, s); break;
  }
  GPTOSS_LAUNCH_CHECK("scan_kernel");
  return GPTOSS_OK;
}

int run_gated_norm(const GatedNorm &g, int n, hipStream_t s) {
  TraceScope ts("gated_norm", s);
  const dim3 grid(cdiv(g.groups, 4), n);
  if (g.out_f32) gated_norm_kernel<float><<<grid, 256, 0, s>>>(g);
  else gated_norm_kernel<bf16_t><<<grid, 256, 0, s>>>(g);
  GPTOSS_LAUNCH_CHECK("gated_norm_kernel");
  return GPTOSS_OK;
}

int run_column_map(const float *in, int ld_in, int col, int width, bool relu_squared, void *out, int ld_out,
                   int out_col, bool out_f32, int n, hipStream_t s) {
  TraceScope ts(relu_squared ? "relu_squared" : "column_copy", s);
  const dim3 grid(cdiv(width, 256), n);
  if (out_f32) column_map_kernel<float><<<grid, 256, 0, s>>>(in, ld_in, col, width, relu_squared, (float *)out, ld_out, out_col);
  else column_map_kernel<bf16_t><<<grid, 256, 0, s>>>(in, ld_in, col, width, relu_squared, (bf16_t *)out, ld_out, out_col);
  GPTOSS_LAUNCH_CHECK("column_map_kernel");
  return GPTOSS_OK;
}

}  // namespace gptoss
