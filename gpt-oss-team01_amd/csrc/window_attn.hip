// Attention over a sliding window or a chunk of the sequence, for the rows of a step on gfx950: decoding rows
// and stretches of prompts, any head sizes up to 256 (padded to multiples of 32 in the cache), grouped queries.
//
// The arithmetic is that of the decode attention (attn_decode.hip): scores and outputs on the matrix
// cores in transposed form, S^T = K Q^T and O^T += V^T P^T (16x16x32), K rows and V operands in 64-slot
// blocks, q and p split into bf16 hi + lo so that scores and weights keep fp32-like precision, online
// softmax in the exp2 domain.
//   * A row that is alone in its sequence: one workgroup per (row, kv head, 16 query heads); its four
//     waves take the window's blocks in turn and merge their states in LDS.
//   * A stretch of rows: one workgroup per (piece of a stretch, kv head); every K/V block of the
//     piece's range goes through LDS once and serves up to 128 queries (rows x heads), 32 per wave.
#include "window_attn.hpp"

namespace gptoss {

constexpr float WNEG = -1.0e30f;

// ---- norms and K/V store -------------------------------------------------------------------------
// Places of one position's key and value elements in the cache: the block of its slot, then kv_k_elem /
// kv_v_elem with rows of DK and DV.
struct StorePlace {
  bf16_t *blk;
  int slot, DK, DV;
  __device__ bf16_t *key(int d) const { return blk + (slot & 63) * DK + d; }
  __device__ bf16_t *value(int d) const {
    const int tt = slot & 31, within = tt & 15;
    return blk + KV_BLOCK * DK + (((slot & 63) >> 5) * (DV >> 4) + (d >> 4)) * 512 +
           ((within >> 2) * 16 + (d & 15)) * 8 + (tt >> 4) * 4 + (within & 3);
  }
};

// One wave per (RT rows, head): query heads, key heads, value heads.
template <bool F32, int RT>
__global__ __launch_bounds__(256) void window_store_kernel(WindowAttn a, const int *__restrict__ slots,
                                                           const int *__restrict__ lens, int n) {
  constexpr int PIECES = WINDOW_ATTN_MAX_DIM / 64;
  const int row0 = blockIdx.y * RT, lane = threadIdx.x & 63, live = min(RT, n - row0);
  const int unit = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int H = a.heads, G = a.kv_heads;
  if (unit >= H + 2 * G) return;
  const int DK = F32 ? a.dim : a.dim_pad(), DV = a.vdim_pad();
  const bool is_q = unit < H, is_v = unit >= H + G;
  const int head = is_q ? unit : is_v ? unit - H - G : unit - H;
  const int width = is_v ? a.vdim : a.dim, padded = F32 ? width : is_v ? DV : DK;
  const float *src = a.in + (is_q ? a.q_col : is_v ? a.v_col : a.k_col) + head * width;
  float v[PIECES][RT], ss[RT];
#pragma unroll
  for (int r = 0; r < RT; r++) ss[r] = 0.f;
#pragma unroll
  for (int i = 0; i < PIECES; i++) {
    if (64 * i >= padded) break;
    const int d = lane + 64 * i;
#pragma unroll
    for (int r = 0; r < RT; r++) v[i][r] = d < width ? src[(size_t)(row0 + min(r, live - 1)) * a.ld_in + d] : 0.f;
#pragma unroll
    for (int r = 0; r < RT; r++) ss[r] = fmaf(v[i][r], v[i][r], ss[r]);
  }
  if (!is_v) {
    const float *w = is_q ? a.q_norm : a.k_norm;
    float inv[RT];
#pragma unroll
    for (int r = 0; r < RT; r++) {
#pragma unroll
      for (int m = 32; m >= 1; m >>= 1) ss[r] += __shfl_xor(ss[r], m, 64);
      inv[r] = 1.f / sqrtf(ss[r] / a.dim + a.eps);
    }
#pragma unroll
    for (int i = 0; i < PIECES; i++) {
      if (64 * i >= padded) break;
      const int d = lane + 64 * i;
      const float wd = d < width ? w[d] : 0.f;
#pragma unroll
      for (int r = 0; r < RT; r++) v[i][r] = v[i][r] * inv[r] * wd;
    }
  }
#pragma unroll
  for (int r = 0; r < RT; r++) {
    if (r >= live) break;
    const int row = row0 + r;
    if (is_q) {
      float *dst = a.q + ((size_t)row * H + head) * DK;
#pragma unroll
      for (int i = 0; i < PIECES; i++)
        if (lane + 64 * i < DK) dst[lane + 64 * i] = v[i][r];
      continue;
    }
    const int seq = slots[row], cslot = (lens[row] - 1) % a.cap;
    if constexpr (F32) {
      float *dst = (is_v ? a.v32 : a.k32) + (((size_t)seq * a.cap + cslot) * G + head) * width;
#pragma unroll
      for (int i = 0; i < PIECES; i++)
        if (lane + 64 * i < width) dst[lane + 64 * i] = v[i][r];
    } else {
      const StorePlace at{a.kv + ((size_t)(seq * G + head) * (a.cap >> 6) + (cslot >> 6)) * a.block_elems(), cslot, DK, DV};
#pragma unroll
      for (int i = 0; i < PIECES; i++) {
        const int d = lane + 64 * i;
        if (is_v) {
          // operand order of V^T behind the block's 64 key rows
          if (d < DV) *at.value(d) = f32_to_bf16(v[i][r]);
        } else if (d < DK) {
          *at.key(d) = f32_to_bf16(v[i][r]);
        }
      }
    }
  }
}

// Norm over all heads at once, rotation, K/V store: one workgroup per RT rows, whose heads (of a multiple of four
// dimensions, rotated in neighbouring pairs, values the keys as projected) lie in its registers, four values a piece.
template <bool F32, int NV, int RT>
__global__ __launch_bounds__(256) void window_store_rows_kernel(WindowAttn a, const int *__restrict__ slots,
                                                                const int *__restrict__ lens, int n) {
  __shared__ float red[RT][2][4];
  const int row0 = blockIdx.x * RT, tid = threadIdx.x, H = a.heads, G = a.kv_heads, D = a.dim, live = min(RT, n - row0);
  const int DK = F32 ? D : a.dim_pad(), dims = a.rot.table ? a.rot.dims : 0;
  constexpr bool EARLY = RT == 1;   // angles are requested with the rows
  f32x4 x[NV][RT], w[NV], cs[EARLY ? NV : 1];
  int head[NV], d[NV], pos[RT], seq[RT];
#pragma unroll
  for (int r = 0; r < RT; r++) {
    const int row = row0 + min(r, live - 1);
    pos[r] = lens[row] - 1;
    seq[r] = slots[row];
  }
  auto angles = [&](int i, int r) {
    return head[i] < H + G && d[i] < dims ? *reinterpret_cast<const f32x4 *>(a.rot.table + (size_t)pos[r] * dims + d[i])
                                          : f32x4{1.f, 0.f, 1.f, 0.f};
  };
#pragma unroll
  for (int i = 0; i < NV; i++) {
    const int u = tid + 256 * i;
    head[i] = u / (DK >> 2);
    d[i] = (u - head[i] * (DK >> 2)) * 4;
    const bool in = head[i] < H + G && d[i] < D, is_q = head[i] < H;
    const int at = (is_q ? head[i] : head[i] - H) * D + d[i];
    w[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (in) w[i] = *reinterpret_cast<const f32x4 *>((is_q ? a.q_norm : a.k_norm) + at);
#pragma unroll
    for (int r = 0; r < RT; r++) {
      x[i][r] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (in) x[i][r] = *reinterpret_cast<const f32x4 *>(a.in + (size_t)(row0 + min(r, live - 1)) * a.ld_in + (is_q ? a.q_col : a.k_col) + at);
      if (EARLY) cs[i] = angles(i, r);
    }
  }
#pragma unroll
  for (int r = 0; r < RT; r++) {
    float ss[2] = {0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NV; i++) {
      float own = 0.f;
#pragma unroll
      for (int e = 0; e < 4; e++) own = fmaf(x[i][r][e], x[i][r][e], own);
      ss[0] += head[i] < H ? own : 0.f;
      ss[1] += head[i] < H ? 0.f : own;
    }
#pragma unroll
    for (int k = 0; k < 2; k++) {
#pragma unroll
      for (int m = 32; m >= 1; m >>= 1) ss[k] += __shfl_xor(ss[k], m, 64);
      if ((tid & 63) == 0) red[r][k][tid >> 6] = ss[k];
    }
  }
  __syncthreads();
  // four positions from a multiple of four on: a value's places are neighbours
  const bool four = RT == 4 && live == 4 && pos[0] % 4 == 0 && pos[RT - 1] == pos[0] + 3 && seq[RT - 1] == seq[0];
#pragma unroll
  for (int r = 0; r < RT; r++) {
    if (r >= live) break;
    const float inv[2] = {1.f / sqrtf((red[r][0][0] + red[r][0][1] + red[r][0][2] + red[r][0][3]) / (H * D) + a.eps),
                          1.f / sqrtf((red[r][1][0] + red[r][1][1] + red[r][1][2] + red[r][1][3]) / (G * D) + a.eps)};
    const int cslot = pos[r] % a.cap;
#pragma unroll
    for (int i = 0; i < NV; i++) {
      if (head[i] >= H + G) continue;
      const bool is_q = head[i] < H;
      const f32x4 own = x[i][r] * (is_q ? inv[0] : inv[1]) * w[i], c = EARLY ? cs[EARLY ? i : 0] : angles(i, r);
      const f32x4 y = {own[0] * c[0] - own[1] * c[1], own[1] * c[0] + own[0] * c[1],
                       own[2] * c[2] - own[3] * c[3], own[3] * c[2] + own[2] * c[3]};
      const int g = head[i] - H;
      if (is_q) {
        *reinterpret_cast<f32x4 *>(a.q + ((size_t)(row0 + r) * H + head[i]) * DK + d[i]) = y;
      } else if constexpr (F32) {
        const size_t at = (((size_t)seq[r] * a.cap + cslot) * G + g) * D + d[i];
        *reinterpret_cast<f32x4 *>(a.k32 + at) = y;
        *reinterpret_cast<f32x4 *>(a.v32 + at) = x[i][r];
      } else {
        const StorePlace at{a.kv + ((size_t)(seq[r] * G + g) * (a.cap >> 6) + (cslot >> 6)) * a.block_elems(), cslot, DK, DK};
        *reinterpret_cast<u32x2 *>(at.key(d[i])) = u32x2{pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
        bf16_t *v = at.value(d[i]);   // dimensions of a group of 16 lie 8 elements apart
        if (!four) {
#pragma unroll
          for (int e = 0; e < 4; e++) v[8 * e] = f32_to_bf16(x[i][r][e]);
        } else if (r == 0) {
#pragma unroll
          for (int e = 0; e < 4; e++)
            *reinterpret_cast<u32x2 *>(v + 8 * e) = u32x2{pack_bf16x2(x[i][0][e], x[i][RT > 1 ? 1 : 0][e]),
                                                          pack_bf16x2(x[i][RT > 2 ? 2 : 0][e], x[i][RT > 3 ? 3 : 0][e])};
        }
      }
    }
  }
}

// The same for any sizes and either layout of the rotated pairs, one workgroup per row.
template <bool F32>
__global__ __launch_bounds__(256) void window_store_row_kernel(WindowAttn a, const int *__restrict__ slots,
                                                               const int *__restrict__ lens) {
  __shared__ float red[2][4];
  const int row = blockIdx.x, tid = threadIdx.x, H = a.heads, G = a.kv_heads, D = a.dim;
  const float *q = a.in + (size_t)row * a.ld_in + a.q_col, *k = a.in + (size_t)row * a.ld_in + a.k_col;
  float ss[2] = {0.f, 0.f};
  for (int i = tid; i < H * D; i += 256) ss[0] = fmaf(q[i], q[i], ss[0]);
  for (int i = tid; i < G * D; i += 256) ss[1] = fmaf(k[i], k[i], ss[1]);
#pragma unroll
  for (int x = 0; x < 2; x++) {
#pragma unroll
    for (int m = 32; m >= 1; m >>= 1) ss[x] += __shfl_xor(ss[x], m, 64);
    if ((tid & 63) == 0) red[x][tid >> 6] = ss[x];
  }
  __syncthreads();
  const float qi = 1.f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (H * D) + a.eps);
  const float ki = 1.f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (G * D) + a.eps);
  const int DK = F32 ? D : a.dim_pad(), DV = a.vdim_pad();
  const int pos = lens[row] - 1, half = a.rot.table ? a.rot.dims >> 1 : 0, seq = slots[row], cslot = pos % a.cap;
  const float2 *cs = reinterpret_cast<const float2 *>(a.rot.table) + (size_t)pos * half;
  // element d of a head: normed, and turned with its partner
  auto value = [&](const float *x, const float *w, float inv, int head, int d) {
    const int at = head * D + d;
    const float own = x[at] * inv * w[at];
    if (d >= 2 * half) return own;
    const bool second = a.rot.interleaved ? (d & 1) != 0 : d >= half;
    const int i = a.rot.interleaved ? d >> 1 : second ? d - half : d;
    const int pt = head * D + (a.rot.interleaved ? d ^ 1 : second ? i : i + half);
    const float other = x[pt] * inv * w[pt];
    const float2 c = cs[i];
    return second ? own * c.x + other * c.y : own * c.x - other * c.y;
  };
  for (int i = tid; i < H * DK; i += 256) {
    const int head = i / DK, d = i - head * DK;
    a.q[(size_t)row * H * DK + i] = d < D ? value(q, a.q_norm, qi, head, d) : 0.f;
  }
  const float *v = a.in + (size_t)row * a.ld_in + a.v_col;
  if constexpr (F32) {
    float *kd = a.k32 + ((size_t)seq * a.cap + cslot) * G * D, *vd = a.v32 + ((size_t)seq * a.cap + cslot) * G * a.vdim;
    for (int i = tid; i < G * D; i += 256) kd[i] = value(k, a.k_norm, ki, i / D, i % D);
    for (int i = tid; i < G * a.vdim; i += 256) vd[i] = v[i];
  } else {
    for (int i = tid; i < G * DK; i += 256) {
      const int g = i / DK, d = i - g * DK;
      const StorePlace at{a.kv + ((size_t)(seq * G + g) * (a.cap >> 6) + (cslot >> 6)) * a.block_elems(), cslot, DK, DV};
      *at.key(d) = f32_to_bf16(d < D ? value(k, a.k_norm, ki, g, d) : 0.f);
    }
    for (int i = tid; i < G * DV; i += 256) {
      const int g = i / DV, d = i - g * DV;
      const StorePlace at{a.kv + ((size_t)(seq * G + g) * (a.cap >> 6) + (cslot >> 6)) * a.block_elems(), cslot, DK, DV};
      *at.value(d) = f32_to_bf16(d < a.vdim ? v[g * a.vdim + d] : 0.f);
    }
  }
}

// ---- matrix-core pieces --------------------------------------------------------------------------
// q of 16 query columns as hi + lo bf16 operands; lane (n, c) holds dimensions c*8*ks_n + 8 ks .. + 8 of
// column n.
template <int KS>
struct QFrag {
  bf16x8 hi[KS], lo[KS];
};

__device__ __forceinline__ void split8(const float (&x)[8], bf16x8 &hi, bf16x8 &lo) {
  u32x4 h, l;
#pragma unroll
  for (int e = 0; e < 4; e++) {
    h[e] = pack_bf16x2(x[2 * e], x[2 * e + 1]);
    l[e] = pack_bf16x2(x[2 * e] - __uint_as_float(h[e] << 16), x[2 * e + 1] - __uint_as_float(h[e] & 0xffff0000u));
  }
  hi = as_bf16x8(h);
  lo = as_bf16x8(l);
}

template <int KS>
__device__ __forceinline__ void load_q(QFrag<KS> &f, const float *q, int ks_n, int c, float scale) {
#pragma unroll
  for (int ks = 0; ks < KS; ks++) {
    float x[8];
#pragma unroll
    for (int e = 0; e < 8; e++) x[e] = 0.f;
    if (ks < ks_n && q) {
      const f32x4 a = *reinterpret_cast<const f32x4 *>(q + (c * ks_n + ks) * 8);
      const f32x4 b = *reinterpret_cast<const f32x4 *>(q + (c * ks_n + ks) * 8 + 4);
#pragma unroll
      for (int e = 0; e < 4; e++) {
        x[e] = a[e] * scale;
        x[4 + e] = b[e] * scale;
      }
    }
    split8(x, f.hi[ks], f.lo[ks]);
  }
}

// One 64-slot block for 16 query columns, in two halves so that a caller can request the next block's K
// between them.  kf(tb, ks) and vf(kg, db) return operands; key slot i of the block is position
// pos0 + i; the column sees positions lo..hi.
template <int KS, typename KF>
__device__ __forceinline__ void block_scores(const QFrag<KS> &q, int ks_n, f32x4 (&s)[4], KF &&kf) {
#pragma unroll
  for (int tb = 0; tb < 4; tb++) {
    s[tb] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS; ks++)
      if (ks < ks_n) {
        const bf16x8 k = kf(tb, ks);
        s[tb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, q.lo[ks], s[tb], 0, 0, 0);
        s[tb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k, q.hi[ks], s[tb], 0, 0, 0);
      }
  }
}

template <int DB, typename VF>
__device__ __forceinline__ void block_output(f32x4 (&s)[4], int db_n, int pos0, int lo, int hi, int c, float &m, float &l,
                                             f32x4 (&o)[DB], VF &&vf) {
  float mx = WNEG;
#pragma unroll
  for (int tb = 0; tb < 4; tb++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const int pos = pos0 + tb * 16 + c * 4 + e;
      s[tb][e] = (pos >= lo && pos <= hi) ? s[tb][e] : WNEG;
      mx = fmaxf(mx, s[tb][e]);
    }
  mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
  mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
  const float m_new = fmaxf(m, mx);
  const float fade = __builtin_amdgcn_exp2f(m - m_new);
  m = m_new;
  float sum = 0.f;
#pragma unroll
  for (int tb = 0; tb < 4; tb++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      // a masked slot keeps weight 0 also while nothing of the column has been seen (m == WNEG)
      s[tb][e] = s[tb][e] > 0.5f * WNEG ? __builtin_amdgcn_exp2f(s[tb][e] - m_new) : 0.f;
      sum += s[tb][e];
    }
  l = l * fade + sum;
#pragma unroll
  for (int db = 0; db < DB; db++)
#pragma unroll
    for (int e = 0; e < 4; e++) o[db][e] *= fade;
#pragma unroll
  for (int kg = 0; kg < 2; kg++) {
    float x[8];
#pragma unroll
    for (int e = 0; e < 4; e++) {
      x[e] = s[2 * kg][e];
      x[4 + e] = s[2 * kg + 1][e];
    }
    bf16x8 hi8, lo8;
    split8(x, hi8, lo8);
#pragma unroll
    for (int db = 0; db < DB; db++)
      if (db < db_n) {
        const bf16x8 v = vf(kg, db);
        o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, lo8, o[db], 0, 0, 0);
        o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, hi8, o[db], 0, 0, 0);
      }
  }
}

template <int KS, int DB, typename KF, typename VF>
__device__ __forceinline__ void attend_block(const QFrag<KS> &q, int ks_n, int db_n, int pos0, int lo, int hi, int c,
                                             float &m, float &l, f32x4 (&o)[DB], KF &&kf, VF &&vf) {
  f32x4 s[4];
  block_scores<KS>(q, ks_n, s, kf);
  block_output<DB>(s, db_n, pos0, lo, hi, c, m, l, o, vf);
}

// Row sums over the four lane groups of a column (each lane has summed its own key rows).
__device__ __forceinline__ float column_sum(float l) {
  l += __shfl_xor(l, 16, 64);
  return l + __shfl_xor(l, 32, 64);
}

// lane (n, c) stores dimensions 16 db + 4 c .. + 4 of its column
template <int DB>
__device__ __forceinline__ void store_column(bf16_t *dst, int vdim, int db_n, int c, float f, const f32x4 (&o)[DB]) {
  const bool wide = (reinterpret_cast<uintptr_t>(dst) & 7) == 0;
#pragma unroll
  for (int db = 0; db < DB; db++) {
    const int d = db * 16 + c * 4;
    if (db < db_n && d < vdim) {
      if (wide && d + 4 <= vdim) {
        *reinterpret_cast<u32x2 *>(dst + d) =
            u32x2{pack_bf16x2(o[db][0] * f, o[db][1] * f), pack_bf16x2(o[db][2] * f, o[db][3] * f)};
      } else {
#pragma unroll
        for (int e = 0; e < 4; e++)
          if (d + e < vdim) dst[d + e] = f32_to_bf16(o[db][e] * f);
      }
    }
  }
}

// ---- decoding rows -------------------------------------------------------------------------------
// EXACT: both head sizes are DMAX, so every operand has its place in registers: a wave's K and V of the next
// block are requested as soon as those of the current one have been used.
template <int DMAX, bool EXACT>
__global__ __launch_bounds__(256) void window_decode_kernel(WindowAttn a, const RowSeg *__restrict__ singles) {
  constexpr int KS = DMAX / 32, DB = DMAX / 16;
  __shared__ float so[3][DMAX][16], sm[3][16], sl[3][16];
  const RowSeg seg = singles[blockIdx.x];
  const int g = blockIdx.y, per = a.heads / a.kv_heads;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int n = lane & 15, c = lane >> 4;
  const int ks_n = EXACT ? KS : a.dim_pad() / 32, db_n = EXACT ? DB : a.vdim_pad() / 16, DK = EXACT ? DMAX : a.dim_pad();
  const size_t block = EXACT ? (size_t)KV_BLOCK * 2 * DMAX : a.block_elems();
  const int hh = blockIdx.z * 16 + n;             // head within the group
  const bool live = hh < per;
  const int head = g * per + min(hh, per - 1);
  const int hi = seg.pos0, lo = a.first(hi);
  float m = WNEG, l = 0.f;
  f32x4 o[DB];
#pragma unroll
  for (int db = 0; db < DB; db++) o[db] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int ring = a.cap >> 6;
  const bf16_t *plane = a.kv + (size_t)(seg.slot * a.kv_heads + g) * ring * block;
  const size_t k_lane = n * DK + c * ks_n * 8, v_lane = KV_BLOCK * DK + lane * 8;
  const int b_last = hi >> 6;
  int b = (lo >> 6) + wave, rb = b % ring;   // block and its place in the ring
  auto fetch = [](const bf16_t *x) { return __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(x)); };
  if constexpr (EXACT) {
    u32x4 kr[4][KS], vr[2][DB];
    auto load_k = [&](int at) {
      const bf16_t *x = plane + (size_t)at * block + k_lane;
#pragma unroll
      for (int tb = 0; tb < 4; tb++)
#pragma unroll
        for (int ks = 0; ks < KS; ks++) kr[tb][ks] = fetch(x + tb * 16 * DMAX + ks * 8);
    };
    auto load_v = [&](int at) {
      const bf16_t *x = plane + (size_t)at * block + v_lane;
#pragma unroll
      for (int kg = 0; kg < 2; kg++)
#pragma unroll
        for (int db = 0; db < DB; db++) vr[kg][db] = fetch(x + (kg * DB + db) * 512);
    };
    if (b <= b_last) {
      load_k(rb);
      load_v(rb);
    }
    QFrag<KS> q;
    load_q<KS>(q, a.q + ((size_t)seg.row0 * a.heads + head) * DK, ks_n, c, a.scale * 1.4426950408889634f);
    while (b <= b_last) {
      const int next = b + 4 <= b_last ? (rb + 4) % ring : rb;   // past the end: this block again, unused
      f32x4 s[4];
      block_scores<KS>(q, KS, s, [&](int tb, int ks) { return as_bf16x8(kr[tb][ks]); });
      load_k(next);
      block_output<DB>(s, DB, b << 6, lo, hi, c, m, l, o, [&](int kg, int db) { return as_bf16x8(vr[kg][db]); });
      load_v(next);
      b += 4;
      rb = next;
    }
  } else {
    QFrag<KS> q;
    load_q<KS>(q, a.q + ((size_t)seg.row0 * a.heads + head) * DK, ks_n, c, a.scale * 1.4426950408889634f);
    for (; b <= b_last; b += 4) {
      const bf16_t *blk = plane + (size_t)(b % ring) * block;
      attend_block<KS, DB>(q, ks_n, db_n, b << 6, lo, hi, c, m, l, o,
                           [&](int tb, int ks) { return as_bf16x8(fetch(blk + k_lane + tb * 16 * DK + ks * 8)); },
                           [&](int kg, int db) { return as_bf16x8(fetch(blk + v_lane + (kg * db_n + db) * 512)); });
    }
  }
  l = column_sum(l);
  if (wave > 0) {
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
      for (int e = 0; e < 4; e++) so[wave - 1][db * 16 + c * 4 + e][n] = o[db][e];
    if (c == 0) {
      sm[wave - 1][n] = m;
      sl[wave - 1][n] = l;
    }
  }
  __syncthreads();
  if (wave > 0 || !live) return;
  for (int w = 0; w < 3; w++) {
    const float mw = sm[w][n], m_new = fmaxf(m, mw);
    const float f0 = __builtin_amdgcn_exp2f(m - m_new), f1 = __builtin_amdgcn_exp2f(mw - m_new);
    m = m_new;
    l = l * f0 + sl[w][n] * f1;
#pragma unroll
    for (int db = 0; db < DB; db++)
#pragma unroll
      for (int e = 0; e < 4; e++) o[db][e] = o[db][e] * f0 + so[w][db * 16 + c * 4 + e][n] * f1;
  }
  store_column<DB>((bf16_t *)a.out + (size_t)seg.row0 * a.ld_out + a.out_col + head * a.vdim, a.vdim, db_n, c,
                   a.out_scale / l, o);
}

// ---- stretches of rows ---------------------------------------------------------------------------
template <int DMAX>
__global__ __launch_bounds__(256, DMAX > 128 ? 1 : 2) void window_tile_kernel(WindowAttn a, const RowSeg *__restrict__ tiles) {
  constexpr int KS = DMAX / 32, DB = DMAX / 16;
  constexpr int CH = DMAX * 2 * KV_BLOCK * 2 / 16 / 256;   // 16-byte pieces of a K/V block per thread
  // K rows padded by 16 bytes against bank conflicts, then V in operand order
  __shared__ __attribute__((aligned(16))) bf16_t lds[KV_BLOCK * (DMAX + 8) + KV_BLOCK * DMAX];
  const RowSeg seg = tiles[blockIdx.x];
  const int g = blockIdx.y, per = a.heads / a.kv_heads;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 15, c = lane >> 4;
  const int DK = a.dim_pad(), DV = a.vdim_pad(), ks_n = DK / 32, db_n = DV / 16;
  const int kstride = DK + 8, vbase = KV_BLOCK * kstride;
  const int k_pieces = KV_BLOCK * DK / 8, pieces = k_pieces + KV_BLOCK * DV / 8, row_pieces = DK / 8;
  const int ring = a.cap >> 6;
  const bf16_t *plane = a.kv + (size_t)(seg.slot * a.kv_heads + g) * ring * a.block_elems();
  const int queries = seg.n * per;
  u32x4 stage[CH];
  auto fetch = [&](int b) {
    const u32x4 *src = reinterpret_cast<const u32x4 *>(plane + (size_t)(b % ring) * a.block_elems());
#pragma unroll
    for (int i = 0; i < CH; i++)
      if (tid + 256 * i < pieces) stage[i] = src[tid + 256 * i];
  };
  auto put = [&]() {
#pragma unroll
    for (int i = 0; i < CH; i++) {
      const int x = tid + 256 * i;
      if (x < pieces) {
        const int at = x < k_pieces ? (x / row_pieces) * kstride + (x % row_pieces) * 8 : vbase + (x - k_pieces) * 8;
        *reinterpret_cast<u32x4 *>(lds + at) = stage[i];
      }
    }
  };
  for (int q0 = 0; q0 < queries; q0 += 128) {
    // this pass: queries q0 .. q0 + 127; wave w has columns q0 + 32 w .. + 31 in two tiles of 16
    QFrag<KS> q[2];
    int lo[2], hi[2], qi[2];
    float m[2] = {WNEG, WNEG}, l[2] = {0.f, 0.f};
    f32x4 o[2][DB];
#pragma unroll
    for (int i = 0; i < 2; i++) {
      qi[i] = q0 + wave * 32 + i * 16 + n;
      const int use = min(qi[i], queries - 1), r = use / per;
      hi[i] = seg.pos0 + r;
      lo[i] = a.first(hi[i]);
      load_q<KS>(q[i], a.q + ((size_t)(seg.row0 + r) * a.heads + g * per + (use - r * per)) * DK, ks_n, c,
                 a.scale * 1.4426950408889634f);
#pragma unroll
      for (int db = 0; db < DB; db++) o[i][db] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const int r_first = q0 / per, r_last = min(q0 + 127, queries - 1) / per;
    const int b_lo = a.first(seg.pos0 + r_first) >> 6, b_hi = (seg.pos0 + r_last) >> 6;
    const bool busy0 = q0 + wave * 32 < queries, busy1 = q0 + wave * 32 + 16 < queries;   // wave-uniform
    fetch(b_lo);
    for (int b = b_lo; b <= b_hi; b++) {
      __syncthreads();
      put();
      __syncthreads();
      if (b < b_hi) fetch(b + 1);
      const bf16_t *kl = lds + n * kstride + c * ks_n * 8, *vl = lds + vbase + lane * 8;
      auto kf = [&](int tb, int ks) { return as_bf16x8(*reinterpret_cast<const u32x4 *>(kl + tb * 16 * kstride + ks * 8)); };
      auto vf = [&](int kg, int db) { return as_bf16x8(*reinterpret_cast<const u32x4 *>(vl + (kg * db_n + db) * 512)); };
      if (busy0) attend_block<KS, DB>(q[0], ks_n, db_n, b << 6, lo[0], hi[0], c, m[0], l[0], o[0], kf, vf);
      if (busy1) attend_block<KS, DB>(q[1], ks_n, db_n, b << 6, lo[1], hi[1], c, m[1], l[1], o[1], kf, vf);
    }
#pragma unroll
    for (int i = 0; i < 2; i++) {
      const float sum = column_sum(l[i]);
      if (qi[i] < queries) {
        const int r = qi[i] / per;
        store_column<DB>((bf16_t *)a.out + (size_t)(seg.row0 + r) * a.ld_out + a.out_col +
                             (g * per + (qi[i] - r * per)) * a.vdim,
                         a.vdim, db_n, c, a.out_scale / sum, o[i]);
      }
    }
  }
}

// ---- fp32 ----------------------------------------------------------------------------------------
// One workgroup per (row, head): online softmax over tiles of 256 positions.
__global__ __launch_bounds__(256) void window_f32_kernel(WindowAttn a, const int *__restrict__ slots,
                                                         const int *__restrict__ lens) {
  __shared__ float sq[WINDOW_ATTN_MAX_DIM], sp[256], red[8];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int g = h / (a.heads / a.kv_heads);
  const int hi = lens[row] - 1, lo = a.first(hi);
  const size_t base = (size_t)slots[row] * a.cap;
  if (tid < a.dim) sq[tid] = a.q[((size_t)row * a.heads + h) * a.dim + tid];
  __syncthreads();
  float m = -INFINITY, l = 0.f, o = 0.f;
  for (int p0 = lo; p0 <= hi; p0 += 256) {
    const int pos = p0 + tid;
    float s = -INFINITY;
    if (pos <= hi) {
      const float *k = a.k32 + ((base + pos % a.cap) * a.kv_heads + g) * a.dim;
      s = 0.f;
      for (int d = 0; d < a.dim; d++) s = fmaf(sq[d], k[d], s);
      s *= a.scale;
    }
    float mx = s;
    for (int x = 32; x >= 1; x >>= 1) mx = fmaxf(mx, __shfl_xor(mx, x, 64));
    if (lane == 0) red[wave] = mx;
    __syncthreads();
    const float m_new = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float e = pos <= hi ? expf(s - m_new) : 0.f;
    sp[tid] = e;
    float sum = e;
    for (int x = 32; x >= 1; x >>= 1) sum += __shfl_xor(sum, x, 64);
    if (lane == 0) red[4 + wave] = sum;
    __syncthreads();
    const float fade = expf(m - m_new);   // 0 on the first tile
    m = m_new;
    l = l * fade + ((red[4] + red[5]) + (red[6] + red[7]));
    if (tid < a.vdim) {
      o *= fade;
      const int cnt = min(256, hi - p0 + 1);
      for (int i = 0; i < cnt; i++)
        o = fmaf(sp[i], a.v32[((base + (p0 + i) % a.cap) * a.kv_heads + g) * a.vdim + tid], o);
    }
    __syncthreads();
  }
  if (tid < a.vdim)
    ((float *)a.out)[(size_t)row * a.ld_out + a.out_col + h * a.vdim + tid] = o / l * a.out_scale;
}

// ---- launches ------------------------------------------------------------------------------------
template <bool F32>
static void launch_store_rows(const WindowAttn &a, const StepRows &r, hipStream_t s) {
  const bool pieces = a.dim % 4 == 0 && a.v_col == a.k_col && a.vdim == a.dim && a.ld_in % 4 == 0 && a.q_col % 4 == 0 &&
                      a.k_col % 4 == 0 && aligned(a.in, 16) && aligned(a.q_norm, 16) && aligned(a.k_norm, 16) &&
                      (!a.rot.table || (a.rot.interleaved && a.rot.dims % 4 == 0));
  const int per_thread = cdiv((a.heads + a.kv_heads) * ((F32 ? a.dim : a.dim_pad()) / 4), 256);
  auto go = [&](auto kern, int rt) { kern<<<cdiv(r.n, rt), 256, 0, s>>>(a, r.slots, r.lens, r.n); };
  if (!pieces || per_thread > 8) {
    window_store_row_kernel<F32><<<r.n, 256, 0, s>>>(a, r.slots, r.lens);
  } else if (!F32 && r.n >= 1024 && per_thread <= 5) {
    if constexpr (!F32) {
      if (per_thread <= 1) go(window_store_rows_kernel<F32, 1, 4>, 4);
      else if (per_thread <= 2) go(window_store_rows_kernel<F32, 2, 4>, 4);
      else if (per_thread <= 3) go(window_store_rows_kernel<F32, 3, 4>, 4);
      else go(window_store_rows_kernel<F32, 5, 4>, 4);
    }
  } else if (per_thread <= 1) {
    go(window_store_rows_kernel<F32, 1, 1>, 1);
  } else if (per_thread <= 3) {
    go(window_store_rows_kernel<F32, 3, 1>, 1);
  } else if (per_thread <= 5) {
    go(window_store_rows_kernel<F32, 5, 1>, 1);
  } else {
    go(window_store_rows_kernel<F32, 8, 1>, 1);
  }
}

int run_window_attn(const WindowAttn &a, const StepRows &r, hipStream_t s) {
  GPTOSS_REQUIRE(a.dim >= 1 && a.dim <= WINDOW_ATTN_MAX_DIM && a.vdim >= 1 && a.vdim <= WINDOW_ATTN_MAX_DIM &&
                     a.kv_heads >= 1 && a.heads % a.kv_heads == 0 && a.window >= 1 && a.cap % 64 == 0,
                 GPTOSS_ERR_DIM, "window_attn: heads of at most %d (%d, %d), %d query over %d kv heads, window %d",
                 WINDOW_ATTN_MAX_DIM, a.dim, a.vdim, a.heads, a.kv_heads, a.window);
  GPTOSS_REQUIRE(r.max_len <= a.cap || a.window - 1 + r.longest <= a.cap, GPTOSS_ERR_DIM,
                 "window_attn: a ring of %d slots cannot hold a window of %d and %d rows", a.cap, a.window, r.longest);
  GPTOSS_REQUIRE(a.whole_norm || !a.rot.table, GPTOSS_ERR_DIM, "window_attn: rotation needs a norm over the whole projection");
  GPTOSS_REQUIRE(!a.rot.table || (a.rot.dims >= 2 && a.rot.dims % 2 == 0 && a.rot.dims <= a.dim), GPTOSS_ERR_DIM,
                 "window_attn: %d of %d dimensions rotated (an even number)", a.rot.dims, a.dim);
  const int units = a.heads + 2 * a.kv_heads;
  if (a.k32) {
    {
      TraceScope ts("window_store", s);
      if (a.whole_norm) launch_store_rows<true>(a, r, s);
      else window_store_kernel<true, 1><<<dim3(cdiv(units, 4), r.n), 256, 0, s>>>(a, r.slots, r.lens, r.n);
    }
    GPTOSS_LAUNCH_CHECK("window_store_kernel");
    TraceScope ts("window_attn_f32", s);
    window_f32_kernel<<<dim3(a.heads, r.n), 256, 0, s>>>(a, r.slots, r.lens);
    GPTOSS_LAUNCH_CHECK("window_f32_kernel");
    return GPTOSS_OK;
  }
  {
    TraceScope ts("window_store", s);
    if (a.whole_norm) launch_store_rows<false>(a, r, s);
    else if (r.n >= 1024) window_store_kernel<false, 4><<<dim3(cdiv(units, 4), cdiv(r.n, 4)), 256, 0, s>>>(a, r.slots, r.lens, r.n);
    else window_store_kernel<false, 1><<<dim3(cdiv(units, 4), r.n), 256, 0, s>>>(a, r.slots, r.lens, r.n);
  }
  GPTOSS_LAUNCH_CHECK("window_store_kernel");
  const int widest = std::max(a.dim, a.vdim);
  if (r.n_singles) {
    TraceScope ts("window_decode", s);
    const dim3 grid(r.n_singles, a.kv_heads, cdiv(a.heads / a.kv_heads, 16));
    const bool both = a.dim_pad() == a.vdim_pad();
    if (widest <= 64)
      both && a.dim_pad() == 64 ? window_decode_kernel<64, true><<<grid, 256, 0, s>>>(a, r.singles)
                                : window_decode_kernel<64, false><<<grid, 256, 0, s>>>(a, r.singles);
    else if (widest <= 128)
      both && a.dim_pad() == 128 ? window_decode_kernel<128, true><<<grid, 256, 0, s>>>(a, r.singles)
                                 : window_decode_kernel<128, false><<<grid, 256, 0, s>>>(a, r.singles);
    else window_decode_kernel<256, false><<<grid, 256, 0, s>>>(a, r.singles);
    GPTOSS_LAUNCH_CHECK("window_decode_kernel");
  }
  const StepRows::Tiles &t = r.tiles[a.tiles];
  if (t.n) {
    TraceScope ts("window_tiles", s);
    const dim3 grid(t.n, a.kv_heads);
    if (widest <= 64) window_tile_kernel<64><<<grid, 256, 0, s>>>(a, t.tiles);
    else if (widest <= 128) window_tile_kernel<128><<<grid, 256, 0, s>>>(a, t.tiles);
    else window_tile_kernel<256><<<grid, 256, 0, s>>>(a, t.tiles);
    GPTOSS_LAUNCH_CHECK("window_tile_kernel");
  }
  return GPTOSS_OK;
}

}  // namespace gptoss
