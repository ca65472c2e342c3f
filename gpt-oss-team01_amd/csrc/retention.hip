// Retention over the rows of a step on gfx950: S_t = d S_(t-1) + k_t v_t^T, o_t = S_t^T q_t with a fixed decay d per
// head, in chunks of C tokens on the matrix cores.  With t and s counting from the chunk's first token and S the
// state in front of it
//   o_t = d^(t+1) S^T q_t + sum_{s <= t} d^(t-s) (k_s . q_t) v_s
//   S  <- d^C S + sum_s d^(C-1-s) k_s v_s^T
// A workgroup has one head's state columns c0 .. c0 + 63 of one sequence, a wave 16 of them, in fp32 registers
// (accumulators of the second line).  Every operand, the state's copy for the first line included, enters the matrix
// cores as bf16 hi + lo parts (products hi hi + hi lo + lo hi), so that sums keep about 16 bits of each factor; only
// powers 0 .. C of d occur.  Tokens are rotated where they are staged.
//
// Reduction indices are taken in the order in which a 16x16 result lies in its lanes: the eight elements of lane
// group c (lane >> 4) in a step of 32 are 4c .. 4c + 3 and 16 + 4c .. 16 + 4c + 3.  Two result tiles side by side are
// then an operand as they are.
#include "recurrent.hpp"

namespace gptoss {

struct Split4 {
  u32x2 hi, lo;
};
__device__ __forceinline__ Split4 split4(f32x4 x) {
  Split4 s;
#pragma unroll
  for (int e = 0; e < 2; e++) {
    s.hi[e] = pack_bf16x2(x[2 * e], x[2 * e + 1]);
    s.lo[e] = pack_bf16x2(x[2 * e] - __uint_as_float(s.hi[e] << 16), x[2 * e + 1] - __uint_as_float(s.hi[e] & 0xffff0000u));
  }
  return s;
}

struct Operand {
  bf16x8 hi, lo;
};
__device__ __forceinline__ Operand make_operand(f32x4 a, f32x4 b) {
  const Split4 x = split4(a), y = split4(b);
  return {as_bf16x8(u32x4{x.hi[0], x.hi[1], y.hi[0], y.hi[1]}), as_bf16x8(u32x4{x.lo[0], x.lo[1], y.lo[0], y.lo[1]})};
}
// `lo` elements behind `hi`
__device__ __forceinline__ Operand read_operand(const bf16_t *at, int lo) {
  return {as_bf16x8(*reinterpret_cast<const u32x4 *>(at)), as_bf16x8(*reinterpret_cast<const u32x4 *>(at + lo))};
}
__device__ __forceinline__ void multiply_add(f32x4 &acc, const Operand &a, const Operand &b) {
  acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.lo, b.hi, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.hi, b.lo, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.hi, b.hi, acc, 0, 0, 0);
}
// place of element i (a multiple of 4) of a row in operand order
__device__ __forceinline__ constexpr int operand_place(int i) { return (i & ~31) + ((i >> 2) & 3) * 8 + ((i >> 4) & 1) * 4; }

// Keys of 32 NI dimensions (padded), chunks of C tokens.
template <int NI, int C>
struct RetentionTile {
  static constexpr int KP = 32 * NI, TT = C / 16, SG = C / 32;
  static constexpr int ROW = KP + 8, COL = C + 8;   // rows of an operand matrix, 16 bytes apart in their banks
  // hi parts, then lo parts
  static constexpr int Q = 0, K = Q + 2 * C * ROW, KT = K + 2 * C * ROW, P = KT + 2 * KP * COL, X = P + 2 * TT * SG * 512;
  static constexpr int ELEMS = X + 8 * (TT / 2) * 64 * 8;   // X: fp32
};

// Waves w and w + 4 share 16 columns: the first has the lower half of their state (by key dimension) and, in the end,
// of the chunk's rows.  The first four waves stage keys, the others queries.
template <int NI, int C>
__global__ __launch_bounds__(512) void retention_chunk_kernel(Scan p, const RowSeg *__restrict__ segs, int n_seg) {
  using L = RetentionTile<NI, C>;
  constexpr int KP = L::KP, TT = L::TT, SG = L::SG, UPT = KP / 8;   // units of 8 dimensions x 4 tokens
  constexpr int OWN = TT * TT > 8 ? TT * TT / 8 : 1;                // tiles of the token products per wave
  constexpr int NK = (NI + 1) / 2, HT = TT / 2;                     // of a wave: 32-key steps (at most), row tiles
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  const int seg_id = blockIdx.x % n_seg, unit = blockIdx.x / n_seg, blocks = (p.V + 63) / 64;
  const RowSeg seg = segs[seg_id];
  const int h = unit / blocks, kh = h / (p.heads / p.key_heads);
  const int tid = threadIdx.x & 255, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int half = wave >> 2, k0 = half * NK, n_k = half ? NI - NK : NK;
  const int n = lane & 15, c = lane >> 4;
  const int c0 = (unit - h * blocks) * 64 + (wave & 3) * 16, col = min(c0 + n, p.V - 1);   // columns c0 .. + 15 of the wave
  const bool live = c0 + n < p.V;
  const float *power = p.decay_powers + h * (RETENTION_CHUNK + 1);

  f32x4 S[2 * NK];   // d = 32 k0 + 16 b + 4 c + e of column c0 + n
  float *st = p.state + (((size_t)seg.slot * p.heads + h) * p.V + col) * KP + 32 * k0 + 4 * c;
#pragma unroll
  for (int b = 0; b < 2 * NK; b++) {
    S[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (seg.pos0 > 0 && live && b < 2 * n_k) S[b] = __builtin_nontemporal_load(reinterpret_cast<const f32x4 *>(st + 16 * b));
  }

  // powers that do not change from chunk to chunk: of this wave's tiles of token products, and of the rows of the output
  const int p_t = wave % TT, p_s = wave / TT;   // token tile of the queries; tiles p_s, p_s + 8 / TT, .. of the keys
  float tri[OWN][4], from[TT];
#pragma unroll
  for (int i = 0; i < OWN; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const int back = p_t * 16 + n - ((p_s + i * (8 / TT)) * 16 + 4 * c + e);
      tri[i][e] = back >= 0 ? p.value_scale * power[max(back, 0)] : 0.f;
    }
#pragma unroll
  for (int t = 0; t < TT; t++) from[t] = power[t * 16 + n + 1];

  // One staging unit per thread: dimensions d0 .. + 3 and d1 .. + 3 (partners where they are rotated) of tokens
  // 4 a .. 4 a + 3.  Addresses are a base per workgroup and a 32-bit offset per lane.
  const int y = tid % UPT, a = tid / UPT, pairs = p.rot.table ? p.rot.dims >> 1 : 0;
  const bool stages = UPT * (C / 4) == 256 || a < C / 4, turned = 4 * y < pairs, keys = half == 0;
  const int d0 = turned ? 4 * y : 2 * pairs + 8 * (y - pairs / 4), d1 = turned ? 4 * y + pairs : d0 + 4;
  const unsigned x0 = 4 * min(d0, p.K - 4), x1 = 4 * min(d1, p.K - 4), x_cs = 8 * min(4 * y, max(pairs - 4, 0));
  const unsigned ld = 4 * p.ld_conv, ld_cs = 8 * pairs;   // in bytes
  const int src_col = (keys ? p.k_col : p.q_col) + kh * p.K;
  auto at4 = [](const void *base, unsigned offset) {
    return *reinterpret_cast<const f32x4 *>(static_cast<const char *>(base) + offset);
  };
  f32x4 rx[4][2], cs[4][2];
  float rv[SG * 8], rw[4], fade;
#pragma unroll
  for (int i = 0; i < 4; i++)
#pragma unroll
    for (int x = 0; x < 2; x++) rx[i][x] = cs[i][x] = f32x4{0.f, 0.f, 0.f, 0.f};
  auto fetch = [&](int t0) {
    const int T = min(C, seg.n - t0);
    const float *rows = p.conv + (size_t)(seg.row0 + t0) * p.ld_conv;
    const float *src = rows + src_col, *v = rows + p.v_col + h * p.V;
    const float *angles = p.rot.table + (size_t)(seg.pos0 + t0) * pairs * 2;
    fade = power[T];
    if (stages) {
      unsigned t[4];
#pragma unroll
      for (int i = 0; i < 4; i++) t[i] = min(4 * a + i, T - 1);
#pragma unroll
      for (int i = 0; i < 4; i++) {
        rx[i][0] = at4(src, t[i] * ld + x0);
        rx[i][1] = at4(src, t[i] * ld + x1);
        rw[i] = power[max(T - 1 - (4 * a + i), 0)];
      }
      if (pairs)
#pragma unroll
        for (int i = 0; i < 4; i++) {
          cs[i][0] = at4(angles, t[i] * ld_cs + x_cs);
          cs[i][1] = at4(angles, t[i] * ld_cs + x_cs + 16);
        }
    }
#pragma unroll
    for (int x = 0; x < SG * 8; x++) {
      const int t = (x >> 3) * 32 + ((x >> 2) & 1) * 16 + 4 * c + (x & 3);
      rv[x] = *reinterpret_cast<const float *>(reinterpret_cast<const char *>(v) + (min(t, T - 1) * ld + 4 * col));
    }
  };
  auto put = [&](int T) {
    if (!stages) return;
    if (T < C || p.K < KP) {   // rows and columns outside the problem
#pragma unroll
      for (int i = 0; i < 4; i++)
#pragma unroll
        for (int x = 0; x < 2; x++) {
          const bool out = (x ? d1 : d0) >= p.K || 4 * a + i >= T;
#pragma unroll
          for (int e = 0; e < 4; e++) rx[i][x][e] = out ? 0.f : rx[i][x][e];
        }
    }
    bf16_t *rows = lds + (keys ? L::K : L::Q);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      f32x4 z[2];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const float cosine = turned ? cs[i][e >> 1][2 * (e & 1)] : 1.f, sine = turned ? cs[i][e >> 1][2 * (e & 1) + 1] : 0.f;
        z[0][e] = rx[i][0][e] * cosine - rx[i][1][e] * sine;
        z[1][e] = rx[i][1][e] * cosine + rx[i][0][e] * sine;
      }
#pragma unroll
      for (int x = 0; x < 2; x++) {
        const int at = (4 * a + i) * L::ROW + operand_place(x ? d1 : d0);
        const Split4 s = split4(z[x]);
        *reinterpret_cast<u32x2 *>(rows + at) = s.hi;
        *reinterpret_cast<u32x2 *>(rows + C * L::ROW + at) = s.lo;
        rx[i][x] = z[x] * (p.value_scale * rw[i]);
      }
    }
    if (!keys) return;
#pragma unroll
    for (int x = 0; x < 2; x++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const Split4 s = split4(f32x4{rx[0][x][e], rx[1][x][e], rx[2][x][e], rx[3][x][e]});
        const int at = ((x ? d1 : d0) + e) * L::COL + operand_place(4 * a);
        *reinterpret_cast<u32x2 *>(lds + L::KT + at) = s.hi;
        *reinterpret_cast<u32x2 *>(lds + L::KT + KP * L::COL + at) = s.lo;
      }
  };

  // Every tile is multiplied, also where a chunk has fewer tokens or a tile lies behind its queries: the operands or
  // the powers are zero there.
  fetch(0);
  for (int t0 = 0; t0 < seg.n; t0 += C) {
    const int T = min(C, seg.n - t0);
    put(T);   // the last reads of Q, K and KT lie before the barrier in front of the previous chunk's last products
    if (T < C || c0 + 16 > p.V) {
#pragma unroll
      for (int x = 0; x < SG * 8; x++) {
        const int t = (x >> 3) * 32 + ((x >> 2) & 1) * 16 + 4 * c + (x & 3);
        rv[x] = t < T && live ? rv[x] : 0.f;
      }
    }
    Operand v[SG];
#pragma unroll
    for (int x = 0; x < SG; x++)
      v[x] = make_operand(f32x4{rv[8 * x], rv[8 * x + 1], rv[8 * x + 2], rv[8 * x + 3]},
                          f32x4{rv[8 * x + 4], rv[8 * x + 5], rv[8 * x + 6], rv[8 * x + 7]});
    const float faded = fade;
    __syncthreads();
    if (t0 + C < seg.n) fetch(t0 + C);

    // products of keys and queries, [key][query], masked and decayed, in operand order
    if (TT * TT >= 8 || wave < TT * TT) {
      f32x4 prod[OWN];
#pragma unroll
      for (int i = 0; i < OWN; i++) prod[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < NI; ks++) {
        const Operand q = read_operand(lds + L::Q + (p_t * 16 + n) * L::ROW + ks * 32 + c * 8, C * L::ROW);
#pragma unroll
        for (int i = 0; i < OWN; i++)
          multiply_add(prod[i], read_operand(lds + L::K + ((p_s + i * (8 / TT)) * 16 + n) * L::ROW + ks * 32 + c * 8, C * L::ROW), q);
      }
#pragma unroll
      for (int i = 0; i < OWN; i++) {
        const int s = p_s + i * (8 / TT);
        f32x4 w;
#pragma unroll
        for (int e = 0; e < 4; e++) w[e] = prod[i][e] * tri[i][e];
        const Split4 x = split4(w);
        bf16_t *at = lds + L::P + ((p_t * SG + s / 2) * 64 + lane) * 8 + (s & 1) * 4;
        *reinterpret_cast<u32x2 *>(at) = x.hi;
        *reinterpret_cast<u32x2 *>(at + TT * SG * 512) = x.lo;
      }
    }

    // what this half of the state in front of the chunk gives: [column][query]
    f32x4 o[TT];
#pragma unroll
    for (int t = 0; t < TT; t++) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < NK; ks++) {
      if (NI % 2 && ks >= n_k) break;
      const Operand s = make_operand(S[2 * ks], S[2 * ks + 1]);
#pragma unroll
      for (int t = 0; t < TT; t++)
        multiply_add(o[t], s, read_operand(lds + L::Q + (t * 16 + n) * L::ROW + (k0 + ks) * 32 + c * 8, C * L::ROW));
    }
    // the other wave's rows go to it
    f32x4 mine[HT];
    f32x4 *exchange = reinterpret_cast<f32x4 *>(lds + L::X) + lane;
#pragma unroll
    for (int i = 0; i < HT; i++) {
      mine[i] = half ? o[HT + i] * from[HT + i] : o[i] * from[i];
      exchange[(wave * HT + i) * 64] = half ? o[i] * from[i] : o[HT + i] * from[HT + i];
    }

    // the state behind it
#pragma unroll
    for (int b = 0; b < 2 * NK; b++) {
      if (NI % 2 && b >= 2 * n_k) break;
      S[b] *= faded;
#pragma unroll
      for (int x = 0; x < SG; x++)
        multiply_add(S[b], read_operand(lds + L::KT + (k0 * 32 + b * 16 + n) * L::COL + x * 32 + c * 8, KP * L::COL), v[x]);
    }
    __syncthreads();

#pragma unroll
    for (int i = 0; i < HT; i++) mine[i] += exchange[((wave ^ 4) * HT + i) * 64];
#pragma unroll
    for (int x = 0; x < SG; x++) {
      if (x > (half * HT + HT - 1) / 2) break;   // behind the queries
#pragma unroll
      for (int i = 0; i < HT; i++)
        multiply_add(mine[i], v[x], read_operand(lds + L::P + (((half * HT + i) * SG + x) * 64 + lane) * 8, TT * SG * 512));
    }
    const int first = c0 + 4 * c, row = half * HT * 16 + n;
    float *out = p.out + (size_t)(seg.row0 + t0) * p.ld_out + h * p.V;
    if (p.vec && T == C && c0 + 16 <= p.V) {
#pragma unroll
      for (int i = 0; i < HT; i++) *reinterpret_cast<f32x4 *>(out + (unsigned)((row + i * 16) * p.ld_out + first)) = mine[i];
    } else {
#pragma unroll
      for (int i = 0; i < HT; i++)
#pragma unroll
        for (int e = 0; e < 4; e++)
          if (row + i * 16 < T && first + e < p.V) out[(row + i * 16) * p.ld_out + first + e] = mine[i][e];
    }
  }
  if (live) {
#pragma unroll
    for (int b = 0; b < 2 * NK; b++)
      if (b < 2 * n_k) __builtin_nontemporal_store(S[b], reinterpret_cast<f32x4 *>(st + 16 * b));
  }
}

template <int NI>
static int launch_chunks(const Scan &p, const StepRows &r, hipStream_t s) {
  constexpr int C = NI <= 4 ? RETENTION_CHUNK : 32;
  constexpr int bytes = RetentionTile<NI, C>::ELEMS * (int)sizeof(bf16_t);
  auto kern = retention_chunk_kernel<NI, C>;
  static bool ready = false;
  if (!ready) {
    GPTOSS_HIP(hipFuncSetAttribute(reinterpret_cast<const void *>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, bytes));
    ready = true;
  }
  TraceScope ts("retention_chunks", s);
  kern<<<(unsigned)((size_t)r.n_seg * p.heads * cdiv(p.V, 64)), 512, bytes, s>>>(p, r.segs, r.n_seg);
  GPTOSS_LAUNCH_CHECK("retention_chunk_kernel");
  return GPTOSS_OK;
}

int run_retention(const Scan &scan, const StepRows &r, bool tokens_only, float *rows, hipStream_t s) {
  Scan p = scan;
  GPTOSS_REQUIRE(p.kind == SCAN_RETENTION && p.conv == rows && p.k_col == p.q_col + p.key_heads * p.K, GPTOSS_ERR_DIM,
                 "retention: keys must follow the queries of the same rows");
  GPTOSS_REQUIRE(p.K >= 1 && p.K <= SCAN_MAX_KEY && p.V >= 1 && p.key_heads >= 1 && p.heads % p.key_heads == 0, GPTOSS_ERR_DIM,
                 "retention: key dimension %d (at most %d), %d heads over %d", p.K, SCAN_MAX_KEY, p.heads, p.key_heads);
  GPTOSS_REQUIRE((long long)r.n_seg * p.heads * cdiv(p.V, 64) < (1ll << 31), GPTOSS_ERR_DIM, "retention: too many workgroups");
  // whole rotation groups of four, rows read 16 bytes at a time
  const bool rot_ok = !p.rot.table || (!p.rot.interleaved && p.rot.dims % 8 == 0 && p.rot.dims <= p.K);
  const bool wide = scan_reads_wide(p);
  if (!tokens_only && r.longest > RETENTION_FEW && wide && rot_ok && p.decay_powers) {
    p.vec = aligned(p.out, 16) && p.ld_out % 4 == 0;
    switch (scan_key_pad(p.K) / 32) {
      case 1: return launch_chunks<1>(p, r, s);
      case 2: return launch_chunks<2>(p, r, s);
      case 3: return launch_chunks<3>(p, r, s);
      case 4: return launch_chunks<4>(p, r, s);
      case 5: return launch_chunks<5>(p, r, s);
      case 6: return launch_chunks<6>(p, r, s);
      case 7: return launch_chunks<7>(p, r, s);
      default: return launch_chunks<8>(p, r, s);
    }
  }
  // token by token: decoding rows are rotated by the scan itself
  if (!(r.longest == 1 && wide && rot_ok)) {
    if (p.rot.table) GPTOSS_STEP(run_rotary(p.rot, rows, p.ld_conv, p.q_col, 2 * p.key_heads, p.K, r.lens, r.n, s));
    p.rot = Rotary();
  }
  return run_scan(p, r, s);
}

}  // namespace gptoss
