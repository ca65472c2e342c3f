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
  static constexpr int Q = 0, K = Q + 2 * C * ROW, KT = K + 2 * C * ROW, P = KT + 2 * KP * COL;   // hi parts, then lo parts
  static constexpr int ELEMS = P + 2 * TT * SG * 512;
};

template <int NI, int C>
__global__ __launch_bounds__(256) void retention_chunk_kernel(Scan p, const RowSeg *__restrict__ segs, int n_seg) {
  using L = RetentionTile<NI, C>;
  constexpr int KP = L::KP, TT = L::TT, SG = L::SG, UPT = KP / 8;   // units of 8 dimensions x 4 tokens
  constexpr int OWN = TT * TT / 4;                                  // tiles of the token products per wave
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  const int seg_id = blockIdx.x % n_seg, unit = blockIdx.x / n_seg, blocks = (p.V + 63) / 64;
  const RowSeg seg = segs[seg_id];
  const int h = unit / blocks, kh = h / (p.heads / p.key_heads);
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int n = lane & 15, c = lane >> 4;
  const int c0 = (unit - h * blocks) * 64 + wave * 16, col = min(c0 + n, p.V - 1);   // columns c0 .. + 15 of the wave
  const bool live = c0 + n < p.V;
  const float *power = p.decay_powers + h * (RETENTION_CHUNK + 1);

  f32x4 S[2 * NI];   // d = 16 b + 4 c + e of column c0 + n
  float *st = p.state + (((size_t)seg.slot * p.heads + h) * p.V + col) * KP + 4 * c;
#pragma unroll
  for (int b = 0; b < 2 * NI; b++) {
    S[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (seg.pos0 > 0 && live) S[b] = __builtin_nontemporal_load(reinterpret_cast<const f32x4 *>(st + 16 * b));
  }

  // powers that do not change from chunk to chunk: of this wave's tiles of token products, and of the rows of the output
  const int p_t = wave % TT, p_s = wave / TT;   // token tile of the queries; tiles p_s, p_s + 4 / TT, .. of the keys
  float tri[OWN][4], from[TT];
#pragma unroll
  for (int i = 0; i < OWN; i++)
#pragma unroll
    for (int e = 0; e < 4; e++) {
      const int back = p_t * 16 + n - ((p_s + i * (4 / TT)) * 16 + 4 * c + e);
      tri[i][e] = back >= 0 ? power[max(back, 0)] : 0.f;
    }
#pragma unroll
  for (int t = 0; t < TT; t++) from[t] = power[t * 16 + n + 1];

  // one staging unit per thread: dimensions d0 .. + 3 and d1 .. + 3 (partners where they are rotated) of tokens 4 a .. 4 a + 3
  const int y = tid % UPT, a = tid / UPT, half = p.rot.table ? p.rot.dims >> 1 : 0;
  const bool stages = a < C / 4, turned = 4 * y < half;
  const int d0 = turned ? 4 * y : 2 * half + 8 * (y - half / 4), d1 = turned ? 4 * y + half : d0 + 4;
  const float *k_src = p.conv + p.k_col + kh * p.K, *q_src = p.conv + p.q_col + kh * p.K, *v_src = p.conv + p.v_col + h * p.V + col;
  f32x4 rq[4][2], rk[4][2], cs[4][2];
  float rv[SG * 8];
  auto fetch = [&](int t0) {
    const int T = min(C, seg.n - t0);
    const size_t first = seg.row0 + t0;
    if (stages) {
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int t = min(4 * a + i, T - 1);
        const float *q = q_src + (first + t) * p.ld_conv, *k = k_src + (first + t) * p.ld_conv;
        const int x0 = min(d0, p.K - 4), x1 = min(d1, p.K - 4);
        rq[i][0] = *reinterpret_cast<const f32x4 *>(q + x0);
        rq[i][1] = *reinterpret_cast<const f32x4 *>(q + x1);
        rk[i][0] = *reinterpret_cast<const f32x4 *>(k + x0);
        rk[i][1] = *reinterpret_cast<const f32x4 *>(k + x1);
        if (turned) {
          const f32x4 *at = reinterpret_cast<const f32x4 *>(p.rot.table + ((size_t)(seg.pos0 + t0 + t) * half + 4 * y) * 2);
          cs[i][0] = at[0];
          cs[i][1] = at[1];
        }
      }
    }
#pragma unroll
    for (int x = 0; x < SG * 8; x++) {
      const int t = (x >> 3) * 32 + ((x >> 2) & 1) * 16 + 4 * c + (x & 3);
      rv[x] = v_src[(first + min(t, T - 1)) * p.ld_conv];
    }
  };
  auto put = [&](int T) {
    if (!stages) return;
    f32x4 kw[4][2];
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int t = 4 * a + i;
      f32x4 q[2] = {rq[i][0], rq[i][1]}, k[2] = {rk[i][0], rk[i][1]};
      if (turned) {
#pragma unroll
        for (int e = 0; e < 4; e++) {
          const float cosine = cs[i][e >> 1][2 * (e & 1)], sine = cs[i][e >> 1][2 * (e & 1) + 1];
          q[0][e] = rq[i][0][e] * cosine - rq[i][1][e] * sine;
          q[1][e] = rq[i][1][e] * cosine + rq[i][0][e] * sine;
          k[0][e] = rk[i][0][e] * cosine - rk[i][1][e] * sine;
          k[1][e] = rk[i][1][e] * cosine + rk[i][0][e] * sine;
        }
      }
      const float w = t < T ? power[max(T - 1 - t, 0)] : 0.f;
#pragma unroll
      for (int x = 0; x < 2; x++) {
        const int d = x ? d1 : d0;
        if (d >= p.K) q[x] = k[x] = f32x4{0.f, 0.f, 0.f, 0.f};
        if (t >= T) k[x] = f32x4{0.f, 0.f, 0.f, 0.f};
        kw[i][x] = k[x] * w;
        const int at = t * L::ROW + operand_place(d);
        const Split4 sq = split4(q[x]), sk = split4(k[x]);
        *reinterpret_cast<u32x2 *>(lds + L::Q + at) = sq.hi;
        *reinterpret_cast<u32x2 *>(lds + L::Q + C * L::ROW + at) = sq.lo;
        *reinterpret_cast<u32x2 *>(lds + L::K + at) = sk.hi;
        *reinterpret_cast<u32x2 *>(lds + L::K + C * L::ROW + at) = sk.lo;
      }
    }
#pragma unroll
    for (int x = 0; x < 2; x++)
#pragma unroll
      for (int e = 0; e < 4; e++) {
        const Split4 s = split4(f32x4{kw[0][x][e], kw[1][x][e], kw[2][x][e], kw[3][x][e]});
        const int at = ((x ? d1 : d0) + e) * L::COL + operand_place(4 * a);
        *reinterpret_cast<u32x2 *>(lds + L::KT + at) = s.hi;
        *reinterpret_cast<u32x2 *>(lds + L::KT + KP * L::COL + at) = s.lo;
      }
  };

  fetch(0);
  for (int t0 = 0; t0 < seg.n; t0 += C) {
    const int T = min(C, seg.n - t0), nt = (T + 15) / 16;
    put(T);   // the last reads of Q, K and KT lie before the barrier in front of the previous chunk's last products
    Operand v[SG];
#pragma unroll
    for (int x = 0; x < SG; x++) {
      f32x4 part[2];
#pragma unroll
      for (int e = 0; e < 8; e++) {
        const int t = x * 32 + (e >> 2) * 16 + 4 * c + (e & 3);
        part[e >> 2][e & 3] = t < T && live ? p.value_scale * rv[x * 8 + e] : 0.f;
      }
      v[x] = make_operand(part[0], part[1]);
    }
    __syncthreads();
    if (t0 + C < seg.n) fetch(t0 + C);

    // products of keys and queries, [key][query], masked and decayed, in operand order
    f32x4 prod[OWN];
#pragma unroll
    for (int i = 0; i < OWN; i++) prod[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (p_t < nt) {
#pragma unroll
      for (int ks = 0; ks < NI; ks++) {
        const Operand q = read_operand(lds + L::Q + (p_t * 16 + n) * L::ROW + ks * 32 + c * 8, C * L::ROW);
#pragma unroll
        for (int i = 0; i < OWN; i++) {
          const int s = p_s + i * (4 / TT);
          if (s <= p_t)
            multiply_add(prod[i], read_operand(lds + L::K + (s * 16 + n) * L::ROW + ks * 32 + c * 8, C * L::ROW), q);
        }
      }
#pragma unroll
      for (int i = 0; i < OWN; i++) {
        const int s = p_s + i * (4 / TT);
        if (s / 2 <= p_t / 2) {
          f32x4 w;
#pragma unroll
          for (int e = 0; e < 4; e++) w[e] = prod[i][e] * tri[i][e];
          const Split4 x = split4(w);
          bf16_t *at = lds + L::P + ((p_t * SG + s / 2) * 64 + lane) * 8 + (s & 1) * 4;
          *reinterpret_cast<u32x2 *>(at) = x.hi;
          *reinterpret_cast<u32x2 *>(at + TT * SG * 512) = x.lo;
        }
      }
    }

    // what the state in front of the chunk gives: [column][query]
    f32x4 o[TT];
#pragma unroll
    for (int t = 0; t < TT; t++) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (seg.pos0 + t0 > 0) {
#pragma unroll
      for (int ks = 0; ks < NI; ks++) {
        const Operand s = make_operand(S[2 * ks], S[2 * ks + 1]);
#pragma unroll
        for (int t = 0; t < TT; t++)
          if (t < nt) multiply_add(o[t], s, read_operand(lds + L::Q + (t * 16 + n) * L::ROW + ks * 32 + c * 8, C * L::ROW));
      }
#pragma unroll
      for (int t = 0; t < TT; t++) o[t] *= from[t];
    }

    // the state behind it
    const float fade = power[T];
#pragma unroll
    for (int b = 0; b < 2 * NI; b++) {
      S[b] *= fade;
#pragma unroll
      for (int x = 0; x < SG; x++)
        if (32 * x < T)
          multiply_add(S[b], read_operand(lds + L::KT + (b * 16 + n) * L::COL + x * 32 + c * 8, KP * L::COL), v[x]);
    }
    __syncthreads();

#pragma unroll
    for (int t = 0; t < TT; t++) {
      if (t >= nt) break;
#pragma unroll
      for (int x = 0; x <= t / 2; x++)
        multiply_add(o[t], v[x], read_operand(lds + L::P + ((t * SG + x) * 64 + lane) * 8, TT * SG * 512));
      const int row = t * 16 + n, first = c0 + 4 * c;
      if (row < T) {
        float *dst = p.out + (size_t)(seg.row0 + t0 + row) * p.ld_out + h * p.V + first;
        if (p.vec && first + 4 <= p.V) {
          *reinterpret_cast<f32x4 *>(dst) = o[t];
        } else {
#pragma unroll
          for (int e = 0; e < 4; e++)
            if (first + e < p.V) dst[e] = o[t][e];
        }
      }
    }
  }
  if (live) {
#pragma unroll
    for (int b = 0; b < 2 * NI; b++) __builtin_nontemporal_store(S[b], reinterpret_cast<f32x4 *>(st + 16 * b));
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
  kern<<<(unsigned)((size_t)r.n_seg * p.heads * cdiv(p.V, 64)), 256, bytes, s>>>(p, r.segs, r.n_seg);
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
