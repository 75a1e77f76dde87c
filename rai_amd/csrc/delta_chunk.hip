// The gated delta rule over chunks of 64 tokens on MFMA.  Within a chunk, with G_t the running sum of log decays (per key
// channel), S0 the state before the chunk and ~ marking a row scaled by exp(G_t),
//   u_t = beta_t (v_t - S0^T k~_t - sum_{s<t} A_ts u_s),     A_ts = sum_d k_td k_sd exp(G_td - G_sd)
//   o_t = S0^T q~_t + sum_{s<=t} P_ts u_s,                   P_ts = sum_d q_td k_sd exp(G_td - G_sd)
//   S0 <- exp(G_C) S0 + sum_s (k_s exp(G_C - G_s)) u_s^T.
// With L = beta A (strictly lower), U = U0 - W S0 where (1 + L) [U0 | W] = beta [V | K~].
//   k_delta_chunk  everything that does not depend on the state, all chunks at once: A and P, then U0 and W by forward
//                  substitution in blocks of 16 rows; the operands of the second kernel leave in MFMA-fragment order
//   k_delta_pass   chunk after chunk per head and 16 to 64 columns of the state, which stays in accumulation registers
// exp(G_t - G_s) is never formed over a range that could overflow: block row i refers both factors to R_i, the sum at the
// end of the block before it, so that each is at most 1 outside the block on the diagonal.  On the diagonal the second
// factor is at least 1; if it would exceed e^60 there, that block is summed up pair by pair.
// Products that feed the recurrence take their operands as two bf16 parts each (three MFMAs, 16 bits of mantissa);
// the read-out's operands are rounded to bf16 once, as its result is.
//
// The order of the 32 terms of an MFMA step is free as long as both operands agree.  Here lane l's eight terms are
// 4 (l / 16) .. + 3 of one block of 16 and the same of the next: exactly the rows that lane holds of two accumulator
// tiles, so within k_delta_chunk a product's result is the next product's operand as it stands ("paired order" below).
#include <cmath>

#include "delta.h"
#include "delta_device.h"

namespace rai {

typedef __attribute__((ext_vector_type(8))) __bf16 dc_bf16x8;
typedef __attribute__((ext_vector_type(4))) float dc_f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t dc_u32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t dc_u32x2;

struct Halves { dc_bf16x8 hi, lo; };
__device__ __forceinline__ float bf_lo(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float bf_hi(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }
__device__ __forceinline__ dc_bf16x8 round8(const float (&x)[8]) {
  const dc_u32x4 w = {pack_bf16x2(x[0], x[1]), pack_bf16x2(x[2], x[3]), pack_bf16x2(x[4], x[5]), pack_bf16x2(x[6], x[7])};
  return __builtin_bit_cast(dc_bf16x8, w);
}
__device__ __forceinline__ Halves split8(const float (&x)[8]) {
  Halves r;
  dc_u32x4 h, l;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack_bf16x2(x[2 * i], x[2 * i + 1]);
    l[i] = pack_bf16x2(x[2 * i] - bf_lo(h[i]), x[2 * i + 1] - bf_hi(h[i]));
  }
  r.hi = __builtin_bit_cast(dc_bf16x8, h);
  r.lo = __builtin_bit_cast(dc_bf16x8, l);
  return r;
}
__device__ __forceinline__ dc_f32x4 mma(dc_bf16x8 a, dc_bf16x8 b, dc_f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ dc_f32x4 mma3(const Halves &a, const Halves &b, dc_f32x4 c) {
  c = mma(a.lo, b.hi, c);
  c = mma(a.hi, b.lo, c);
  return mma(a.hi, b.hi, c);
}
__device__ __forceinline__ float fast_exp(float x) { return __builtin_amdgcn_exp2f(x * 1.4426950408889634f); }
constexpr int C = kDeltaChunk;
// One (sequence, chunk, head)'s part of the workspace, in bytes.
struct ChunkLayout {
  int w, q, k, p, u, g, total;
};
__host__ __device__ inline ChunkLayout chunk_layout(int D, int E) {
  ChunkLayout l;
  l.w = 0;                      // [4 row blocks][D / 32][hi, lo][64 lanes][8]      rows t, terms d in paired order
  l.q = l.w + C * D * 4;        // [4][D / 32][64][8]                               rows t, terms d
  l.k = l.q + C * D * 2;        // [D / 16][2 steps of 32 tokens][hi, lo][64][8]    rows d, terms t
  l.p = l.k + C * D * 4;        // [4][2][64][8]                                    rows t, terms s (step 1 of blocks 0, 1 unused)
  l.u = l.p + C * C * 2;        // [4][E / 16][64][4] f32                           accumulator order
  l.g = l.u + C * E * 4;        // [D] f32: exp(G_C)
  l.total = l.g + D * 4;
  return l;
}

// Two runs of four values, 16 apart: a lane's share of a step in paired order.
__device__ __forceinline__ void load_pair(const float *p, float (&x)[8]) {
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const dc_f32x4 v = *reinterpret_cast<const dc_f32x4 *>(p + 16 * i);
#pragma unroll
    for (int e = 0; e < 4; ++e) x[4 * i + e] = v[e];
  }
}
// Two accumulator tiles as one operand; a missing second one counts as zeros.
__device__ __forceinline__ Halves split_pair(const dc_f32x4 &a, const dc_f32x4 &b) {
  const float x[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
  return split8(x);
}

constexpr int kLP = 20;   // pitch of a 16 x 16 block in LDS (floats)
template <int D> constexpr int chunk_lds_floats() { return 2 * C * (D + 4) + 10 * 16 * kLP + 2 * C; }   // D = 128: two blocks to a CU

// WAVES = 8 for few chunks, 4 (two blocks to a CU) for many.  Both kernels have the heads in the grid's fastest dimension:
// blocks go round the eight XCDs, so what a head's chunks leave is read through the same L2 if heads are a multiple of 8.
template <int D, int WAVES>
__global__ void __launch_bounds__(WAVES * 64) k_delta_chunk(DeltaArgs a) {
  constexpr int KS = D / 32, KP = D + 4, kChunkWaves = WAVES, kChunkThreads = WAVES * 64;
  extern __shared__ __attribute__((aligned(16))) float dc_lds[];
  float *Kl = dc_lds, *Gl = Kl + C * KP;      // [64][D] keys and running sums; rows past the end: 0 and the last sum
  float *Ls = Gl + C * KP;                    // blocks (i, j <= i) of beta A, strictly lower, number i (i + 1) / 2 + j; on the
                                              // diagonal later the inverses of the blocks of 1 + L
  float *bs = Ls + 10 * 16 * kLP, *qs = bs + C;   // beta, and what makes a query a unit vector
  const DeltaShape &z = a.s;
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, lq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, n = blockIdx.y, b = blockIdx.z, kv = h / (z.heads / z.kv_heads);
  const int len = a.S - n * C < C ? a.S - n * C : C;
  const int64_t row0 = (int64_t)b * a.S + n * C;
  const int64_t ldk = (int64_t)z.kv_heads * D, ldg = (int64_t)z.heads * D, ldv = (int64_t)z.heads * z.Vp;
  const uint16_t *q = (const uint16_t *)a.q + row0 * ldk + kv * D, *k = (const uint16_t *)a.k + row0 * ldk + kv * D;
  const bf16_raw *v = (const bf16_raw *)a.v + row0 * ldv + h * z.Vp;
  const ChunkLayout lay = chunk_layout(D, z.Vp);
  char *ws = a.chunk_ws + (((int64_t)b * gridDim.y + n) * z.heads + h) * lay.total;
  // queries of row t, a step's terms; scaled to unit length where they are used
  auto query = [&](int t, int ks, dc_u32x2 (&x)[2]) {
#pragma unroll
    for (int e = 0; e < 2; ++e)
      x[e] = t < len ? *reinterpret_cast<const dc_u32x2 *>(q + (int64_t)t * ldk + 32 * ks + 16 * e + 4 * lq) : dc_u32x2{0u, 0u};
  };
  // block (i, j) of the lower triangle number idx
  auto block_row = [](int idx) { return idx < 1 ? 0 : idx < 3 ? 1 : idx < 6 ? 2 : 3; };

  dc_u32x2 qt[KS][2];
#pragma unroll
  for (int ks = 0; ks < KS; ++ks) query(16 * block_row(wave) + l16, ks, qt[ks]);
  // ---- sums of the log decays: a thread takes RUN tokens of one channel, the runs' totals are then added up
  constexpr int RUN = C * D / kChunkThreads, RUNS = C / RUN;
  const int gd = tid % D, g0 = tid / D * RUN;
  float gr[RUN];
  {
    const float rate = -expf(ld<bf16_raw>(a.A_log, h)), bias = ld<bf16_raw>(a.dt_bias, h * D + gd);
    const float *src = a.decay + row0 * ldg + h * D + gd;
#pragma unroll
    for (int t = 0; t < RUN; ++t) gr[t] = src[(int64_t)(g0 + t < len ? g0 + t : len - 1) * ldg];
    for (int e = tid; e < C * D / 8; e += kChunkThreads) {   // keys, meanwhile
      const int t = e / (D / 8), d = (e - t * (D / 8)) * 8;
      dc_u32x4 x = *reinterpret_cast<const dc_u32x4 *>(k + (int64_t)(t < len ? t : len - 1) * ldk + d);
      const float r = t < len ? a.kn[(row0 + t) * z.kv_heads + kv] : 0.f;
      *reinterpret_cast<dc_f32x4 *>(Kl + t * KP + d) = dc_f32x4{bf_lo(x[0]) * r, bf_hi(x[0]) * r, bf_lo(x[1]) * r, bf_hi(x[1]) * r};
      *reinterpret_cast<dc_f32x4 *>(Kl + t * KP + d + 4) = dc_f32x4{bf_lo(x[2]) * r, bf_hi(x[2]) * r, bf_lo(x[3]) * r, bf_hi(x[3]) * r};
    }
    float run = 0.f;
#pragma unroll
    for (int t = 0; t < RUN; ++t) {
      if (g0 + t < len && gd < z.dim) run += rate * softplus_for<bf16_raw>(gr[t] + bias);   // padding channels do not decay: their factors stay finite
      gr[t] = run;
    }
    Ls[(g0 / RUN) * D + gd] = run;   // not yet used for its blocks
  }
  if (tid < C) {
    bs[tid] = tid < len ? dl_sigmoid(ld<bf16_raw>(a.dn, (row0 + tid) * z.ldn + z.off_b + h)) : 0.f;
    qs[tid] = tid < len ? a.qn[(row0 + tid) * z.kv_heads + kv] : 0.f;
  }
  __syncthreads();
  {
    float before = 0.f;
#pragma unroll
    for (int r = 0; r < RUNS - 1; ++r)
      if (r < g0 / RUN) before += Ls[r * D + gd];
#pragma unroll
    for (int t = 0; t < RUN; ++t) Gl[(g0 + t) * KP + gd] = gr[t] + before;
    if (g0 + RUN == C) reinterpret_cast<float *>(ws + lay.g)[gd] = fast_exp(gr[RUN - 1] + before);
  }
  __syncthreads();

  // ---- blocks of A and P
  for (int idx = wave; idx < 10; idx += kChunkWaves) {
    const int i = block_row(idx), j = idx - i * (i + 1) / 2, t0 = 16 * i, t = t0 + l16, s = 16 * j + l16;
    dc_f32x4 A = {0.f, 0.f, 0.f, 0.f}, P = A;   // A: rows t, columns s;  P: rows s, columns t
    float range = 0.f;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const int d = 32 * ks + 4 * lq;
      float R[8], kt[8], gt[8], kb[8], gs[8], qx[8];
#pragma unroll
      for (int y = 0; y < 8; ++y) qx[y] = qs[t] * (y & 1 ? bf_hi(qt[ks][y >> 2][(y & 3) >> 1]) : bf_lo(qt[ks][y >> 2][(y & 3) >> 1]));
      load_pair(Kl + t * KP + d, kt);
      load_pair(Gl + t * KP + d, gt);
      load_pair(Kl + s * KP + d, kb);
      load_pair(Gl + s * KP + d, gs);
      if (i > 0) load_pair(Gl + (t0 - 1) * KP + d, R);
      else {
#pragma unroll
        for (int y = 0; y < 8; ++y) R[y] = 0.f;
      }
      if (i == j) {
        float ge[8];
        load_pair(Gl + (t0 + 15) * KP + d, ge);
#pragma unroll
        for (int y = 0; y < 8; ++y) range = fmaxf(range, R[y] - ge[y]);
      }
      if (i == j) {   // the scaled queries of this row block, on the way
        float x[8];
#pragma unroll
        for (int y = 0; y < 8; ++y) x[y] = qx[y] * fast_exp(gt[y]);
        *reinterpret_cast<dc_bf16x8 *>(ws + lay.q + ((i * KS + ks) * 64 + lane) * 16) = round8(x);
      }
#pragma unroll
      for (int y = 0; y < 8; ++y) {
        const float e = fast_exp(gt[y] - R[y]);
        kt[y] *= e;
        qx[y] *= e;
        kb[y] *= fast_exp(R[y] - gs[y]);
      }
      if (idx + kChunkWaves < 10) query(16 * block_row(idx + kChunkWaves) + l16, ks, qt[ks]);   // for the next block
      const Halves kB = split8(kb);
      A = mma3(split8(kt), kB, A);
      P = mma(kB.hi, round8(qx), P);
    }
    if (i == j && wave_max(range) > 60.f) {   // pair by pair
#pragma unroll 1
      for (int r = 0; r < 4; ++r) {
        const int m = 4 * lq + r;             // A of (t0 + m, t0 + l16) and P of (t0 + l16, t0 + m)
        float sa = 0.f, sp = 0.f;
        for (int d = 0; d < D; ++d) {
          const float gm = Gl[(t0 + m) * KP + d], gl = Gl[t * KP + d], km = Kl[(t0 + m) * KP + d], kl = Kl[t * KP + d];
          if (l16 <= m) sa = fmaf(km * kl, fast_exp(gm - gl), sa);
          if (m <= l16 && t < len) sp = fmaf(bf16_bits_to_f32(q[(int64_t)t * ldk + d]) * qs[t] * km, fast_exp(gl - gm), sp);
        }
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (e == r) { A[e] = sa; P[e] = sp; }
      }
    }
    dc_u32x2 pw;
    float px[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = 4 * lq + r;
      Ls[(idx * 16 + m) * kLP + l16] = s < t0 + m ? bs[t0 + m] * A[r] : 0.f;
      px[r] = 16 * j + m <= t ? P[r] : 0.f;
    }
    pw.x = pack_bf16x2(px[0], px[1]);
    pw.y = pack_bf16x2(px[2], px[3]);
    *reinterpret_cast<dc_u32x2 *>(ws + lay.p + ((i * 2 + j / 2) * 64 + lane) * 16 + (j & 1) * 8) = pw;
  }
  if (wave >= kChunkWaves - 2) {   // the blocks above the diagonal that share a step with one on or below it
    const int i = wave == kChunkWaves - 1 ? 2 : 0;
    *reinterpret_cast<dc_u32x2 *>(ws + lay.p + ((i * 2 + i / 2) * 64 + lane) * 16 + 8) = dc_u32x2{0u, 0u};
  }
  __syncthreads();
  // values of the first pair of column tiles, ahead of their use
  const int vp = z.Vp / 32;
  uint16_t vr[2][4][4];
  auto values = [&](int pair) {
#pragma unroll
    for (int e = 0; e < 2; ++e)
#pragma unroll
      for (int ib = 0; ib < 4; ++ib)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * ib + 4 * lq + r;
          vr[e][ib][r] = v[(int64_t)(t < len ? t : len - 1) * ldv + pair * 32 + 16 * e + l16].bits;
        }
  };
  if (wave < vp) values(wave);
  // ---- operand of the state's update: k_s exp(G_C - G_s), rows d
  auto update_operand = [&](int f) {
    const int dt = f >> 1, ks = f & 1, d = 16 * dt + l16;
    const float gc = Gl[(C - 1) * KP + d];
    float x[8];
#pragma unroll
    for (int y = 0; y < 8; ++y) {
      const int s = 32 * ks + 16 * (y >> 2) + 4 * lq + (y & 3);
      x[y] = Kl[s * KP + d] * fast_exp(gc - Gl[s * KP + d]);
    }
    const Halves o = split8(x);
    char *dst = ws + lay.k + (f * 2 * 64 + lane) * 16;
    *reinterpret_cast<dc_bf16x8 *>(dst) = o.hi;
    *reinterpret_cast<dc_bf16x8 *>(dst + 64 * 16) = o.lo;
  };
  if (wave < 4) {
    // ---- inverses of the diagonal blocks, lane = column (four copies); a block is read whole before it is overwritten
    float *blk = Ls + (wave * (wave + 1) / 2 + wave) * 16 * kLP;
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float s0 = t == l16 ? 1.f : 0.f, s1 = 0.f;
#pragma unroll
      for (int m = 0; m < t; ++m) (m & 1 ? s1 : s0) = fmaf(-blk[t * kLP + m], x[m], m & 1 ? s1 : s0);
      x[t] = s0 + s1;
    }
    __builtin_amdgcn_wave_barrier();
    if (lq == 0) {
#pragma unroll
      for (int t = 0; t < 16; ++t) blk[t * kLP + l16] = x[t];
    }
    if constexpr (WAVES == 4)
      for (int f = wave; f < D / 8; f += 4) update_operand(f);
  } else {
    for (int f = wave - 4; f < D / 8; f += 4) update_operand(f);
  }
  __syncthreads();
  // ---- (1 + L) X = beta [V | K~], two tiles of 16 columns at a time
  Halves Lf[4], Nf[4], one;   // L of block rows 1, 2, 3 (first two blocks) and 3 (third), the inverses, the unit matrix
#pragma unroll
  for (int ib = 0; ib < 4; ++ib) {
    float x[8];
#pragma unroll
    for (int y = 0; y < 8; ++y) x[y] = 0.f;
    const dc_f32x4 nv = *reinterpret_cast<const dc_f32x4 *>(Ls + ((ib * (ib + 1) / 2 + ib) * 16 + l16) * kLP + 4 * lq);
#pragma unroll
    for (int y = 0; y < 4; ++y) x[y] = nv[y];
    Nf[ib] = split8(x);
    const int row = ib < 3 ? ib + 1 : 3, col = ib < 3 ? 0 : 2, blk = row * (row + 1) / 2 + col;
#pragma unroll
    for (int y = 0; y < 2; ++y) {   // the second block of the step may lie on the diagonal
      const bool below = col + y < row;
      const dc_f32x4 lv = *reinterpret_cast<const dc_f32x4 *>(Ls + ((below ? blk + y : blk) * 16 + l16) * kLP + 4 * lq);
#pragma unroll
      for (int e = 0; e < 4; ++e) x[4 * y + e] = below ? lv[e] : 0.f;
    }
    Lf[ib] = split8(x);
  }
  {
    float x[8];
#pragma unroll
    for (int y = 0; y < 8; ++y) x[y] = y < 4 && 4 * lq + y == l16 ? 1.f : 0.f;
    one.hi = round8(x);
  }
  const dc_f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  for (int pair = wave; pair < vp + KS; pair += kChunkWaves) {
    const bool val = pair < vp;
    if (val && pair >= kChunkWaves) values(pair);
    const int c0 = (val ? pair : pair - vp) * 32 + l16;
    dc_f32x4 X[2][4];
#pragma unroll
    for (int e = 0; e < 2; ++e)
#pragma unroll
      for (int ib = 0; ib < 4; ++ib)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * ib + 4 * lq + r, c = c0 + 16 * e;
          X[e][ib][r] = bs[t] * (val ? bf16_bits_to_f32(vr[e][ib][r]) : Kl[t * KP + c] * fast_exp(Gl[t * KP + c]));
        }
    Halves first[2];   // solved blocks 0 and 1
#pragma unroll
    for (int ib = 0; ib < 4; ++ib) {
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        dc_f32x4 y = X[e][ib];
        if (ib > 0) {
          dc_f32x4 acc = mma3(Lf[ib - 1], first[e], zero);
          if (ib == 3) acc = mma3(Lf[3], split_pair(X[e][2], zero), acc);
#pragma unroll
          for (int r = 0; r < 4; ++r) y[r] -= acc[r];
        }
        X[e][ib] = mma3(Nf[ib], split_pair(y, zero), zero);
        if (ib == 0) first[e] = split_pair(X[e][0], zero);
        if (ib == 1) first[e] = split_pair(X[e][0], X[e][1]);
      }
    }
#pragma unroll
    for (int ib = 0; ib < 4; ++ib) {
      if (val) {
#pragma unroll
        for (int e = 0; e < 2; ++e) *reinterpret_cast<dc_f32x4 *>(ws + lay.u + ((ib * 2 * vp + pair * 2 + e) * 64 + lane) * 16) = X[e][ib];
      } else {   // rows t, columns d become rows d, columns t: each lane then holds the terms d of its own row t
        dc_f32x4 Xt[2];
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const Halves x = split_pair(X[e][ib], zero);
          Xt[e] = mma(x.hi, one.hi, mma(x.lo, one.hi, zero));
        }
        const Halves o = split_pair(Xt[0], Xt[1]);
        char *dst = ws + lay.w + ((ib * KS + pair - vp) * 2 * 64 + lane) * 16;
        *reinterpret_cast<dc_bf16x8 *>(dst) = o.hi;
        *reinterpret_cast<dc_bf16x8 *>(dst + 64 * 16) = o.lo;
      }
    }
  }
}

// Block = (16 EB columns e of the state, head, sequence).  Wave w owns rows 16 w .. + 15 of a chunk in the products over
// the state, and channels w D / 4 .. of the state itself: rows d, columns e.  State and U pass through LDS as
// operands, their terms stored in paired order.  The operands of either half of a chunk are requested SETS chunks ahead, as
// soon as the registers they go to have been used; every load and store of the loop is unconditional (rows past the end go to a row
// behind the last), so that the compiler can count them and wait for no more than it needs.
__device__ __forceinline__ int paired(int term) { return (term & ~31) | ((term & 12) << 1) | ((term & 16) >> 2) | (term & 3); }
template <int D, int EB, int SETS>
__global__ void __launch_bounds__(256, 1) k_delta_pass(DeltaArgs a) {
  constexpr int KS = D / 32, DT = D / 64, SP = D + 8, UP = C + 8;
  __shared__ __attribute__((aligned(16))) uint16_t St[2][16 * EB * SP];   // hi / lo of the state, [e][d]
  __shared__ __attribute__((aligned(16))) uint16_t Ut[2][16 * EB * UP];   // of U, [e][t]
  const DeltaShape &z = a.s;
  const int tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, lq = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, e0 = blockIdx.y * 16 * EB, b = blockIdx.z;
  const int chunks = (a.S + C - 1) / C, vt = z.Vp / 16;
  const ChunkLayout lay = chunk_layout(D, z.Vp);
  const int pos0 = a.state->pos;
  const char *ws0 = a.chunk_ws + ((int64_t)b * chunks * z.heads + h) * lay.total;
  const int64_t step = (int64_t)z.heads * lay.total;
  float *const carried = a.carried + ((int64_t)b * z.heads + h) * D * z.Vp + e0;
  dc_f32x4 S[DT][EB];
  auto state_at = [&](int dt, int e, int r) { return carried + (int64_t)((wave * DT + dt) * 16 + 4 * lq + r) * z.Vp + 16 * e + l16; };
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int e = 0; e < EB; ++e)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[dt][e][r] = pos0 > 0 ? *state_at(dt, e, r) : 0.f;
  struct Operands {
    dc_bf16x8 wh[KS], wl[KS], q[KS], p[2], kh[DT][2], kl[DT][2];
    dc_f32x4 u[EB], w[DT];
  };
  auto request_first = [&](int n, Operands &x) {
    const char *ws = ws0 + (n < chunks ? n : chunks - 1) * step;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const char *src = ws + lay.w + ((wave * KS + ks) * 2 * 64 + lane) * 16;
      x.wh[ks] = *reinterpret_cast<const dc_bf16x8 *>(src);
      x.wl[ks] = *reinterpret_cast<const dc_bf16x8 *>(src + 64 * 16);
      x.q[ks] = *reinterpret_cast<const dc_bf16x8 *>(ws + lay.q + ((wave * KS + ks) * 64 + lane) * 16);
    }
#pragma unroll
    for (int e = 0; e < EB; ++e) x.u[e] = *reinterpret_cast<const dc_f32x4 *>(ws + lay.u + ((wave * vt + e0 / 16 + e) * 64 + lane) * 16);
  };
  auto request_second = [&](int n, Operands &x) {
    const char *ws = ws0 + (n < chunks ? n : chunks - 1) * step;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      x.w[dt] = *reinterpret_cast<const dc_f32x4 *>(ws + lay.g + ((wave * DT + dt) * 16 + 4 * lq) * 4);
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const char *src = ws + lay.k + (((wave * DT + dt) * 2 + ks) * 2 * 64 + lane) * 16;
        x.kh[dt][ks] = *reinterpret_cast<const dc_bf16x8 *>(src);
        x.kl[dt][ks] = *reinterpret_cast<const dc_bf16x8 *>(src + 64 * 16);
      }
    }
    x.p[0] = *reinterpret_cast<const dc_bf16x8 *>(ws + lay.p + (wave * 2 * 64 + lane) * 16);
    x.p[1] = *reinterpret_cast<const dc_bf16x8 *>(ws + lay.p + ((wave * 2 + 1) * 64 + lane) * 16);
  };
  // four consecutive terms of one column, hi and lo
  auto put = [&](auto &dst, int at, const dc_f32x4 &y) {
    const dc_u32x2 hi = {pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
    const dc_u32x2 lo = {pack_bf16x2(y[0] - bf_lo(hi.x), y[1] - bf_hi(hi.x)), pack_bf16x2(y[2] - bf_lo(hi.y), y[3] - bf_hi(hi.y))};
    *reinterpret_cast<dc_u32x2 *>(dst[0] + at) = hi;
    *reinterpret_cast<dc_u32x2 *>(dst[1] + at) = lo;
  };
  const int64_t ldo = (int64_t)z.heads * z.Vp;
  float *const o0 = a.o + h * z.Vp + e0 + l16, *const behind = o0 + (int64_t)a.B * a.S * ldo;
  float *out[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) out[r] = o0 + ((int64_t)b * a.S + 16 * wave + 4 * lq + r) * ldo;
  auto chunk = [&](int n, Operands &c) __attribute__((always_inline)) {
    // ---- the state as an operand
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int e = 0; e < EB; ++e) put(St, (16 * e + l16) * SP + paired((wave * DT + dt) * 16 + 4 * lq), S[dt][e]);
    __syncthreads();
    dc_f32x4 O[EB];
#pragma unroll
    for (int e = 0; e < EB; ++e) {
      dc_f32x4 x = {0.f, 0.f, 0.f, 0.f}, x2 = x, x3 = x;
      O[e] = x;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const int at = (16 * e + l16) * SP + 32 * ks + 8 * lq;
        const dc_bf16x8 sh = *reinterpret_cast<const dc_bf16x8 *>(St[0] + at), sl = *reinterpret_cast<const dc_bf16x8 *>(St[1] + at);
        x = mma(c.wh[ks], sh, x);
        x2 = mma(c.wh[ks], sl, x2);
        x3 = mma(c.wl[ks], sh, x3);
        O[e] = mma(c.q[ks], sh, O[e]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) x[r] = c.u[e][r] - (x[r] + (x2[r] + x3[r]));
      put(Ut, (16 * e + l16) * UP + paired(16 * wave + 4 * lq), x);
    }
    request_first(n + SETS, c);
    __syncthreads();
    // ---- update and read-out
#pragma unroll
    for (int e = 0; e < EB; ++e) {
      Halves ua[2];
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const int at = (16 * e + l16) * UP + 32 * ks + 8 * lq;
        ua[ks].hi = *reinterpret_cast<const dc_bf16x8 *>(Ut[0] + at);
        ua[ks].lo = *reinterpret_cast<const dc_bf16x8 *>(Ut[1] + at);
      }
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[dt][e][r] *= c.w[dt][r];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          Halves kb;
          kb.hi = c.kh[dt][ks];
          kb.lo = c.kl[dt][ks];
          S[dt][e] = mma3(kb, ua[ks], S[dt][e]);
        }
      }
      O[e] = mma(c.p[0], ua[0].hi, O[e]);
      if (wave >= 2) O[e] = mma(c.p[1], ua[1].hi, O[e]);
    }
    request_second(n + SETS, c);
    const int left = a.S - n * C - 16 * wave - 4 * lq;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      float *const p = r < left ? out[r] : behind;
#pragma unroll
      for (int e = 0; e < EB; ++e) p[16 * e] = O[e][r];
      out[r] += C * ldo;
    }
  };
  Operands ops[SETS];
#pragma unroll
  for (int i = 0; i < SETS; ++i) {
    request_first(i, ops[i]);
    request_second(i, ops[i]);
  }
  int n = 0;
  for (; n + SETS <= chunks; n += SETS) {
#pragma unroll
    for (int i = 0; i < SETS; ++i) chunk(n + i, ops[i]);
  }
  if (SETS > 1 && n < chunks) chunk(n, ops[0]);
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int e = 0; e < EB; ++e)
#pragma unroll
      for (int r = 0; r < 4; ++r) *state_at(dt, e, r) = S[dt][e][r];
  if (blockIdx.y == 0) update_ring<bf16_raw>(a, b, h, pos0, tid, 256);
}

bool delta_chunk_serves(int dtype, const DeltaShape &z) {
  return dtype == RAI_BF16 && (z.Dk == 64 || z.Dk == 128 || z.Dk == 256) && z.Vp % 32 == 0;
}
size_t delta_chunk_ws_bytes(const DeltaShape &z, int64_t max_batch, int64_t max_rows) {
  return (size_t)(max_rows / C + max_batch) * z.heads * chunk_layout(z.Dk, z.Vp).total;
}

template <int D, int WAVES> static int launch_chunk_w(hipStream_t st, const DeltaArgs &a) {
  constexpr size_t lds = chunk_lds_floats<D>() * sizeof(float);
  static_assert(lds <= 160 * 1024 && (D > 128 || lds <= 80 * 1024), "a chunk's keys and sums fit LDS");
  static bool attr_set = false;
  if (lds > 64 * 1024 && !attr_set) {
    RAI_HIP_TRY(hipFuncSetAttribute((const void *)k_delta_chunk<D, WAVES>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    attr_set = true;
  }
  hipLaunchKernelGGL((k_delta_chunk<D, WAVES>), dim3(a.s.heads, (a.S + C - 1) / C, a.B), dim3(WAVES * 64), lds, st, a);
  return launch_check("delta_chunk");
}
template <int D> static int launch_chunks(hipStream_t st, const DeltaArgs &a) {
  const DeltaShape &z = a.s;
  const int64_t heads = (int64_t)z.heads * a.B;
  if (D > 128 || heads * ((a.S + C - 1) / C) <= kNumCU) RAI_TRY((launch_chunk_w<D, 8>(st, a)));
  else RAI_TRY((launch_chunk_w<D, (D > 128 ? 8 : 4)>(st, a)));
  // 64 columns a block read the operands half as often as 32; 16 make the shortest chain while there are CUs to spare
  if (D <= 128 && heads * (z.Vp / 16) <= kNumCU)
    hipLaunchKernelGGL((k_delta_pass<D, 1, (D > 128 ? 1 : 2)>), dim3(z.heads, z.Vp / 16, a.B), dim3(256), 0, st, a);
  else if (D <= 128 && z.Vp % 64 == 0 && heads * (z.Vp / 32) > 2 * kNumCU)
    hipLaunchKernelGGL((k_delta_pass<D, (D > 128 ? 2 : 4), (D > 128 ? 1 : 2)>), dim3(z.heads, z.Vp / 64, a.B), dim3(256), 0, st, a);
  else
    hipLaunchKernelGGL((k_delta_pass<D, 2, (D > 128 ? 1 : 2)>), dim3(z.heads, z.Vp / 32, a.B), dim3(256), 0, st, a);
  return launch_check("delta_pass");
}
int launch_delta_chunks(hipStream_t st, const DeltaArgs &a) {
  RAI_REQUIRE(a.chunk_ws && delta_chunk_serves(RAI_BF16, a.s), RAI_ERR_BAD_ARG, "delta chunks: not served");
  if (a.s.Dk == 64) return launch_chunks<64>(st, a);
  if (a.s.Dk == 128) return launch_chunks<128>(st, a);
  return launch_chunks<256>(st, a);
}

}  // namespace rai
