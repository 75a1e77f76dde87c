// The gated delta rule over chunks of 64 tokens on MFMA.  Within a chunk, with G_t the running sum of log decays (per key
// channel), S0 the state before the chunk and ~ marking a row scaled by exp(G_t),
//   u_t = beta_t (v_t - S0^T k~_t - sum_{s<t} A_ts u_s),     A_ts = sum_d k_td k_sd exp(G_td - G_sd)
//   o_t = S0^T q~_t + sum_{s<=t} P_ts u_s,                   P_ts = sum_d q_td k_sd exp(G_td - G_sd)
//   S0 <- exp(G_C) S0 + sum_s (k_s exp(G_C - G_s)) u_s^T.
// With L = beta A (strictly lower), U = U0 - W S0 where (1 + L) [U0 | W] = beta [V | K~].
//   k_delta_chunk  everything that does not depend on the state, all chunks at once: A and P, then U0 and W by forward
//                  substitution in blocks of 16 rows; the operands of the second kernel leave in MFMA-fragment order
//   k_delta_pass   chunk after chunk per head and 32 columns of the state, which stays in accumulation registers
// exp(G_t - G_s) is never formed over a range that could overflow: block row i refers both factors to R_i, the sum at the
// end of the block before it, so that each is at most 1 outside the block on the diagonal.  On the diagonal the second
// factor is at least 1; if it would exceed e^60 there, that block is summed up pair by pair.
// Products that feed the recurrence take their operands as two bf16 parts each (three MFMAs, 16 bits of mantissa);
// the read-out's operands are rounded to bf16 once, as its result is.
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
__device__ __forceinline__ dc_bf16x8 zero8() { return __builtin_bit_cast(dc_bf16x8, dc_u32x4{0u, 0u, 0u, 0u}); }
// Lanes of one wave hand values to each other through LDS.
__device__ __forceinline__ void wave_lds_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

constexpr int C = kDeltaChunk;
// One (sequence, chunk, head)'s part of the workspace, in bytes.
struct ChunkLayout {
  int w, q, k, p, u, total;
};
__host__ __device__ inline ChunkLayout chunk_layout(int D, int E) {
  ChunkLayout l;
  l.w = 0;                      // [4 row blocks][D / 32][hi, lo][64 lanes][8]      A operand, rows t
  l.q = l.w + C * D * 4;        // [4][D / 32][64][8]                               A operand, rows t
  l.k = l.q + C * D * 2;        // [D / 16][2 steps of 32 tokens][hi, lo][64][8]    B operand, columns d
  l.p = l.k + C * D * 4;        // [4][2][64][8]                                    A operand, rows t
  l.u = l.p + C * C * 2;        // [4][E / 16][64][4] f32                           accumulator order
  l.total = l.u + C * E * 4;
  return l;
}

__device__ __forceinline__ void load8(const float *p, bool ok, float (&x)[8]) {
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const dc_f32x4 v = ok ? *reinterpret_cast<const dc_f32x4 *>(p + 4 * i) : dc_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int e = 0; e < 4; ++e) x[4 * i + e] = v[e];
  }
}

constexpr int kAP = C + 4, kNP = 20, kXP = C + 8;   // LDS pitches
template <int D>
__global__ void __launch_bounds__(256) k_delta_chunk(DeltaArgs a) {
  constexpr int KS = D / 32;
  __shared__ __attribute__((aligned(16))) float Ls[C * kAP];              // beta A, strictly lower
  __shared__ __attribute__((aligned(16))) float Ns[4 * 16 * kNP];         // inverses of the diagonal blocks of 1 + L
  __shared__ __attribute__((aligned(16))) uint16_t Xs[4][2][16 * kXP];    // per wave: solved rows of a 16-column tile, transposed, hi / lo
  const DeltaShape &z = a.s;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
  const int n = blockIdx.x, h = blockIdx.y, b = blockIdx.z, kv = h / (z.heads / z.kv_heads);
  const int len = a.S - n * C < C ? a.S - n * C : C;
  const int64_t row0 = (int64_t)b * a.S + n * C;
  const int64_t ldk = (int64_t)z.kv_heads * D, ldg = (int64_t)z.heads * D, ldv = (int64_t)z.heads * z.Vp;
  const float *q = a.q + row0 * ldk + kv * D, *k = a.k + row0 * ldk + kv * D, *G = a.decay + row0 * ldg + h * D;
  const float *beta = a.beta + row0 * z.heads + h;
  const bf16_raw *v = (const bf16_raw *)a.v + row0 * ldv + h * z.Vp;
  const ChunkLayout lay = chunk_layout(D, z.Vp);
  char *ws = a.chunk_ws + (((int64_t)b * gridDim.x + n) * z.heads + h) * lay.total;
  for (int i = lane; i < 16 * kXP; i += 64) Xs[wave][0][i] = Xs[wave][1][i] = 0;   // multiplied by zeros before they are solved

  // ---- A and P, block row `wave`
  const int i = wave, t0 = 16 * i;
  const int prev = t0 - 1 < len - 1 ? t0 - 1 : len - 1;                  // the token that R_i is the sum at
  const int tl = t0 + l16, last = t0 + 15 < len - 1 ? t0 + 15 : len - 1;
  dc_f32x4 A[4], P[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) A[j] = P[j] = dc_f32x4{0.f, 0.f, 0.f, 0.f};
  float range = 0.f;
  for (int ks = 0; ks < KS; ++ks) {
    const int d = 32 * ks + 8 * lq;
    const bool in = tl < len;
    float R[8], kt[8], qt[8], gt[8], e[8], x[8];
    load8(G + (int64_t)prev * ldg + d, i > 0, R);
    load8(k + (int64_t)tl * ldk + d, in, kt);
    load8(q + (int64_t)tl * ldk + d, in, qt);
    load8(G + (int64_t)tl * ldg + d, in, gt);
    if (t0 < len) {
      float ge[8];
      load8(G + (int64_t)last * ldg + d, true, ge);
#pragma unroll
      for (int y = 0; y < 8; ++y) range = fmaxf(range, R[y] - ge[y]);
    }
#pragma unroll
    for (int y = 0; y < 8; ++y) x[y] = in ? qt[y] * fast_exp(gt[y]) : 0.f;
    *reinterpret_cast<dc_bf16x8 *>(ws + lay.q + ((i * KS + ks) * 64 + lane) * 16) = round8(x);
#pragma unroll
    for (int y = 0; y < 8; ++y) {
      e[y] = in ? fast_exp(gt[y] - R[y]) : 0.f;
      kt[y] *= e[y];
      qt[y] *= e[y];
    }
    const Halves ka = split8(kt);
    const dc_bf16x8 qa = round8(qt);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j > i) continue;
      const int s = 16 * j + l16;
      float kb[8], gs[8];
      load8(k + (int64_t)s * ldk + d, s < len, kb);
      load8(G + (int64_t)s * ldg + d, s < len, gs);
#pragma unroll
      for (int y = 0; y < 8; ++y) kb[y] = s < len ? kb[y] * fast_exp(R[y] - gs[y]) : 0.f;
      const Halves kB = split8(kb);
      A[j] = mma3(ka, kB, A[j]);
      P[j] = mma(qa, kB.hi, P[j]);
    }
  }
  if (wave_max(range) > 60.f) {   // the diagonal block pair by pair
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = t0 + 4 * lq + r, s = t0 + l16;
      float sa = 0.f, sp = 0.f;
      if (s <= t && t < len)
        for (int d = 0; d < D; ++d) {
          const float w = k[(int64_t)s * ldk + d] * fast_exp(G[(int64_t)t * ldg + d] - G[(int64_t)s * ldg + d]);
          sa = fmaf(k[(int64_t)t * ldk + d], w, sa);
          sp = fmaf(q[(int64_t)t * ldk + d], w, sp);
        }
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (j == i) { A[j][r] = sa; P[j][r] = sp; }
    }
  }
  float bt[4];   // beta of the rows this lane holds of a block's accumulator, per block
#pragma unroll
  for (int r = 0; r < 4; ++r) bt[r] = t0 + 4 * lq + r < len ? beta[(int64_t)(t0 + 4 * lq + r) * z.heads] : 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = t0 + 4 * lq + r, s = 16 * j + l16;
      if (j <= i) Ls[t * kAP + s] = s < t ? bt[r] * A[j][r] : 0.f;
      const float p = j <= i && s <= t ? P[j][r] : 0.f;
      reinterpret_cast<uint16_t *>(ws + lay.p)[((i * 2 + j / 2) * 64 + (t & 15) + 16 * ((s & 31) >> 3)) * 8 + (s & 7)] = f32_to_bf16_bits(p);
    }
  __syncthreads();
  // ---- the diagonal block's inverse, lane = column (four copies)
  {
    float x[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float s = t == l16 ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < t; ++m) s = fmaf(-Ls[(t0 + t) * kAP + t0 + m], x[m], s);
      x[t] = s;
      if (lq == 0) Ns[(i * 16 + t) * kNP + l16] = s;
    }
  }
  // ---- operand of the state's update: k_s exp(G_C - G_s), channels as columns
  for (int dt = wave; dt < D / 16; dt += 4) {
    const int d = 16 * dt + l16;
    const float gc = G[(int64_t)(len - 1) * ldg + d];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      float x[8];
#pragma unroll
      for (int y = 0; y < 8; ++y) {
        const int s = 32 * ks + 8 * lq + y;
        x[y] = s < len ? k[(int64_t)s * ldk + d] * fast_exp(gc - G[(int64_t)s * ldg + d]) : 0.f;
      }
      const Halves o = split8(x);
      char *dst = ws + lay.k + ((dt * 2 + ks) * 2 * 64 + lane) * 16;
      *reinterpret_cast<dc_bf16x8 *>(dst) = o.hi;
      *reinterpret_cast<dc_bf16x8 *>(dst + 64 * 16) = o.lo;
    }
  }
  __syncthreads();
  // ---- (1 + L) X = beta [V | K~], a tile of 16 columns at a time
  const int vt = z.Vp / 16;
  uint16_t *xh = Xs[wave][0], *xl = Xs[wave][1];
  auto put = [&](int at, const dc_f32x4 &y) {   // rows at + 4 lq .. + 3 of column l16
    const dc_u32x2 hi = {pack_bf16x2(y[0], y[1]), pack_bf16x2(y[2], y[3])};
    const dc_u32x2 lo = {pack_bf16x2(y[0] - bf_lo(hi.x), y[1] - bf_hi(hi.x)), pack_bf16x2(y[2] - bf_lo(hi.y), y[3] - bf_hi(hi.y))};
    *reinterpret_cast<dc_u32x2 *>(xh + l16 * kXP + at + 4 * lq) = hi;
    *reinterpret_cast<dc_u32x2 *>(xl + l16 * kXP + at + 4 * lq) = lo;
  };
  auto get = [&](int at) {                      // rows at .. + 7 of column l16
    Halves r;
    r.hi = *reinterpret_cast<const dc_bf16x8 *>(xh + l16 * kXP + at);
    r.lo = *reinterpret_cast<const dc_bf16x8 *>(xl + l16 * kXP + at);
    return r;
  };
  for (int tile = wave; tile < vt + D / 16; tile += 4) {
    const bool val = tile < vt;
    const int c = (val ? tile : tile - vt) * 16 + l16;
    float rhs[4][4];
#pragma unroll
    for (int ib = 0; ib < 4; ++ib)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * ib + 4 * lq + r;
        rhs[ib][r] = 0.f;
        if (t < len) {
          const float be = beta[(int64_t)t * z.heads];
          rhs[ib][r] = be * (val ? bf16_bits_to_f32(v[(int64_t)t * ldv + c].bits) : k[(int64_t)t * ldk + c] * fast_exp(G[(int64_t)t * ldg + c]));
        }
      }
#pragma unroll
    for (int ib = 0; ib < 4; ++ib) {
      dc_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < (16 * ib + 31) / 32; ++ks) {
        const int s = 32 * ks + 8 * lq;
        float x[8];
#pragma unroll
        for (int y = 0; y < 8; ++y) x[y] = 0.f;
        if (s < 16 * ib) load8(Ls + (16 * ib + l16) * kAP + s, true, x);
        acc = mma3(split8(x), get(s), acc);
      }
      dc_f32x4 y;
#pragma unroll
      for (int r = 0; r < 4; ++r) y[r] = rhs[ib][r] - acc[r];
      wave_lds_sync();
      put(16 * ib, y);
      wave_lds_sync();
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = 0.f;
      Halves yb;
      yb.hi = yb.lo = zero8();
      if (lq < 2) {
        load8(Ns + (ib * 16 + l16) * kNP + 8 * lq, true, x);
        yb = get(16 * ib + 8 * lq);
      }
      const dc_f32x4 o = mma3(split8(x), yb, dc_f32x4{0.f, 0.f, 0.f, 0.f});
      wave_lds_sync();
      put(16 * ib, o);
      wave_lds_sync();
      if (val) *reinterpret_cast<dc_f32x4 *>(ws + lay.u + ((ib * vt + tile) * 64 + lane) * 16) = o;
      else {
        uint16_t *dst = reinterpret_cast<uint16_t *>(ws + lay.w) + (((ib * KS + (c >> 5)) * 2 * 64) + 16 * ((c & 31) >> 3)) * 8 + (c & 7);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const uint16_t hi = f32_to_bf16_bits(o[r]);
          dst[(4 * lq + r) * 8] = hi;
          dst[(64 + 4 * lq + r) * 8] = f32_to_bf16_bits(o[r] - bf16_bits_to_f32(hi));
        }
      }
    }
  }
}

// One wave's operands of one chunk.
template <int D> struct PassOperands {
  static constexpr int KS = D / 32, DT = D / 64;
  dc_bf16x8 wh[KS], wl[KS], q[KS], p[2], kh[DT][2], kl[DT][2];
  dc_f32x4 u[2];
  float g[DT];
  __device__ __forceinline__ void load(const char *ws, const ChunkLayout &lay, int wave, int lane, int e16, int vt, const float *G) {
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      const char *p = ws + lay.w + ((wave * KS + ks) * 2 * 64 + lane) * 16;
      wh[ks] = *reinterpret_cast<const dc_bf16x8 *>(p);
      wl[ks] = *reinterpret_cast<const dc_bf16x8 *>(p + 64 * 16);
      q[ks] = *reinterpret_cast<const dc_bf16x8 *>(ws + lay.q + ((wave * KS + ks) * 64 + lane) * 16);
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) u[e] = *reinterpret_cast<const dc_f32x4 *>(ws + lay.u + ((wave * vt + e16 + e) * 64 + lane) * 16);
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) p[ks] = *reinterpret_cast<const dc_bf16x8 *>(ws + lay.p + ((wave * 2 + ks) * 64 + lane) * 16);
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      g[dt] = G[(wave * DT + dt) * 16 + (lane & 15)];
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const char *p = ws + lay.k + (((wave * DT + dt) * 2 + ks) * 2 * 64 + lane) * 16;
        kh[dt][ks] = *reinterpret_cast<const dc_bf16x8 *>(p);
        kl[dt][ks] = *reinterpret_cast<const dc_bf16x8 *>(p + 64 * 16);
      }
    }
  }
};

// Block = (32 columns e of the state, head, sequence).  Wave w owns rows 16 w .. + 15 of a chunk in the products over the
// state, and channels w D / 4 .. of the state itself, transposed: rows e, columns d.
template <int D>
__global__ void __launch_bounds__(256) k_delta_pass(DeltaArgs a) {
  constexpr int KS = D / 32, DT = D / 64, SP = D + 8, UP = C + 8;
  __shared__ __attribute__((aligned(16))) uint16_t St[2][32 * SP];   // hi / lo of the state, [e][d]
  __shared__ __attribute__((aligned(16))) uint16_t Ut[2][32 * UP];   // of U, [e][t]
  const DeltaShape &z = a.s;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lq = lane >> 4;
  const int e0 = blockIdx.x * 32, h = blockIdx.y, b = blockIdx.z;
  const int chunks = (a.S + C - 1) / C, vt = z.Vp / 16;
  const ChunkLayout lay = chunk_layout(D, z.Vp);
  const int pos0 = a.state->pos;
  const char *ws = a.chunk_ws + ((int64_t)b * chunks * z.heads + h) * lay.total;
  const int64_t step = (int64_t)z.heads * lay.total, ldg = (int64_t)z.heads * D;
  const float *G = a.decay + (int64_t)b * a.S * ldg + h * D;
  float *carried = a.carried + ((int64_t)b * z.heads + h) * D * z.Vp + e0;
  dc_f32x4 S[DT][2];
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      const int d = (wave * DT + dt) * 16 + l16;
      S[dt][e] = dc_f32x4{0.f, 0.f, 0.f, 0.f};
      if (pos0 > 0) S[dt][e] = *reinterpret_cast<const dc_f32x4 *>(carried + (int64_t)d * z.Vp + 16 * e + 4 * lq);
    }
  PassOperands<D> cur;
  auto request = [&](int n) {
    const int last = (n + 1) * C < a.S ? (n + 1) * C - 1 : a.S - 1;
    cur.load(ws + n * step, lay, wave, lane, e0 / 16, vt, G + (int64_t)last * ldg);
  };
  request(0);
  for (int n = 0; n < chunks; ++n) {
    // ---- the state as an operand
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int e = 0; e < 2; ++e)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int at = (16 * e + 4 * lq + r) * SP + (wave * DT + dt) * 16 + l16;
          const uint16_t hi = f32_to_bf16_bits(S[dt][e][r]);
          St[0][at] = hi;
          St[1][at] = f32_to_bf16_bits(S[dt][e][r] - bf16_bits_to_f32(hi));
        }
    __syncthreads();
    dc_f32x4 U[2], O[2];
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      dc_f32x4 x = {0.f, 0.f, 0.f, 0.f}, x2 = x, x3 = x;
      O[e] = x;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const int at = (16 * e + l16) * SP + 32 * ks + 8 * lq;
        const dc_bf16x8 sh = *reinterpret_cast<const dc_bf16x8 *>(St[0] + at), sl = *reinterpret_cast<const dc_bf16x8 *>(St[1] + at);
        x = mma(cur.wh[ks], sh, x);
        x2 = mma(cur.wh[ks], sl, x2);
        x3 = mma(cur.wl[ks], sh, x3);
        O[e] = mma(cur.q[ks], sh, O[e]);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) U[e][r] = cur.u[e][r] - (x[r] + (x2[r] + x3[r]));
      const dc_u32x2 hi = {pack_bf16x2(U[e][0], U[e][1]), pack_bf16x2(U[e][2], U[e][3])};
      const dc_u32x2 lo = {pack_bf16x2(U[e][0] - bf_lo(hi.x), U[e][1] - bf_hi(hi.x)), pack_bf16x2(U[e][2] - bf_lo(hi.y), U[e][3] - bf_hi(hi.y))};
      const int at = (16 * e + l16) * UP + 16 * wave + 4 * lq;
      *reinterpret_cast<dc_u32x2 *>(Ut[0] + at) = hi;
      *reinterpret_cast<dc_u32x2 *>(Ut[1] + at) = lo;
    }
    __syncthreads();
    // ---- read-out and update
    Halves ua[2][2];
#pragma unroll
    for (int e = 0; e < 2; ++e)
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) {
        const int at = (16 * e + l16) * UP + 32 * ks + 8 * lq;
        ua[e][ks].hi = *reinterpret_cast<const dc_bf16x8 *>(Ut[0] + at);
        ua[e][ks].lo = *reinterpret_cast<const dc_bf16x8 *>(Ut[1] + at);
      }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const float w = fast_exp(cur.g[dt]);
#pragma unroll
      for (int e = 0; e < 2; ++e) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[dt][e][r] *= w;
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          Halves kb;
          kb.hi = cur.kh[dt][ks];
          kb.lo = cur.kl[dt][ks];
          S[dt][e] = mma3(ua[e][ks], kb, S[dt][e]);
        }
      }
    }
#pragma unroll
    for (int e = 0; e < 2; ++e) {
#pragma unroll
      for (int ks = 0; ks < 2; ++ks) O[e] = mma(cur.p[ks], ua[e][ks].hi, O[e]);   // U's columns serve as B: lane = column e
    }
    const int t0 = n * C + 16 * wave + 4 * lq;
    if (n + 1 < chunks) request(n + 1);
#pragma unroll
    for (int e = 0; e < 2; ++e)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (t0 + r < a.S) a.o[(((int64_t)b * a.S + t0 + r) * z.heads + h) * z.Vp + e0 + 16 * e + l16] = O[e][r];
  }
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int e = 0; e < 2; ++e)
      *reinterpret_cast<dc_f32x4 *>(carried + (int64_t)((wave * DT + dt) * 16 + l16) * z.Vp + 16 * e + 4 * lq) = S[dt][e];
  if (blockIdx.x == 0) update_ring<bf16_raw>(a, b, h, pos0, tid, 256);
}

bool delta_chunk_serves(int dtype, const DeltaShape &z) {
  return dtype == RAI_BF16 && (z.Dk == 64 || z.Dk == 128 || z.Dk == 256) && z.Vp % 32 == 0;
}
size_t delta_chunk_ws_bytes(const DeltaShape &z, int64_t max_batch, int64_t max_rows) {
  return (size_t)(max_rows / C + max_batch) * z.heads * chunk_layout(z.Dk, z.Vp).total;
}

template <int D> static int launch_chunks(hipStream_t st, const DeltaArgs &a) {
  const DeltaShape &z = a.s;
  hipLaunchKernelGGL(k_delta_chunk<D>, dim3((a.S + C - 1) / C, z.heads, a.B), dim3(256), 0, st, a);
  RAI_TRY(launch_check("delta_chunk"));
  hipLaunchKernelGGL(k_delta_pass<D>, dim3(z.Vp / 32, z.heads, a.B), dim3(256), 0, st, a);
  return launch_check("delta_pass");
}
int launch_delta_chunks(hipStream_t st, const DeltaArgs &a) {
  RAI_REQUIRE(a.chunk_ws && delta_chunk_serves(RAI_BF16, a.s), RAI_ERR_BAD_ARG, "delta chunks: not served");
  if (a.s.Dk == 64) return launch_chunks<64>(st, a);
  if (a.s.Dk == 128) return launch_chunks<128>(st, a);
  return launch_chunks<256>(st, a);
}

}  // namespace rai
