// Attention over cached latents.  A layer's cache holds one normalised latent c[Rp] per token, and head h's key and
// value are uk[h] c and uv[h] c.  Two evaluations of the same sums:
//   - long runs of query rows (prefill) expand keys and values with one Linear and use the flash kernel
//     (attention.hip); nothing here but the norm of the latents;
//   - few query rows (decode, short portions) are absorbed: q . (uk c) = (uk^T q) . c, so the query is taken into the
//     latent space once per head, every head then reads the same cache rows, and the weighted sum of latents goes
//     through uv at the end.  The cache is read once for all heads instead of once per head.
#include <cstdlib>

#include "latent.h"

namespace rai {

template <typename T> struct alignas(16) LPack { T v[16 / sizeof(T)]; };

// acc + the dot product of two packs; bf16 pairs through v_dot2_f32_bf16 (exact products, f32 sums)
__device__ __forceinline__ float pack_dot(const LPack<float> &a, const LPack<float> &b, float acc) {
#pragma unroll
  for (int e = 0; e < 4; ++e) acc = fmaf(a.v[e], b.v[e], acc);
  return acc;
}
__device__ __forceinline__ float pack_dot(const LPack<bf16_raw> &a, const LPack<bf16_raw> &b, float acc) {
  typedef __attribute__((ext_vector_type(2))) __bf16 pair;
#pragma unroll
  for (int e = 0; e < 8; e += 2) {
    pair p, q;
    __builtin_memcpy(&p, &a.v[e], 4);
    __builtin_memcpy(&q, &b.v[e], 4);
    acc = __builtin_amdgcn_fdot2_f32_bf16(p, q, acc, false);
  }
  return acc;
}

// ---------------------------------------------------------------- norms of the two latents, cache append
// One wave per (row, latent): kind 0 = query latent, 1 = cached latent.
template <typename T>
__global__ void __launch_bounds__(256) k_latent_norm(LatentNormArgs a) {
  constexpr int V = 16 / sizeof(T);
  const int64_t job = blockIdx.x * 4ll + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (job >= 2ll * a.B * a.S) return;
  const int64_t row = job >> 1;
  const bool latent = job & 1;
  const int n = latent ? a.kv_rank : a.q_rank;
  const T *x = (const T *)a.dn + row * a.ldn + (latent ? a.Qp : 0);
  const T *w = (const T *)(latent ? a.c_w : a.q_w);
  T *o1, *o2 = nullptr;
  if (latent) {
    const int b = (int)(row / a.S), s = (int)(row % a.S);
    o1 = (T *)a.cache + ((int64_t)b * a.Tmax + a.state->pos + s) * a.Rp;
    if (a.cn) o2 = (T *)a.cn + row * a.Rp;
  } else {
    o1 = (T *)a.cq + row * a.Qp;
  }
  float q = 0.f;
  const int packs = n / V;
  for (int p = lane; p < packs; p += 64) {
    const LPack<T> v = *reinterpret_cast<const LPack<T> *>(x + p * V);
#pragma unroll
    for (int e = 0; e < V; ++e) { const float f = (float)Scalar<T>::load(&v.v[e]); q = fmaf(f, f, q); }
  }
  for (int i = packs * V + lane; i < n; i += 64) { const float f = (float)Scalar<T>::load(x + i); q = fmaf(f, f, q); }
  const float sc = 1.0f / sqrtf(wave_sum(q) / (float)n + a.eps);
  for (int p = lane; p < packs; p += 64) {
    LPack<T> v = *reinterpret_cast<const LPack<T> *>(x + p * V);
#pragma unroll
    for (int e = 0; e < V; ++e) Scalar<T>::store(&v.v[e], (float)Scalar<T>::load(&v.v[e]) * sc * (float)Scalar<T>::load(w + p * V + e));
    *reinterpret_cast<LPack<T> *>(o1 + p * V) = v;
    if (o2) *reinterpret_cast<LPack<T> *>(o2 + p * V) = v;
  }
  // the last partial pack, and zeros in the padding
  const int np = latent ? a.Rp : a.Qp;
  for (int i = packs * V + lane; i < np; i += 64) {
    const float f = i < n ? (float)Scalar<T>::load(x + i) * sc * (float)Scalar<T>::load(w + i) : 0.f;
    Scalar<T>::store(o1 + i, f);
    if (o2) Scalar<T>::store(o2 + i, f);
  }
}

int launch_latent_norm(hipStream_t st, int dtype, const LatentNormArgs &a) {
  const int64_t jobs = 2ll * a.B * a.S;
  const dim3 grid((unsigned)((jobs + 3) / 4)), block(256);
  if (dtype == RAI_BF16) hipLaunchKernelGGL(k_latent_norm<bf16_raw>, grid, block, 0, st, a);
  else hipLaunchKernelGGL(k_latent_norm<float>, grid, block, 0, st, a);
  return launch_check("latent_norm");
}

// ---------------------------------------------------------------- queries into the latent space
// qa[row, h, r] = sum_d WukT[h][r][d] q[row, h * Dp + d].  A block serves 64 latent features of one head; four threads
// share a feature's dot product, their 16-byte pieces of it interleaved so that a wave reads whole lines.  The weights
// stay in registers (NP pieces per thread; NP == 0: re-read) while the rows of blockIdx.z's share pass by.
template <typename T, int NP>
__global__ void __launch_bounds__(256) k_latent_absorb(const T *q, const T *WukT, T *qa, int rows, int rows_per_block, int heads, int Dp, int Rp) {
  constexpr int V = 16 / sizeof(T);
  const int h = blockIdx.x, r = blockIdx.y * 64 + (threadIdx.x >> 2), part = threadIdx.x & 3;
  const int np = NP > 0 ? NP : Dp / (4 * V);
  const T *w = WukT + ((int64_t)h * Rp + r) * Dp + part * V;
  LPack<T> wr[NP > 0 ? NP : 1];
#pragma unroll
  for (int i = 0; i < NP; ++i) wr[i] = *reinterpret_cast<const LPack<T> *>(w + i * 4 * V);
  const int m0 = blockIdx.z * rows_per_block, m1 = m0 + rows_per_block < rows ? m0 + rows_per_block : rows;
  auto finish = [&](int m, float acc) {
    acc += __shfl_xor(acc, 1, 64);
    acc += __shfl_xor(acc, 2, 64);
    if (part == 0 && m < m1) Scalar<T>::store(qa + ((int64_t)m * heads + h) * Rp + r, acc);
  };
  if constexpr (NP > 0) {
    constexpr int G = NP <= 4 ? 4 : 2;   // rows whose queries are in flight together
    for (int m = m0; m < m1; m += G) {
      LPack<T> qv[G][NP];
#pragma unroll
      for (int g = 0; g < G; ++g) {
        const T *qr = q + ((int64_t)(m + g < m1 ? m + g : m1 - 1) * heads + h) * Dp + part * V;
#pragma unroll
        for (int i = 0; i < NP; ++i) qv[g][i] = *reinterpret_cast<const LPack<T> *>(qr + i * 4 * V);
      }
#pragma unroll
      for (int g = 0; g < G; ++g) {
        float acc = 0.f;
#pragma unroll
        for (int i = 0; i < NP; ++i) acc = pack_dot(wr[i], qv[g][i], acc);
        finish(m + g, acc);
      }
    }
  } else {
    for (int m = m0; m < m1; ++m) {
      const T *qr = q + ((int64_t)m * heads + h) * Dp + part * V;
      float acc = 0.f;
      for (int i = 0; i < np; ++i)
        acc = pack_dot(*reinterpret_cast<const LPack<T> *>(w + i * 4 * V), *reinterpret_cast<const LPack<T> *>(qr + i * 4 * V), acc);
      finish(m, acc);
    }
  }
}

template <typename T> __global__ void __launch_bounds__(256) k_latent_transpose_uk(const T *uk, T *ukT, int heads, int Dp, int Rp) {
  const int64_t n = (int64_t)heads * Dp * Rp;
  for (int64_t i = blockIdx.x * 256ll + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const int d = (int)(i % Dp);
    const int64_t hr = i / Dp;
    const int r = (int)(hr % Rp), h = (int)(hr / Rp);
    ukT[i] = uk[((int64_t)h * Dp + d) * Rp + r];
  }
}
int launch_latent_transpose_uk(hipStream_t st, int dtype, const void *Wuk, void *WukT, int heads, int Dp, int Rp) {
  if (dtype == RAI_BF16)
    hipLaunchKernelGGL(k_latent_transpose_uk<uint16_t>, dim3(kNumCU * 4), dim3(256), 0, st, (const uint16_t *)Wuk, (uint16_t *)WukT, heads, Dp, Rp);
  else
    hipLaunchKernelGGL(k_latent_transpose_uk<float>, dim3(kNumCU * 4), dim3(256), 0, st, (const float *)Wuk, (float *)WukT, heads, Dp, Rp);
  return launch_check("latent_transpose_uk");
}

// ---------------------------------------------------------------- absorbed attention
// The context is split for about this many blocks: two per CU of the MFMA form (a block serves up to 16 heads), four of
// the other.
constexpr int kLatentBlocks = 4 * kNumCU, kLatentMfmaBlocks = 2 * kNumCU;

// Keys of query row m: the last min(pos + 1, window) positions up to its own, shared out evenly over the splits.
struct LatentSpan { int lo, hi; };
__device__ __forceinline__ LatentSpan latent_span(const LatentAttnArgs &a, int m, int split) {
  const int pos = a.state->pos + m % a.S;
  const int n = a.window > 0 && a.window < pos + 1 ? a.window : pos + 1;
  const int per = (n + a.splits - 1) / a.splits;
  const int lo = pos + 1 - n + split * per;
  return {lo, lo + per < pos + 1 ? lo + per : pos + 1};
}

// ws of (row, head, split): max, sum, weighted latents[Rp]
__device__ __forceinline__ float *latent_ws(const LatentAttnArgs &a, int m, int h, int split) {
  return a.ws + (((int64_t)m * a.heads + h) * a.splits + split) * (a.Rp + 2);
}

// Any dtype: one block per (split, head, row), keys 64 at a time, scores in f32 in LDS.
template <typename T>
__global__ void __launch_bounds__(256) k_latent_attn(LatentAttnArgs a) {
  constexpr int V = 16 / sizeof(T);
  extern __shared__ __attribute__((aligned(16))) float la_lds[];   // qa[Rp] | o[Rp] | p[64]
  __shared__ float sh_m, sh_l, sh_alpha;
  const int split = blockIdx.x, h = blockIdx.y, m = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  float *qs = la_lds, *o = qs + a.Rp, *p = o + a.Rp;
  const LatentSpan sp = latent_span(a, m, split);
  float *ws = latent_ws(a, m, h, split);
  if (sp.lo >= sp.hi) {
    if (tid == 0) { ws[0] = -INFINITY; ws[1] = 0.f; }
    return;
  }
  const T *qa = (const T *)a.qa + ((int64_t)m * a.heads + h) * a.Rp;
  for (int r = tid; r < a.Rp; r += 256) { qs[r] = (float)Scalar<T>::load(qa + r); o[r] = 0.f; }
  if (tid == 0) { sh_m = -INFINITY; sh_l = 0.f; }
  const T *cache = (const T *)a.cache + (int64_t)(m / a.S) * a.Tmax * a.Rp;
  for (int k0 = sp.lo; k0 < sp.hi; k0 += 64) {
    const int nk = sp.hi - k0 < 64 ? sp.hi - k0 : 64;
    __syncthreads();
    for (int k = wave; k < nk; k += 4) {
      const T *c = cache + (int64_t)(k0 + k) * a.Rp;
      float acc = 0.f;
      for (int r = lane * V; r < a.Rp; r += 64 * V) {
        const LPack<T> cv = *reinterpret_cast<const LPack<T> *>(c + r);
#pragma unroll
        for (int e = 0; e < V; ++e) acc = fmaf(qs[r + e], (float)Scalar<T>::load(&cv.v[e]), acc);
      }
      acc = wave_sum(acc);
      if (lane == 0) p[k] = acc * a.scale;
    }
    __syncthreads();
    if (wave == 0) {
      const float s = lane < nk ? p[lane] : -INFINITY;
      const float m_old = sh_m, m_new = fmaxf(m_old, wave_max(s));
      const float e = expf(s - m_new);
      const float alpha = expf(m_old - m_new), l = sh_l * alpha + wave_sum(e);   // every lane reads before lane 0 writes
      p[lane] = e;
      if (lane == 0) { sh_m = m_new; sh_l = l; sh_alpha = alpha; }
    }
    __syncthreads();
    for (int r = tid; r < a.Rp; r += 256) {
      float acc = o[r] * sh_alpha;
      for (int k = 0; k < nk; ++k) acc = fmaf(p[k], (float)Scalar<T>::load(cache + (int64_t)(k0 + k) * a.Rp + r), acc);
      o[r] = acc;
    }
  }
  __syncthreads();
  if (tid == 0) { ws[0] = sh_m; ws[1] = sh_l; }
  for (int r = tid; r < a.Rp; r += 256) ws[2 + r] = o[r];
}

// bf16 on MFMA: one block per (split, 16 heads, row).  The keys' latents come 64 at a time into LDS, where they serve
// twice: as they lie for the scores S[16 heads][64 keys] = QA . C^T (wave w takes keys 16w .. 16w+15), and read
// transposed (ds_read_b64_tr_b16) for O[16 heads][Rp] += P . C (wave w takes a quarter of the latent features).  The
// softmax statistics of 4 heads live in the registers of each wave.  NT >= Rp / 64: accumulator tiles of a wave.
//   16x16x32 fragments: lane l holds row (column) l % 16, k = 8 (l / 16) .. + 7; accumulator register r of lane l is
//   D[4 (l / 16) + r][l % 16].  A transposing read hands lane i of 16 element i % 4 of the 8 bytes that lanes
//   4j + i / 4, j = 0..3, point at: with lane a pointing at row a / 4, columns 4 (a % 4), lane i receives column i.
typedef __attribute__((ext_vector_type(8))) __bf16 la_bf16x8;
typedef __attribute__((ext_vector_type(4))) float la_f32x4;
typedef __attribute__((ext_vector_type(4))) short la_s16x4;
typedef __attribute__((ext_vector_type(4))) uint32_t la_u32x4;

constexpr int kLatKeys = 64, kLatPPitch = kLatKeys + 8, kLatSPitch = kLatKeys + 4;
static size_t latent_mfma_lds(int Rp) {
  return (size_t)kLatKeys * (Rp + 8) * 2 + 16 * kLatSPitch * 4 + 16 * kLatPPitch * 2 + 16 * 4;
}

template <int NT>
__global__ void __launch_bounds__(256) k_latent_attn_mfma(LatentAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint16_t lm_lds[];
  const int split = blockIdx.x, h0 = blockIdx.y * 16, m = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, lq = lane >> 4;
  const int Rp = a.Rp, pitch = Rp + 8, nt = Rp / 64, cpr = Rp / 8;
  uint16_t *cs = lm_lds;                                                    // [64][pitch]
  float *sc = reinterpret_cast<float *>(cs + kLatKeys * pitch);            // [16][kLatSPitch]
  uint16_t *ps = reinterpret_cast<uint16_t *>(sc + 16 * kLatSPitch);       // [16][kLatPPitch]
  float *al = reinterpret_cast<float *>(ps + 16 * kLatPPitch);             // [16]
  const LatentSpan sp = latent_span(a, m, split);
  const int n_heads = a.heads - h0 < 16 ? a.heads - h0 : 16;
  if (sp.lo >= sp.hi) {
    if (tid < n_heads) {
      float *ws = latent_ws(a, m, h0 + tid, split);
      ws[0] = -INFINITY;
      ws[1] = 0.f;
    }
    return;
  }
  const int hq = h0 + (l16 < n_heads ? l16 : n_heads - 1);   // heads past the end repeat the last one and are not stored
  const uint16_t *qa = (const uint16_t *)a.qa + ((int64_t)m * a.heads + hq) * Rp + lq * 8;
  const uint16_t *cache = (const uint16_t *)a.cache + (int64_t)(m / a.S) * a.Tmax * Rp;
  la_bf16x8 qf[2 * NT];
#pragma unroll
  for (int ks = 0; ks < 2 * NT; ++ks)
    if (ks < 2 * nt) qf[ks] = *reinterpret_cast<const la_bf16x8 *>(qa + ks * 32);
  la_f32x4 o[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = la_f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run[4], l_run[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) { m_run[i] = -INFINITY; l_run[i] = 0.f; }

  for (int k0 = sp.lo; k0 < sp.hi; k0 += kLatKeys) {
    if (k0 != sp.lo) __syncthreads();   // the tile before has been read
    constexpr int U = 8;   // a thread's pieces of the tile in flight
    for (int c = tid; c < kLatKeys * cpr; c += 256 * U) {
      la_u32x4 v[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int cc = c + u * 256;
        const int row = cc / cpr;
        const int key = k0 + row < sp.hi ? k0 + row : sp.hi - 1;   // rows past the span repeat its last key, masked below
        if (cc < kLatKeys * cpr) v[u] = *reinterpret_cast<const la_u32x4 *>(cache + (int64_t)key * Rp + (cc - row * cpr) * 8);
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int cc = c + u * 256;
        const int row = cc / cpr;
        if (cc < kLatKeys * cpr) *reinterpret_cast<la_u32x4 *>(cs + row * pitch + (cc - row * cpr) * 8) = v[u];
      }
    }
    __syncthreads();
    {
      la_f32x4 s = {0.f, 0.f, 0.f, 0.f};
      const uint16_t *cr = cs + (16 * wave + l16) * pitch + lq * 8;
#pragma unroll
      for (int ks = 0; ks < 2 * NT; ++ks)
        if (ks < 2 * nt) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], *reinterpret_cast<const la_bf16x8 *>(cr + ks * 32), s, 0, 0, 0);
      const bool seen = k0 + 16 * wave + l16 < sp.hi;
#pragma unroll
      for (int r = 0; r < 4; ++r) sc[(4 * lq + r) * kLatSPitch + 16 * wave + l16] = seen ? s[r] * a.scale : -INFINITY;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {   // heads 4 * wave + i, one key per lane; every tile has a visible key
      const float s = sc[(4 * wave + i) * kLatSPitch + lane];
      const float m_new = fmaxf(m_run[i], wave_max(s));
      const float p = __expf(s - m_new), alpha = __expf(m_run[i] - m_new);
      l_run[i] = l_run[i] * alpha + wave_sum(p);
      m_run[i] = m_new;
      ps[(4 * wave + i) * kLatPPitch + lane] = f32_to_bf16_bits(p);
      if (lane == 0) al[4 * wave + i] = alpha;
    }
    __syncthreads();
    const la_f32x4 scale = *reinterpret_cast<const la_f32x4 *>(al + 4 * lq);
    la_bf16x8 pf[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) pf[ks] = *reinterpret_cast<const la_bf16x8 *>(ps + l16 * kLatPPitch + ks * 32 + lq * 8);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if (t < nt) {
#pragma unroll
        for (int r = 0; r < 4; ++r) o[t][r] *= scale[r];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
          typedef __attribute__((address_space(3))) la_s16x4 *tr_ptr;
          const uint16_t *src = cs + (ks * 32 + lq * 8 + (l16 >> 2)) * pitch + (wave * nt + t) * 16 + 4 * (l16 & 3);
          const la_s16x4 lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_ptr)src);
          const la_s16x4 hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((tr_ptr)(src + 4 * pitch));
          const __attribute__((ext_vector_type(8))) short cf = {lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
          o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[ks], __builtin_bit_cast(la_bf16x8, cf), o[t], 0, 0, 0);
        }
      }
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int h = 4 * lq + r;
    if (h < n_heads) {
      float *ws = latent_ws(a, m, h0 + h, split) + 2;
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if (t < nt) ws[(wave * nt + t) * 16 + l16] = o[t][r];
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int h = 4 * wave + i;
    if (lane == 0 && h < n_heads) {
      float *ws = latent_ws(a, m, h0 + h, split);
      ws[0] = m_run[i];
      ws[1] = l_run[i];
    }
  }
}

// Merges the splits of one (row, head) and takes the latent through `features` rows of uv and the output gate.  With few
// rows a head's features are shared out over several blocks, each of which merges for itself (what is merged is small and
// in the L2); with many, one block serves the whole head.  A wave's first weight rows are requested before anything else.
// R weight rows of C 16-byte chunks per lane are requested at a time.
template <typename T, int R, int C>
__global__ void __launch_bounds__(256) k_latent_out(LatentAttnArgs a, int features) {
  constexpr int V = 16 / sizeof(T);
  extern __shared__ __attribute__((aligned(16))) float lo_lds[];   // latents[Rp] | weight[splits]
  const int h = blockIdx.x, d0 = blockIdx.y * features, m = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  T *o = reinterpret_cast<T *>(lo_lds);
  float *wt = lo_lds + a.Rp;
  const float *ws = latent_ws(a, m, h, 0);
  const int64_t step = a.Rp + 2;
  const T *W = (const T *)a.Wuv + ((int64_t)h * a.Dp + d0 + wave * R) * a.Rp + lane * V;   // rows d0 + wave * R + 16 i + r
  LPack<T> w[R][C], next[R][C];
  const bool whole = a.Rp <= C * 64 * V;   // one request holds whole rows: the next rows fly while these are multiplied
  auto request = [&](LPack<T> (&w)[R][C], const T *p, int c0) {
#pragma unroll
    for (int r = 0; r < R; ++r)
#pragma unroll
      for (int c = 0; c < C; ++c)
        if ((c0 + c) * 64 * V + lane * V < a.Rp) w[r][c] = *reinterpret_cast<const LPack<T> *>(p + (int64_t)r * a.Rp + (c0 + c) * 64 * V);
  };
  request(w, W, 0);
  // the splits' weights: one split per lane, every wave for itself
  {
    constexpr int SL = kLatentBlocks / 64;   // most splits of a lane
    float ms[SL], ls[SL], mx = -INFINITY, l = 0.f;
#pragma unroll
    for (int i = 0; i < SL; ++i) {
      const int s = lane + i * 64;
      ms[i] = s < a.splits ? ws[s * step] : -INFINITY;
      ls[i] = s < a.splits ? ws[s * step + 1] : 0.f;
      mx = fmaxf(mx, ms[i]);
    }
    mx = wave_max(mx);
#pragma unroll
    for (int i = 0; i < SL; ++i) {
      ms[i] = ls[i] > 0.f ? expf(ms[i] - mx) : 0.f;
      l = fmaf(ls[i], ms[i], l);
    }
    const float inv = 1.0f / wave_sum(l);
    if (wave == 0) {
#pragma unroll
      for (int i = 0; i < SL; ++i)
        if (lane + i * 64 < a.splits) wt[lane + i * 64] = ms[i] * inv;
    }
  }
  __syncthreads();
  typedef __attribute__((ext_vector_type(2))) float f32x2;
  for (int r = 2 * tid; r < a.Rp; r += 512) {
    f32x2 acc = {0.f, 0.f};
    for (int s0 = 0; s0 < a.splits; s0 += 16) {   // sixteen splits in flight
      f32x2 x[16];
#pragma unroll
      for (int i = 0; i < 16; ++i) x[i] = *reinterpret_cast<const f32x2 *>(ws + (s0 + i < a.splits ? s0 + i : a.splits - 1) * step + 2 + r);
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const float f = s0 + i < a.splits ? wt[s0 + i] : 0.f;
        if (f > 0.f) { acc.x = fmaf(f, x[i].x, acc.x); acc.y = fmaf(f, x[i].y, acc.y); }   // a split without keys has written no latents
      }
    }
    // the merged latent meets uv as the value it stands for would meet the cache: in T
    Scalar<T>::store(o + r, acc.x);
    Scalar<T>::store(o + r + 1, acc.y);
  }
  __syncthreads();
  for (int d = d0 + wave * R; d < d0 + features; d += 4 * R, W += (int64_t)4 * R * a.Rp) {
    float acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.f;
    const bool more = whole && d + 4 * R < d0 + features;
    if (more) request(next, W + (int64_t)4 * R * a.Rp, 0);
    for (int c0 = 0; c0 * 64 * V < a.Rp; c0 += C) {
      if (!whole && (c0 || d != d0 + wave * R)) request(w, W, c0);
#pragma unroll
      for (int c = 0; c < C; ++c) {
        const int k = (c0 + c) * 64 * V + lane * V;
        if (k < a.Rp) {
          const LPack<T> ov = *reinterpret_cast<const LPack<T> *>(o + k);
#pragma unroll
          for (int r = 0; r < R; ++r) acc[r] = pack_dot(w[r][c], ov, acc[r]);
        }
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = wave_sum(acc[r]);
    if (lane < R) {
      float v = acc[0];
#pragma unroll
      for (int r = 1; r < R; ++r) v = lane == r ? acc[r] : v;
      const int f = h * a.Dp + d + lane;
      const float g = (float)Scalar<T>::load((const T *)a.gate + (int64_t)m * a.ldg + f);
      Scalar<T>::store((T *)a.out + (int64_t)m * a.ldo + f, v / (1.0f + expf(-g)));
    }
    if (more) {
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int c = 0; c < C; ++c) w[r][c] = next[r][c];
    }
  }
}

size_t latent_attn_ws_floats(int rows, int heads, int Rp) {
  return ((size_t)rows * heads + kLatentBlocks + 16 * kLatentMfmaBlocks) * (Rp + 2);
}

static bool latent_mfma_serves(const LatentAttnArgs &a) {
  const char *off = getenv("RAI_HIP_NO_LATENT_MFMA");   // read per call: the tests compare both forms in one process
  return a.Rp <= 1024 && latent_mfma_lds(a.Rp) <= 150 * 1024 && !(off && *off && *off != '0');
}
template <int NT> static int launch_latent_mfma(hipStream_t st, const LatentAttnArgs &a, int rows) {
  const size_t lds = latent_mfma_lds(a.Rp);
  static bool attr_set = false;
  if (!attr_set) {
    RAI_HIP_TRY(hipFuncSetAttribute((const void *)k_latent_attn_mfma<NT>, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
    attr_set = true;
  }
  hipLaunchKernelGGL(k_latent_attn_mfma<NT>, dim3(a.splits, (a.heads + 15) / 16, rows), dim3(256), lds, st, a);
  return launch_check("latent_attn_mfma");
}

template <typename T> static int launch_latent_absorb(hipStream_t st, const LatentAttnArgs &a, int rows) {
  const int per = rows <= 8 ? rows : 8;
  const dim3 grid(a.heads, a.Rp / 64, (rows + per - 1) / per), block(256);
#define RAI_ABSORB(NP) hipLaunchKernelGGL((k_latent_absorb<T, NP>), grid, block, 0, st, (const T *)a.q, (const T *)a.WukT, (T *)a.qa, rows, per, a.heads, a.Dp, a.Rp)
  const int np = sizeof(T) == 2 ? a.Dp / 32 : 0;
  if (np == 1 && a.Dp == 32) RAI_ABSORB(1);
  else if (np == 2 && a.Dp == 64) RAI_ABSORB(2);
  else if (np == 4 && a.Dp == 128) RAI_ABSORB(4);
  else if (np == 6 && a.Dp == 192) RAI_ABSORB(6);
  else if (np == 8 && a.Dp == 256) RAI_ABSORB(8);
  else RAI_ABSORB(0);
#undef RAI_ABSORB
  return launch_check("latent_absorb");
}

template <typename T> static int launch_latent_attention_t(hipStream_t st, LatentAttnArgs a) {
  const int rows = a.B * a.S;
  RAI_TRY(launch_latent_absorb<T>(st, a, rows));
  const int n_max = a.window > 0 && a.window < a.Tmax ? a.window : a.Tmax;
  const bool mfma = sizeof(T) == 2 && latent_mfma_serves(a);
  int splits = mfma ? kLatentMfmaBlocks / (rows * ((a.heads + 15) / 16)) : kLatentBlocks / (rows * a.heads);
  if (splits > (n_max + 63) / 64) splits = (n_max + 63) / 64;
  a.splits = splits < 1 ? 1 : splits;
  if (mfma) {
    if (a.Rp <= 128) RAI_TRY(launch_latent_mfma<2>(st, a, rows));
    else if (a.Rp <= 256) RAI_TRY(launch_latent_mfma<4>(st, a, rows));
    else if (a.Rp <= 512) RAI_TRY(launch_latent_mfma<8>(st, a, rows));
    else RAI_TRY(launch_latent_mfma<16>(st, a, rows));
  } else {
    const size_t lds = (size_t)(2 * a.Rp + 64) * sizeof(float);
    hipLaunchKernelGGL(k_latent_attn<T>, dim3(a.splits, a.heads, rows), dim3(256), lds, st, a);
    RAI_TRY(launch_check("latent_attn"));
  }
  const bool narrow = a.Rp <= 64 * (int)(16 / sizeof(T));   // one chunk per lane holds a weight row
  const bool many = rows * a.heads >= kNumCU;
  const int features = many ? a.Dp : 16;
#define RAI_LATENT_OUT(R, C) \
  hipLaunchKernelGGL((k_latent_out<T, R, C>), dim3(a.heads, a.Dp / features, rows), dim3(256), (size_t)(a.Rp + a.splits) * sizeof(float), st, a, features)
  if (many) { if (narrow) RAI_LATENT_OUT(8, 1); else RAI_LATENT_OUT(8, 2); }
  else { if (narrow) RAI_LATENT_OUT(4, 1); else RAI_LATENT_OUT(4, 2); }
#undef RAI_LATENT_OUT
  return launch_check("latent_out");
}

int launch_latent_attention(hipStream_t st, int dtype, LatentAttnArgs a) {
  RAI_REQUIRE(a.B > 0 && a.S > 0 && a.heads > 0 && a.heads <= 65535 && a.Dp % 32 == 0 && a.Rp % 64 == 0 && (int64_t)a.B * a.S <= 65535,
              RAI_ERR_BAD_SHAPE, "latent attention: %d rows, %d heads of %d, latent %d", a.B * a.S, a.heads, a.Dp, a.Rp);
  RAI_REQUIRE(a.Rp <= 7168, RAI_ERR_UNSUPPORTED, "latent attention: latent %d too wide", a.Rp);
  return dtype == RAI_BF16 ? launch_latent_attention_t<bf16_raw>(st, a) : launch_latent_attention_t<float>(st, a);
}

}  // namespace rai
