// Gated delta rule with a decay per key channel (see delta.h).
//   k_delta_prep  convolution + silu of every token, and what makes its queries and keys unit vectors
//   k_delta_decay decays and step sizes, for k_delta_scan (the chunks form their own)
//   k_delta_scan  the recurrence, token after token: a block owns 16 columns of one head's state, 16 lanes to a column
//                 (f32 models, few tokens, head sizes the chunked form of delta_chunk.hip does not serve)
//   k_delta_out   norm over the head's values, weight and output gate
//   k_delta_step  all of it for one token per sequence: a block owns a head, its state goes through registers once
#include <cstdlib>

#include "delta.h"
#include "delta_device.h"

namespace rai {

// Sum over the 16 lanes of a row, in every lane.
__device__ __forceinline__ float row16_sum(float v) {
#define RAI_ROW_ADD(ctrl) v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), ctrl, 0xf, 0xf, true))
  RAI_ROW_ADD(0xB1);    // quad_perm [1, 0, 3, 2]
  RAI_ROW_ADD(0x4E);    // quad_perm [2, 3, 0, 1]
  RAI_ROW_ADD(0x141);   // mirror within 8 lanes
  RAI_ROW_ADD(0x140);   // mirror within 16 lanes
#undef RAI_ROW_ADD
  return v;
}

// Channel c of token s after convolution and silu.
template <typename T>
__device__ __forceinline__ float conv_silu(const DeltaArgs &a, int b, int s, int pos0, int c) {
  const DeltaShape &z = a.s;
  float y = 0.f;
  for (int j = 0; j < z.taps; ++j) {
    const int t = s - (z.taps - 1) + j;   // token of this call, or an earlier one in the ring
    float x = 0.f;
    if (t >= 0) x = ld<T>(a.dn, ((int64_t)b * a.S + t) * z.ldn + c);
    else if (pos0 + t >= 0) x = ld<T>(a.ring, ((int64_t)b * z.taps + (pos0 + t) % z.taps) * z.channels + c);
    y = fmaf(x, ld<T>(a.conv, (int64_t)c * z.taps + j), y);
  }
  return y * dl_sigmoid(y);
}

constexpr int kPrepTokens = 8;
constexpr int kChunkedFrom = 24;   // tokens of a call from which on the chunked form is the faster one
template <typename T> struct alignas(2 * sizeof(T)) Pair { T v[2]; };
template <typename T> __device__ __forceinline__ float2 ld2(const void *p, int64_t i) {
  const Pair<T> x = *reinterpret_cast<const Pair<T> *>((const T *)p + i);
  return make_float2((float)Scalar<T>::load(&x.v[0]), (float)Scalar<T>::load(&x.v[1]));
}

template <typename T> __device__ __forceinline__ float as_stored(float x) {
  T t;
  Scalar<T>::store(&t, x);
  return (float)Scalar<T>::load(&t);
}

// Channels c, c + 1 (c even) of kPrepTokens tokens from s0 on, after convolution and silu; TAPS == 0: any number of taps.
template <typename T, int TAPS>
__device__ __forceinline__ void conv_run(const DeltaArgs &a, int b, int s0, int pos0, int c, float2 (&y)[kPrepTokens]) {
  const DeltaShape &z = a.s;
  if constexpr (TAPS > 0) {
    float2 x[kPrepTokens + TAPS - 1], w[TAPS];
#pragma unroll
    for (int i = 0; i < kPrepTokens + TAPS - 1; ++i) {
      const int t = s0 - (TAPS - 1) + i;   // token of this call, or an earlier one in the ring
      x[i] = make_float2(0.f, 0.f);
      if (t >= 0 && t < a.S) x[i] = ld2<T>(a.dn, ((int64_t)b * a.S + t) * z.ldn + c);
      else if (t < 0 && pos0 + t >= 0) x[i] = ld2<T>(a.ring, ((int64_t)b * TAPS + (pos0 + t) % TAPS) * z.channels + c);
    }
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[j] = make_float2(ld<T>(a.conv, (int64_t)c * TAPS + j), ld<T>(a.conv, (int64_t)(c + 1) * TAPS + j));
#pragma unroll
    for (int i = 0; i < kPrepTokens; ++i) {
      float2 v = make_float2(0.f, 0.f);
#pragma unroll
      for (int j = 0; j < TAPS; ++j) {
        v.x = fmaf(x[i + j].x, w[j].x, v.x);
        v.y = fmaf(x[i + j].y, w[j].y, v.y);
      }
      y[i] = make_float2(v.x * dl_sigmoid(v.x), v.y * dl_sigmoid(v.y));
    }
  } else {
#pragma unroll
    for (int i = 0; i < kPrepTokens; ++i)
      y[i] = s0 + i < a.S ? make_float2(conv_silu<T>(a, b, s0 + i, pos0, c), conv_silu<T>(a, b, s0 + i, pos0, c + 1)) : make_float2(0.f, 0.f);
  }
}

// A wave takes one q, k or v head over kPrepTokens tokens; lane l holds channels 2 l + 128 i and the next.
template <typename T, int NI, int TAPS>
__global__ void __launch_bounds__(256) k_delta_prep(DeltaArgs a) {
  const DeltaShape &z = a.s;
  const int lane = threadIdx.x & 63, units = 2 * z.kv_heads + z.heads;
  const int64_t job = blockIdx.x * 4ll + (threadIdx.x >> 6);
  const int groups = (a.S + kPrepTokens - 1) / kPrepTokens;
  const int unit = (int)(job % units);
  const int64_t grp = job / units;
  if (grp >= (int64_t)a.B * groups) return;
  const int b = (int)(grp / groups), s0 = (int)(grp % groups) * kPrepTokens;
  const int pos0 = a.state->pos;
  const int64_t row0 = (int64_t)b * a.S + s0;
  const bool qk = unit < 2 * z.kv_heads, query = unit < z.kv_heads;
  const int width = qk ? z.Dk : z.Vp, h = qk ? (query ? unit : unit - z.kv_heads) : unit - 2 * z.kv_heads;
  const int first = qk ? unit * z.Dk : 2 * z.kv_heads * z.Dk + h * z.Vp;
  float2 y[NI][kPrepTokens];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = 2 * lane + 128 * i;
    if (c < width) conv_run<T, TAPS>(a, b, s0, pos0, first + c, y[i]);
    else {
#pragma unroll
      for (int t = 0; t < kPrepTokens; ++t) y[i][t] = make_float2(0.f, 0.f);
    }
  }
  if (!qk) {
#pragma unroll
    for (int t = 0; t < kPrepTokens; ++t)
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        const int c = 2 * lane + 128 * i;
        if (s0 + t < a.S && c < width) {
          Pair<T> o;
          Scalar<T>::store(&o.v[0], y[i][t].x);
          Scalar<T>::store(&o.v[1], y[i][t].y);
          *reinterpret_cast<Pair<T> *>((T *)a.v + ((row0 + t) * z.heads + h) * z.Vp + c) = o;
        }
      }
    return;
  }
  float sum[kPrepTokens];
#pragma unroll
  for (int t = 0; t < kPrepTokens; ++t) {
    sum[t] = 0.f;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const float u = as_stored<T>(y[i][t].x), w = as_stored<T>(y[i][t].y);
      sum[t] = fmaf(u, u, fmaf(w, w, sum[t]));
    }
  }
#pragma unroll
  for (int t = 0; t < kPrepTokens; ++t) sum[t] = wave_sum(sum[t]);
  T *dst = (T *)(query ? a.q : a.k) + h * z.Dk;
  const float mul = query ? 1.0f / sqrtf((float)z.dim) : 1.0f;
#pragma unroll
  for (int t = 0; t < kPrepTokens; ++t) {
    if (s0 + t >= a.S) break;
    if (lane == 0) (query ? a.qn : a.kn)[(row0 + t) * z.kv_heads + h] = mul / sqrtf(sum[t] + 1e-6f);
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = 2 * lane + 128 * i;
      Pair<T> o;
      Scalar<T>::store(&o.v[0], y[i][t].x);
      Scalar<T>::store(&o.v[1], y[i][t].y);
      if (c < width) *reinterpret_cast<Pair<T> *>(dst + (row0 + t) * z.kv_heads * z.Dk + c) = o;
    }
  }
}

// Sum over the `lanes` (a power of two) lanes that share a head.
__device__ __forceinline__ float group_sum(float v, int lanes) {
  if (lanes == 16) return row16_sum(v);
  for (int o = lanes >> 1; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}
__device__ __forceinline__ float fast_silu(float y) { return y * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * y)); }

// The bf16 form for four taps and key heads of 32, 64, 128, 256 or 512 channels: a thread takes eight channels over
// kWideTokens tokens, Dk / 8 neighbouring lanes a head.
constexpr int kWideTokens = 4;
__global__ void __launch_bounds__(256) k_delta_prep_wide(DeltaArgs a) {
  typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
  const DeltaShape &z = a.s;
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8, b = blockIdx.z, s0 = blockIdx.y * kWideTokens;
  const int kd = z.kv_heads * z.Dk;
  if (c >= z.channels) return;   // whole heads: channels is a multiple of 32, the q and k channels of 2 Dk
  const int pos0 = a.state->pos;
  u32x4 x[kWideTokens + 3], wv[4];
#pragma unroll
  for (int i = 0; i < kWideTokens + 3; ++i) {
    const int t = s0 - 3 + i;   // token of this call, or an earlier one in the ring
    x[i] = u32x4{0u, 0u, 0u, 0u};
    if (t >= 0 && t < a.S) x[i] = *reinterpret_cast<const u32x4 *>((const uint16_t *)a.dn + ((int64_t)b * a.S + t) * z.ldn + c);
    else if (t < 0 && pos0 + t >= 0) x[i] = *reinterpret_cast<const u32x4 *>((const uint16_t *)a.ring + ((int64_t)b * 4 + (pos0 + t) % 4) * z.channels + c);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) wv[i] = *reinterpret_cast<const u32x4 *>((const uint16_t *)a.conv + (int64_t)c * 4 + 8 * i);
  // one pair of channels after the other: its taps and rows unpacked, its results packed
  uint32_t o[kWideTokens][4];
  float sum[kWideTokens];
#pragma unroll
  for (int t = 0; t < kWideTokens; ++t) sum[t] = 0.f;
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    float w[2][4], lo[kWideTokens + 3], hi[kWideTokens + 3];
#pragma unroll
    for (int j = 0; j < 4; ++j) {   // channel 2 e + m: words 2 m, 2 m + 1 of wv[e]
      w[0][j] = __uint_as_float(j & 1 ? wv[e][j >> 1] & 0xffff0000u : wv[e][j >> 1] << 16);
      w[1][j] = __uint_as_float(j & 1 ? wv[e][2 + (j >> 1)] & 0xffff0000u : wv[e][2 + (j >> 1)] << 16);
    }
#pragma unroll
    for (int i = 0; i < kWideTokens + 3; ++i) {
      lo[i] = __uint_as_float(x[i][e] << 16);
      hi[i] = __uint_as_float(x[i][e] & 0xffff0000u);
    }
#pragma unroll
    for (int t = 0; t < kWideTokens; ++t) {
      float v0 = lo[t] * w[0][0], v1 = hi[t] * w[1][0];
#pragma unroll
      for (int j = 1; j < 4; ++j) {
        v0 = fmaf(lo[t + j], w[0][j], v0);
        v1 = fmaf(hi[t + j], w[1][j], v1);
      }
      o[t][e] = pack_bf16x2(fast_silu(v0), fast_silu(v1));
      const float u = __uint_as_float(o[t][e] << 16), p = __uint_as_float(o[t][e] & 0xffff0000u);
      sum[t] = fmaf(u, u, fmaf(p, p, sum[t]));
    }
  }
  const bool query = c < kd, key = !query && c < 2 * kd;
  const int Dk = z.Dk, unit = c / Dk;
  uint16_t *dst = query ? (uint16_t *)a.q + c : key ? (uint16_t *)a.k + c - kd : (uint16_t *)a.v + c - 2 * kd;
  const int64_t ldd = query || key ? kd : z.heads * z.Vp;
  const float mul = query ? 1.0f / sqrtf((float)z.dim) : 1.0f;
#pragma unroll
  for (int t = 0; t < kWideTokens; ++t) {
    const int64_t row = (int64_t)b * a.S + s0 + t;
    if (s0 + t < a.S) *reinterpret_cast<uint4 *>(dst + row * ldd) = make_uint4(o[t][0], o[t][1], o[t][2], o[t][3]);
    if (query || key) {
      const float total = group_sum(sum[t], Dk / 8);
      if (c % Dk == 0 && s0 + t < a.S) (query ? a.qn : a.kn)[row * z.kv_heads + (query ? unit : unit - z.kv_heads)] = mul / sqrtf(total + 1e-6f);
    }
  }
}

// A thread takes one channel of one head over a chunk of tokens; the head's first threads also form the step sizes.
constexpr int kDecayRun = 8;
template <typename T>
__global__ void __launch_bounds__(256) k_delta_decay(DeltaArgs a) {
  const DeltaShape &z = a.s;
  const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.z, s0 = blockIdx.y * kDeltaChunk;
  if (c >= z.heads * z.Dk) return;
  const int h = c / z.Dk, s1 = s0 + kDeltaChunk < a.S ? s0 + kDeltaChunk : a.S;
  const float rate = -expf(ld<T>(a.A_log, h)), bias = ld<T>(a.dt_bias, c);
  for (int s = s0; s < s1; s += kDecayRun) {
    float x[kDecayRun];
#pragma unroll
    for (int j = 0; j < kDecayRun; ++j) x[j] = s + j < s1 ? a.decay[((int64_t)b * a.S + s + j) * z.heads * z.Dk + c] : 0.f;
#pragma unroll
    for (int j = 0; j < kDecayRun; ++j)
      if (s + j < s1) {
        const float g = rate * softplus_for<T>(x[j] + bias);
        a.decay[((int64_t)b * a.S + s + j) * z.heads * z.Dk + c] = g;
      }
  }
  for (int s = s0 + c % z.Dk; s < s1; s += z.Dk) a.beta[((int64_t)b * a.S + s) * z.heads + h] = dl_sigmoid(ld<T>(a.dn, ((int64_t)b * a.S + s) * z.ldn + z.off_b + h));
}

// RPL state rows per lane (16 RPL >= Dk); rows past Dk stay zero.
constexpr int kScanTokens = 16;
template <typename T, int RPL>
__global__ void __launch_bounds__(256) k_delta_scan(DeltaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ds_lds[];
  constexpr int R = 16 * RPL;
  const DeltaShape &z = a.s;
  const int tid = threadIdx.x, sub = tid & 15, cl = tid >> 4;
  const int h = blockIdx.y, b = blockIdx.z, kv = h / (z.heads / z.kv_heads);
  const int c = blockIdx.x * 16 + cl;          // Vp is a multiple of 32
  float *qs = ds_lds, *ks = qs + kScanTokens * R, *gs = ks + kScanTokens * R, *vs = gs + kScanTokens * R, *bs = vs + kScanTokens * 16;
  const int pos0 = a.state->pos;
  float *st = a.carried + ((int64_t)b * z.heads + h) * z.Dk * z.Vp;
  float S[RPL];
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int r = sub * RPL + i;
    S[i] = pos0 > 0 && r < z.Dk ? st[(int64_t)r * z.Vp + c] : 0.f;
  }
  for (int s0 = 0; s0 < a.S; s0 += kScanTokens) {
    const int n = a.S - s0 < kScanTokens ? a.S - s0 : kScanTokens;
    const int64_t row0 = (int64_t)b * a.S + s0;
    __syncthreads();
    for (int e = tid; e < n * R; e += 256) {
      const int t = e / R, r = e - t * R;
      const bool in = r < z.Dk;
      const int64_t at = (row0 + t) * z.kv_heads + kv;
      qs[e] = in ? ld<T>(a.q, at * z.Dk + r) * a.qn[at] : 0.f;
      ks[e] = in ? ld<T>(a.k, at * z.Dk + r) * a.kn[at] : 0.f;
      gs[e] = in ? expf(a.decay[((row0 + t) * z.heads + h) * z.Dk + r]) : 0.f;
    }
    if (tid < n * 16) vs[tid] = ld<T>(a.v, ((row0 + (tid >> 4)) * z.heads + h) * z.Vp + blockIdx.x * 16 + (tid & 15));
    if (tid < n) bs[tid] = a.beta[(row0 + tid) * z.heads + h];
    __syncthreads();
    for (int t = 0; t < n; ++t) {
      const float *q = qs + t * R + sub * RPL, *k = ks + t * R + sub * RPL, *g = gs + t * R + sub * RPL;
      float kr[RPL], sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
      for (int i = 0; i < RPL; ++i) {
        kr[i] = k[i];
        const float qi = q[i];
        S[i] *= g[i];
        sk = fmaf(S[i], kr[i], sk);
        sq = fmaf(S[i], qi, sq);
        kq = fmaf(kr[i], qi, kq);
      }
      sk = row16_sum(sk);
      sq = row16_sum(sq);
      kq = row16_sum(kq);
      const float u = bs[t] * (vs[t * 16 + cl] - sk);
#pragma unroll
      for (int i = 0; i < RPL; ++i) S[i] = fmaf(kr[i], u, S[i]);
      if (sub == 0) a.o[((row0 + t) * z.heads + h) * z.Vp + c] = fmaf(kq, u, sq);
    }
  }
#pragma unroll
  for (int i = 0; i < RPL; ++i) {
    const int r = sub * RPL + i;
    if (r < z.Dk) st[(int64_t)r * z.Vp + c] = S[i];
  }
  if (blockIdx.x == 0) update_ring<T>(a, b, h, pos0, tid, 256);
}

// One wave per (row, head).
template <typename T, int NI>
__global__ void __launch_bounds__(256) k_delta_out(DeltaArgs a) {
  const DeltaShape &z = a.s;
  const int lane = threadIdx.x & 63;
  const int64_t job = blockIdx.x * 4ll + (threadIdx.x >> 6);
  if (job >= (int64_t)a.B * a.S * z.heads) return;
  const int h = (int)(job % z.heads);
  const int64_t row = job / z.heads;
  float o[NI], sum = 0.f;
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = lane + 64 * i;
    o[i] = c < z.vdim ? a.o[job * z.Vp + c] : 0.f;
    sum = fmaf(o[i], o[i], sum);
  }
  const float r = 1.0f / sqrtf(wave_sum(sum) / (float)z.vdim + a.eps);
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int c = lane + 64 * i;
    if (c < z.Vp) Scalar<T>::store((T *)a.out + row * a.ldo + h * z.Vp + c, o[i] * r * ld<T>(a.norm_w, c) * dl_sigmoid(ld<T>(a.gate, job * z.Vp + c)));
  }
}

// The bf16 form for value heads of a power of two: Vp / 8 neighbouring lanes a (row, head).
__global__ void __launch_bounds__(256) k_delta_out_wide(DeltaArgs a) {
  const DeltaShape &z = a.s;
  const int lanes = z.Vp / 8;
  const int64_t e = (blockIdx.x * 256ll + threadIdx.x) * 8, job = e / z.Vp;
  const int c = (int)(e - job * z.Vp);
  if (job >= (int64_t)a.B * a.S * z.heads) return;
  const int h = (int)(job % z.heads);
  const int64_t row = job / z.heads;
  const float4 o0 = *reinterpret_cast<const float4 *>(a.o + e), o1 = *reinterpret_cast<const float4 *>(a.o + e + 4);
  const uint4 gv = *reinterpret_cast<const uint4 *>((const uint16_t *)a.gate + e), wv = *reinterpret_cast<const uint4 *>((const uint16_t *)a.norm_w + c);
  float o[8] = {o0.x, o0.y, o0.z, o0.w, o1.x, o1.y, o1.z, o1.w}, sum = 0.f;
  const uint32_t g[4] = {gv.x, gv.y, gv.z, gv.w}, w[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
  for (int i = 0; i < 8; ++i) sum = fmaf(o[i], o[i], sum);   // padding columns hold zeros
  const float r = 1.0f / sqrtf(group_sum(sum, lanes) / (float)z.vdim + a.eps);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float gate = __uint_as_float(i & 1 ? g[i >> 1] & 0xffff0000u : g[i >> 1] << 16), wt = __uint_as_float(i & 1 ? w[i >> 1] & 0xffff0000u : w[i >> 1] << 16);
    o[i] *= r * wt * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * gate));
  }
  *reinterpret_cast<uint4 *>((uint16_t *)a.out + row * a.ldo + h * z.Vp + c) =
      make_uint4(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]), pack_bf16x2(o[4], o[5]), pack_bf16x2(o[6], o[7]));
}

// ---------------------------------------------------------------- one token per sequence
// Thread (column quad cq, row group rg) holds rows rg, rg + RG, ... of four columns: NI of them, requested before
// anything is computed.  Both sums over the state's rows are formed from the decayed state before the write,
//   S^T q after the write = (g S)^T q + (k . q) u,
// so one exchange through LDS serves v's correction and the read-out.
constexpr int kStepThreads = 512;
template <typename T> __device__ __forceinline__ float factor_row(const T *w, const T *x, int rank, int part) {
  constexpr int V = 16 / sizeof(T);
  struct alignas(16) Pack { T v[V]; };
  float acc = 0.f;
  for (int k = part * V; k < rank; k += 4 * V) {
    const Pack p = *reinterpret_cast<const Pack *>(w + k), y = *reinterpret_cast<const Pack *>(x + k);
#pragma unroll
    for (int e = 0; e < V; ++e) acc = fmaf((float)Scalar<T>::load(&p.v[e]), (float)Scalar<T>::load(&y.v[e]), acc);
  }
  acc += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(acc), 0xB1, 0xf, 0xf, true));
  acc += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(acc), 0x4E, 0xf, 0xf, true));
  return acc;
}

template <typename T, int NI, bool FACTORS>
__global__ void __launch_bounds__(kStepThreads) k_delta_step(DeltaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float st_lds[];
  const DeltaShape &z = a.s;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.x, b = blockIdx.y, rep = z.heads / z.kv_heads, kv = h / rep, kd = z.kv_heads * z.Dk;
  const int CQ = z.Vp / 4, RG = kStepThreads / CQ, cq = tid % CQ, rg = tid / CQ;
  float *qs = st_lds, *ks = qs + z.Dk, *gs = ks + z.Dk, *vs = gs + z.Dk, *zs = vs + z.Vp, *us = zs + z.Vp, *red = us + z.Vp;   // red[2][RG][Vp]
  __shared__ float sums[4], part[kStepThreads / 64];
  const int pos0 = a.state->pos;
  float *st = a.carried + ((int64_t)b * z.heads + h) * z.Dk * z.Vp;
  float4 S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int r = rg + i * RG;
    S[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (rg < RG && r < z.Dk && pos0 > 0) S[i] = *reinterpret_cast<const float4 *>(st + (int64_t)r * z.Vp + cq * 4);
  }
  // ---- convolutions; the ring's free place takes this token's inputs
  for (int i = tid; i < 2 * z.Dk + z.Vp; i += kStepThreads) {
    const int c = i < z.Dk ? kv * z.Dk + i : i < 2 * z.Dk ? kd + kv * z.Dk + i - z.Dk : 2 * kd + h * z.Vp + i - 2 * z.Dk;
    (i < 2 * z.Dk ? qs : vs - 2 * z.Dk)[i] = conv_silu<T>(a, b, 0, pos0, c);   // ks follows qs
    if (i >= 2 * z.Dk || h % rep == 0) ((T *)a.ring)[((int64_t)b * z.taps + pos0 % z.taps) * z.channels + c] = ((const T *)a.dn)[b * z.ldn + c];
  }
  // ---- decays and gate
  const float rate = -expf(ld<T>(a.A_log, h));
  if constexpr (FACTORS) {
    const T *a1 = (const T *)a.dn + b * z.ldn + z.off_a1, *g1 = (const T *)a.dn + b * z.ldn + z.off_g1;
    for (int r = tid >> 2; r < z.Dk + z.Vp; r += kStepThreads / 4) {
      const bool dec = r < z.Dk;
      const int n = dec ? h * z.Dk + r : h * z.Vp + r - z.Dk;
      const float y = dec ? factor_row<T>((const T *)a.a2 + (int64_t)n * a.a_rank, a1, a.a_rank, tid & 3)
                          : factor_row<T>((const T *)a.g2 + (int64_t)n * a.g_rank, g1, a.g_rank, tid & 3);
      if ((tid & 3) == 0) {
        if (dec) gs[r] = expf(rate * dl_softplus(y + ld<T>(a.dt_bias, n)));
        else zs[r - z.Dk] = dl_sigmoid(y);
      }
    }
  } else {
    for (int r = tid; r < z.Dk; r += kStepThreads)
      gs[r] = expf(rate * dl_softplus(a.decay[((int64_t)b * z.heads + h) * z.Dk + r] + ld<T>(a.dt_bias, h * z.Dk + r)));
    for (int c = tid; c < z.Vp; c += kStepThreads) zs[c] = dl_sigmoid(ld<T>(a.gate, ((int64_t)b * z.heads + h) * z.Vp + c));
  }
  const float beta = dl_sigmoid(ld<T>(a.dn, b * z.ldn + z.off_b + h));
  __syncthreads();
  if (wave < 3) {   // |q|^2, |k|^2, k . q
    const float *x = wave == 0 ? qs : ks, *y = wave == 1 ? ks : qs;
    float s = 0.f;
    for (int r = lane; r < z.Dk; r += 64) s = fmaf(x[r], y[r], s);
    s = wave_sum(s);
    if (lane == 0) sums[wave] = s;
  }
  float sk[4] = {0.f, 0.f, 0.f, 0.f}, sq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int r = rg + i * RG;
    if (rg < RG && r < z.Dk) {
      const float g = gs[r], k = ks[r], q = qs[r];
      S[i].x *= g; S[i].y *= g; S[i].z *= g; S[i].w *= g;
      sk[0] = fmaf(S[i].x, k, sk[0]); sk[1] = fmaf(S[i].y, k, sk[1]); sk[2] = fmaf(S[i].z, k, sk[2]); sk[3] = fmaf(S[i].w, k, sk[3]);
      sq[0] = fmaf(S[i].x, q, sq[0]); sq[1] = fmaf(S[i].y, q, sq[1]); sq[2] = fmaf(S[i].z, q, sq[2]); sq[3] = fmaf(S[i].w, q, sq[3]);
    }
  }
  if (rg < RG) {
    *reinterpret_cast<float4 *>(red + rg * z.Vp + cq * 4) = make_float4(sk[0], sk[1], sk[2], sk[3]);
    *reinterpret_cast<float4 *>(red + (RG + rg) * z.Vp + cq * 4) = make_float4(sq[0], sq[1], sq[2], sq[3]);
  }
  __syncthreads();
  const float rk = 1.0f / sqrtf(sums[1] + 1e-6f), rq = 1.0f / sqrtf(sums[0] + 1e-6f) / sqrtf((float)z.dim);
  float o = 0.f;
  if (tid < z.Vp) {
    float x = 0.f, y = 0.f;
    for (int g = 0; g < RG; ++g) {
      x += red[g * z.Vp + tid];
      y += red[(RG + g) * z.Vp + tid];
    }
    const float u = beta * (vs[tid] - rk * x);
    us[tid] = u * rk;                                // what a row of the raw k is multiplied with
    o = fmaf(sums[2] * rk * rq, u, rq * y);
  }
  const float s2 = wave_sum(tid < z.vdim ? o * o : 0.f);
  if (lane == 0) part[wave] = s2;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NI; ++i) {
    const int r = rg + i * RG;
    if (rg < RG && r < z.Dk) {
      const float k = ks[r];
      const float4 u = *reinterpret_cast<const float4 *>(us + cq * 4);
      S[i].x = fmaf(k, u.x, S[i].x); S[i].y = fmaf(k, u.y, S[i].y); S[i].z = fmaf(k, u.z, S[i].z); S[i].w = fmaf(k, u.w, S[i].w);
      *reinterpret_cast<float4 *>(st + (int64_t)r * z.Vp + cq * 4) = S[i];
    }
  }
  if (tid < z.Vp) {
    float t = 0.f;
    for (int w = 0; w < kStepThreads / 64; ++w) t += part[w];
    const float r = 1.0f / sqrtf(t / (float)z.vdim + a.eps);
    Scalar<T>::store((T *)a.out + b * a.ldo + h * z.Vp + tid, o * r * ld<T>(a.norm_w, tid) * zs[tid]);
  }
}

// ---------------------------------------------------------------- launchers
static int check_delta(const DeltaArgs &a) {
  const DeltaShape &z = a.s;
  RAI_REQUIRE(z.heads > 0 && z.kv_heads > 0 && z.heads % z.kv_heads == 0 && z.taps > 0 && z.Dk % 32 == 0 && z.Vp % 32 == 0 && z.dim <= z.Dk && z.vdim <= z.Vp &&
                  z.Dk <= kDeltaMaxHead && z.Vp <= kDeltaMaxHead && z.channels == 2 * z.kv_heads * z.Dk + z.heads * z.Vp,
              RAI_ERR_BAD_SHAPE, "delta rule: %d / %d heads of %d x %d", z.heads, z.kv_heads, z.dim, z.vdim);
  RAI_REQUIRE(a.B > 0 && a.S > 0 && a.B <= 65535 && z.heads <= 65535, RAI_ERR_UNSUPPORTED, "delta rule: %d sequences of %d heads", a.B, z.heads);
  return RAI_OK;
}

template <typename T, int RPL> static int launch_scan(hipStream_t st, const DeltaArgs &a) {
  const size_t lds = (size_t)kScanTokens * (3 * 16 * RPL + 16 + 1) * sizeof(float);
  static bool attr_set = false;
  if (lds > 64 * 1024 && !attr_set) {
    RAI_HIP_TRY(hipFuncSetAttribute((const void *)k_delta_scan<T, RPL>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    attr_set = true;
  }
  hipLaunchKernelGGL((k_delta_scan<T, RPL>), dim3(a.s.Vp / 16, a.s.heads, a.B), dim3(256), lds, st, a);
  return launch_check("delta_scan");
}

template <typename T, int NI> static int launch_prep(hipStream_t st, const DeltaArgs &a) {
  const DeltaShape &z = a.s;
  const int64_t jobs = (int64_t)a.B * ((a.S + kPrepTokens - 1) / kPrepTokens) * (2 * z.kv_heads + z.heads);
  RAI_REQUIRE((jobs + 3) / 4 < (1ll << 31), RAI_ERR_UNSUPPORTED, "delta rule: too many tokens");
  const dim3 grid((unsigned)((jobs + 3) / 4)), block(256);
  if (z.taps == 4) hipLaunchKernelGGL((k_delta_prep<T, NI, 4>), grid, block, 0, st, a);
  else hipLaunchKernelGGL((k_delta_prep<T, NI, 0>), grid, block, 0, st, a);
  return launch_check("delta_prep");
}

template <typename T> static int launch_tokens_t(hipStream_t st, int dtype, const DeltaArgs &a) {
  const DeltaShape &z = a.s;
  const int wide = z.Dk > z.Vp ? z.Dk : z.Vp;
  const char *off = getenv("RAI_HIP_NO_DELTA_CHUNK");   // read per call: the tests compare both forms in one process
  const bool chunked = a.chunk_ws && a.S >= kChunkedFrom && delta_chunk_serves(dtype, z) && !(off && *off && *off != '0');
  const int64_t outs = (int64_t)a.B * a.S * z.heads;
  RAI_REQUIRE((outs + 3) / 4 < (1ll << 31) && (a.S + kDeltaChunk - 1) / kDeltaChunk <= 65535, RAI_ERR_UNSUPPORTED, "delta rule: too many tokens");
  const dim3 go((unsigned)((outs + 3) / 4)), block(256);
  auto pow2 = [](int n) { return (n & (n - 1)) == 0; };
  const bool wide_prep = sizeof(T) == 2 && z.taps == 4 && pow2(z.Dk) && (a.S + kWideTokens - 1) / kWideTokens <= 65535;
  if (wide_prep) {
    hipLaunchKernelGGL(k_delta_prep_wide, dim3((z.channels / 8 + 255) / 256, (a.S + kWideTokens - 1) / kWideTokens, a.B), block, 0, st, a);
    RAI_TRY(launch_check("delta_prep_wide"));
  } else if (wide <= 128) RAI_TRY((launch_prep<T, 1>(st, a)));
  else if (wide <= 256) RAI_TRY((launch_prep<T, 2>(st, a)));
  else RAI_TRY((launch_prep<T, 4>(st, a)));
  if (chunked) {
    RAI_TRY(launch_delta_chunks(st, a));
  } else {
    hipLaunchKernelGGL(k_delta_decay<T>, dim3((z.heads * z.Dk + 255) / 256, (a.S + kDeltaChunk - 1) / kDeltaChunk, a.B), block, 0, st, a);
    RAI_TRY(launch_check("delta_decay"));
    if (z.Dk <= 32) RAI_TRY((launch_scan<T, 2>(st, a)));
    else if (z.Dk <= 64) RAI_TRY((launch_scan<T, 4>(st, a)));
    else if (z.Dk <= 128) RAI_TRY((launch_scan<T, 8>(st, a)));
    else if (z.Dk <= 256) RAI_TRY((launch_scan<T, 16>(st, a)));
    else RAI_TRY((launch_scan<T, 32>(st, a)));
  }
  if (sizeof(T) == 2 && pow2(z.Vp) && a.ldo % 8 == 0) {
    hipLaunchKernelGGL(k_delta_out_wide, dim3((unsigned)((outs * (z.Vp / 8) + 255) / 256)), block, 0, st, a);
    return launch_check("delta_out_wide");
  }
  if (z.Vp <= 64) hipLaunchKernelGGL((k_delta_out<T, 1>), go, block, 0, st, a);
  else if (z.Vp <= 128) hipLaunchKernelGGL((k_delta_out<T, 2>), go, block, 0, st, a);
  else if (z.Vp <= 256) hipLaunchKernelGGL((k_delta_out<T, 4>), go, block, 0, st, a);
  else hipLaunchKernelGGL((k_delta_out<T, 8>), go, block, 0, st, a);
  return launch_check("delta_out");
}

int launch_delta_tokens(hipStream_t st, int dtype, const DeltaArgs &a) {
  RAI_TRY(check_delta(a));
  return dtype == RAI_BF16 ? launch_tokens_t<bf16_raw>(st, dtype, a) : launch_tokens_t<float>(st, dtype, a);
}

static int step_rows(const DeltaShape &z) {   // state rows per thread
  const int RG = kStepThreads / (z.Vp / 4);
  return (z.Dk + RG - 1) / RG;
}
bool delta_step_serves(const DeltaShape &z) {
  return z.Dk % 32 == 0 && z.Vp % 32 == 0 && z.Dk <= kDeltaMaxHead && z.Vp <= kDeltaMaxHead && step_rows(z) <= 32;
}

template <typename T, int NI> static int launch_step_n(hipStream_t st, const DeltaArgs &a) {
  const DeltaShape &z = a.s;
  const int RG = kStepThreads / (z.Vp / 4);
  const size_t lds = (size_t)(3 * z.Dk + 3 * z.Vp + 2 * RG * z.Vp) * sizeof(float);   // at most 28 KB
  const dim3 grid(z.heads, a.B), block(kStepThreads);
  if (a.a2) hipLaunchKernelGGL((k_delta_step<T, NI, true>), grid, block, lds, st, a);
  else hipLaunchKernelGGL((k_delta_step<T, NI, false>), grid, block, lds, st, a);
  return launch_check("delta_step");
}
template <typename T> static int launch_step_t(hipStream_t st, const DeltaArgs &a) {
  const int n = step_rows(a.s);
  if (n <= 2) return launch_step_n<T, 2>(st, a);
  if (n <= 4) return launch_step_n<T, 4>(st, a);
  if (n <= 8) return launch_step_n<T, 8>(st, a);
  if (n <= 16) return launch_step_n<T, 16>(st, a);
  return launch_step_n<T, 32>(st, a);
}
int launch_delta_step(hipStream_t st, int dtype, const DeltaArgs &a) {
  RAI_TRY(check_delta(a));
  RAI_REQUIRE(a.S == 1 && delta_step_serves(a.s) && (a.a2 == nullptr) == (a.g2 == nullptr) && (!a.a2 || (a.a_rank % 8 == 0 && a.g_rank % 8 == 0)),
              RAI_ERR_BAD_ARG, "delta step: not served");
  return dtype == RAI_BF16 ? launch_step_t<bf16_raw>(st, a) : launch_step_t<float>(st, a);
}

}  // namespace rai
