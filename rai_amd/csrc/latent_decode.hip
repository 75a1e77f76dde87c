// The single-row step of a latent-attention decoder in bf16: the Linears of a layer in three launches around the
// absorbed attention (latent_attention.hip), each with what precedes it folded in.
//   k_latent_in    both norms of the f32 stream + [query latent | latent | gate] from the first, and from the second the
//                  gated MLP or the router; also the final norm + head
//   k_latent_mid   norm of the query latent + queries; norm of the latent + cache append; choice of the experts + the
//                  chosen experts' gated products on the scaled input
//   k_latent_down  o and down (or the chosen experts' downs) as one contraction per stream element, residual added in f32
// A wave streams R weight rows at a time with the activation vector in registers (as k_gemv_bf16_reg does), lane l
// holding positions l * 8 + 512 u; every wave prepares its activation vector itself while its first weights fly.
#include <cstdlib>

#include "latent.h"
#include "moe.h"

namespace rai {

typedef __attribute__((ext_vector_type(2))) __bf16 ld_bf16x2;
typedef __attribute__((ext_vector_type(4))) uint32_t ld_u32x4;
typedef __attribute__((ext_vector_type(4))) float ld_f32x4;

__device__ __forceinline__ float ld_dot8(ld_u32x4 a, ld_u32x4 b, float c) {
  // elements named one by one: see dot2_bf16 in gemm.hip
  auto dot2 = [](uint32_t x, uint32_t y, float z) {
    ld_bf16x2 p, q;
    __builtin_memcpy(&p, &x, 4);
    __builtin_memcpy(&q, &y, 4);
    return __builtin_amdgcn_fdot2_f32_bf16(p, q, z, false);
  };
  c = dot2(a.x, b.x, c);
  c = dot2(a.y, b.y, c);
  c = dot2(a.z, b.z, c);
  return dot2(a.w, b.w, c);
}
__device__ __forceinline__ float lo_f32(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float hi_f32(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }
__device__ __forceinline__ float gated(int act, float g, float u) { return act_eval(act, g) * u; }
__device__ __forceinline__ float gated(const LatentInArgs &a, float g, float u) {
  return a.act == kActClampedGlu ? glu_clamped_bf16_out(g, u, a.act_limit, a.act_alpha) : gated(a.act, g, u);
}

// R rows of W in flight, rows n .. n + R - 1 clamped to n_last.
template <int KC, int R> struct RowSet {
  ld_u32x4 w[R][KC];
  __device__ __forceinline__ void load(const uint16_t *W, int64_t ldw, int n, int n_last, int K, int lane) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const uint16_t *p = W + (int64_t)(n + r < n_last ? n + r : n_last) * ldw + lane * 8;
#pragma unroll
      for (int u = 0; u < KC; ++u)
        w[r][u] = lane * 8 + u * 512 < K ? __builtin_nontemporal_load(reinterpret_cast<const ld_u32x4 *>(p + u * 512)) : ld_u32x4{0u, 0u, 0u, 0u};
    }
  }
};

// Rows [n0, n1) against the activation vector x, R at a time, the next set requested before the current one's sums are
// reduced; store(n, value of row n, value of row n + 1 or 0) runs on lane 0 for the first row of each pair (R == 2).
template <int KC, typename Store>
__device__ __forceinline__ void stream_rows(RowSet<KC, 2> &rs, const ld_u32x4 (&x)[KC], const uint16_t *W, int64_t ldw, int n0, int n1, int K,
                                            int lane, Store store) {
  for (int n = n0; n < n1; n += 2) {
    float a0 = 0.f, a1 = 0.f;
#pragma unroll
    for (int u = 0; u < KC; ++u) {
      a0 = ld_dot8(rs.w[0][u], x[u], a0);
      a1 = ld_dot8(rs.w[1][u], x[u], a1);
    }
    if (n + 2 < n1) rs.load(W, ldw, n + 2, n1 - 1, K, lane);
    a0 = wave_sum(a0);
    a1 = wave_sum(a1);
    if (lane == 0) store(n, a0, a1);
  }
}

template <int KC>
__global__ void __launch_bounds__(256) k_latent_in(LatentInArgs a) {
  const int lane = threadIdx.x & 63;
  int gw = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6));
  const bool second = gw >= a.waves1;
  if (second) gw -= a.waves1;
  const int N = second ? a.N2 : a.N1;
  const int n0 = gw * a.rows_per_wave, n1 = n0 + a.rows_per_wave < N ? n0 + a.rows_per_wave : N;
  if (n0 >= N) return;
  const uint16_t *W = (const uint16_t *)(second ? a.W2 : a.W1), *nw = (const uint16_t *)(second ? a.n2 : a.n1) + lane * 8;
  // the small, L2-resident vectors first (loads return in order), then the first weights
  float x[KC][8];
  ld_u32x4 wn[KC];
#pragma unroll
  for (int u = 0; u < KC; ++u) {
    const int k = lane * 8 + u * 512;
    wn[u] = ld_u32x4{0u, 0u, 0u, 0u};
#pragma unroll
    for (int e = 0; e < 8; ++e) x[u][e] = 0.f;
    if (k < a.H) {
      if (a.kind != kStreamCopy) wn[u] = *reinterpret_cast<const ld_u32x4 *>(nw + u * 512);
      if (a.src_f32) {
        const ld_f32x4 v0 = *reinterpret_cast<const ld_f32x4 *>((const float *)a.src + k), v1 = *reinterpret_cast<const ld_f32x4 *>((const float *)a.src + k + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) { x[u][e] = v0[e]; x[u][4 + e] = v1[e]; }
      } else {
        const ld_u32x4 v = *reinterpret_cast<const ld_u32x4 *>((const uint16_t *)a.src + k);
#pragma unroll
        for (int e = 0; e < 4; ++e) { x[u][2 * e] = lo_f32(v[e]); x[u][2 * e + 1] = hi_f32(v[e]); }
      }
    }
  }
  RowSet<KC, 2> rs;
  rs.load(W, a.ldw, n0, n1 - 1, a.K, lane);
  if (a.src_scale != 0.f) {
#pragma unroll
    for (int u = 0; u < KC; ++u)
#pragma unroll
      for (int e = 0; e < 8; ++e) x[u][e] *= a.src_scale;
  }
  if (a.kind == kStreamLayerNorm) {
    float s = 0.f;
#pragma unroll
    for (int u = 0; u < KC; ++u)
#pragma unroll
      for (int e = 0; e < 8; ++e) s += x[u][e];
    const float mean = wave_sum(s) / (float)a.H;
#pragma unroll
    for (int u = 0; u < KC; ++u)
#pragma unroll
      for (int e = 0; e < 8; ++e) x[u][e] = lane * 8 + u * 512 < a.H ? x[u][e] - mean : 0.f;
  }
  const int gsize = a.H / a.groups;
  const float h_scale = a.h_scale != 0.f ? a.h_scale : 1.0f;
  float q[KC], sc[KC];
  int grp[KC];
#pragma unroll
  for (int u = 0; u < KC; ++u) {
    q[u] = sc[u] = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) q[u] = fmaf(x[u][e], x[u][e], q[u]);
    grp[u] = (lane * 8 + u * 512) / gsize;
  }
  for (int g = 0; g < a.groups; ++g) {
    float s = 0.f;
#pragma unroll
    for (int u = 0; u < KC; ++u) s += grp[u] == g ? q[u] : 0.f;
    s = h_scale / sqrtf(wave_sum(s) / (float)gsize + a.eps);
#pragma unroll
    for (int u = 0; u < KC; ++u) sc[u] = grp[u] == g ? s : sc[u];
  }
  ld_u32x4 xv[KC];
  if (a.kind == kStreamCopy) {
#pragma unroll
    for (int u = 0; u < KC; ++u) {
      sc[u] = h_scale;
      wn[u] = ld_u32x4{0x3f803f80u, 0x3f803f80u, 0x3f803f80u, 0x3f803f80u};   // ones
    }
  }
#pragma unroll
  for (int u = 0; u < KC; ++u)
#pragma unroll
    for (int e = 0; e < 4; ++e) xv[u][e] = pack_bf16x2(x[u][2 * e] * sc[u] * lo_f32(wn[u][e]), x[u][2 * e + 1] * sc[u] * hi_f32(wn[u][e]));
  if (second && a.h2 && n0 == 0) {
#pragma unroll
    for (int u = 0; u < KC; ++u)
      if (lane * 8 + u * 512 < a.K) *reinterpret_cast<ld_u32x4 *>((uint16_t *)a.h2 + lane * 8 + u * 512) = xv[u];
  }
  stream_rows<KC>(rs, xv, W, a.ldw, n0, n1, a.K, lane, [&](int n, float v0, float v1) {
    if (!second) {
      uint16_t *o = (uint16_t *)a.out1 + n;
      o[0] = f32_to_bf16_bits(v0);
      if (n + 1 < n1) o[1] = f32_to_bf16_bits(v1);
    } else if (a.gated2) {
      ((uint16_t *)a.out2)[n >> 1] = f32_to_bf16_bits(gated(a, v0, v1));
    } else {
      float *o = (float *)a.out2 + n;
      if (a.add2) { v0 += a.add2[n]; if (n + 1 < n1) v1 += a.add2[n + 1]; }
      if (a.bias2) { v0 += bf16_bits_to_f32(((const uint16_t *)a.bias2)[n]); if (n + 1 < n1) v1 += bf16_bits_to_f32(((const uint16_t *)a.bias2)[n + 1]); }
      o[0] = v0;
      if (n + 1 < n1) o[1] = v1;
    }
  });
}

// The expert of rank j among the logits, and its score (the choice of k_moe_route_ranked).
template <int N> __device__ __forceinline__ int nth_of(const float *z, int experts, int j, int lane, float *score) {
  float v[N];
  int rank[N], e = 0;
  float zj = 0.f;
  rank_experts<N>(z, experts, lane, v, rank);
#pragma unroll
  for (int i = 0; i < N; ++i) {
    const unsigned long long hit = __ballot(rank[i] == j);
    if (hit) {   // exactly one lane of one i
      const int l = __ffsll(hit) - 1;
      e = 64 * i + l;
      zj = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v[i]), l));
    }
  }
  *score = router_score(zj);
  return __builtin_amdgcn_readfirstlane(e);
}
__device__ __forceinline__ int nth_expert(const float *z, int experts, int j, int lane, float *score) {
  if (experts <= 64) return nth_of<1>(z, experts, j, lane, score);
  if (experts <= 128) return nth_of<2>(z, experts, j, lane, score);
  return nth_of<4>(z, experts, j, lane, score);
}

// Gated rows [n0, n1) of one expert on score * h, to out[n / 2].
template <int KC>
__device__ __forceinline__ void expert_rows(const uint16_t *h, const uint16_t *W, int K, int n0, int n1, float score, int act, uint16_t *out, int lane) {
  ld_u32x4 xv[KC];
#pragma unroll
  for (int u = 0; u < KC; ++u)
    xv[u] = lane * 8 + u * 512 < K ? *reinterpret_cast<const ld_u32x4 *>(h + lane * 8 + u * 512) : ld_u32x4{0u, 0u, 0u, 0u};
  RowSet<KC, 2> rs;
  rs.load(W, K, n0, n1 - 1, K, lane);
#pragma unroll
  for (int u = 0; u < KC; ++u)
#pragma unroll
    for (int i = 0; i < 4; ++i) xv[u][i] = pack_bf16x2(score * lo_f32(xv[u][i]), score * hi_f32(xv[u][i]));
  stream_rows<KC>(rs, xv, W, K, n0, n1, K, lane, [&](int n, float v0, float v1) { out[n >> 1] = f32_to_bf16_bits(gated(act, v0, v1)); });
}

// Few rows: every (token, choice) slot is a product of its own, the expert's weights shared through the caches where two
// tokens chose it.
template <int KC>
__global__ void __launch_bounds__(256) k_moe_slots(MoeSlotsArgs a) {
  const int lane = threadIdx.x & 63;
  const int gw = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6));
  const int slot = gw / a.waves_e, n0 = (gw - slot * a.waves_e) * a.rows_per_wave, N = 2 * a.EFp;
  if (slot >= a.slots) return;
  const int n1 = n0 + a.rows_per_wave < N ? n0 + a.rows_per_wave : N;
  expert_rows<KC>((const uint16_t *)a.h + (int64_t)(slot / a.top) * a.ld, (const uint16_t *)a.We_gu + (int64_t)a.choice[slot] * a.gu_stride, a.Hp, n0, n1,
                  a.weight[slot], a.act, (uint16_t *)a.eact + (int64_t)slot * a.EFp, lane);
}

template <int KC>
__global__ void __launch_bounds__(256) k_latent_mid(LatentMidArgs a) {
  const int lane = threadIdx.x & 63;
  int gw = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6));
  const int total = a.waves_q + a.top * a.waves_e;
  if (gw > total) return;
  ld_u32x4 xv[KC];
  if (gw == total || gw < a.waves_q) {
    // one of the two latents, normalised: the last wave appends the cached one, the others take the query's
    const bool append = gw == total;
    const int n = append ? a.kv_rank : a.q_rank;
    const uint16_t *src = (const uint16_t *)a.dn + (append ? a.Qp : 0), *w = (const uint16_t *)(append ? a.c_w : a.q_w);
    ld_u32x4 wn[KC];
#pragma unroll
    for (int u = 0; u < KC; ++u) {
      const int k = lane * 8 + u * 512;
      xv[u] = wn[u] = ld_u32x4{0u, 0u, 0u, 0u};
      if (k < n) {   // ranks that are not multiples of 8 end inside a pack: the padding of dn is zero, the norm's guarded
        xv[u] = *reinterpret_cast<const ld_u32x4 *>(src + k);
        if (k + 8 <= n) wn[u] = *reinterpret_cast<const ld_u32x4 *>(w + k);
        else {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (k + e < n) wn[u][e >> 1] |= (uint32_t)w[k + e] << (16 * (e & 1));
        }
      }
    }
    RowSet<KC, 2> rs;
    const int n0 = gw * a.rows_per_wave, n1 = n0 + a.rows_per_wave < a.Nq ? n0 + a.rows_per_wave : a.Nq;
    if (!append) rs.load((const uint16_t *)a.Wuq, a.Qp, n0, n1 - 1, a.Qp, lane);
    float q = 0.f;
#pragma unroll
    for (int u = 0; u < KC; ++u) q = ld_dot8(xv[u], xv[u], q);
    const float sc = 1.0f / sqrtf(wave_sum(q) / (float)n + a.eps);
#pragma unroll
    for (int u = 0; u < KC; ++u)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        xv[u][e] = pack_bf16x2(lo_f32(xv[u][e]) * sc * lo_f32(wn[u][e]), hi_f32(xv[u][e]) * sc * hi_f32(wn[u][e]));
    if (append) {
      uint16_t *dst = (uint16_t *)a.cache + (int64_t)a.state->pos * a.Rp;
#pragma unroll
      for (int u = 0; u < KC; ++u)
        if (lane * 8 + u * 512 < a.Rp) *reinterpret_cast<ld_u32x4 *>(dst + lane * 8 + u * 512) = xv[u];
      return;
    }
    stream_rows<KC>(rs, xv, (const uint16_t *)a.Wuq, a.Qp, n0, n1, a.Qp, lane, [&](int nn, float v0, float v1) {
      uint16_t *o = (uint16_t *)a.q + nn;
      o[0] = f32_to_bf16_bits(v0);
      if (nn + 1 < n1) o[1] = f32_to_bf16_bits(v1);
    });
    return;
  }
  gw -= a.waves_q;
  const int slot = gw / a.waves_e, n0 = (gw - slot * a.waves_e) * a.rows_per_wave, N = 2 * a.EFp;
  const int n1 = n0 + a.rows_per_wave < N ? n0 + a.rows_per_wave : N;
  float score;
  const int e = nth_expert(a.rlogits, a.experts, slot, lane, &score);
  if (n0 == 0 && lane == 0) a.choice[slot] = e;
  expert_rows<KC>((const uint16_t *)a.h2, (const uint16_t *)a.We_gu + (int64_t)e * a.gu_stride, a.Hp, n0, n1, score, a.act,
                  (uint16_t *)a.eact + (int64_t)slot * a.EFp, lane);
}

// Chunks of up to 512 columns of the concatenated contraction: where the weights of row 0 are, the row stride, where the
// activations sit in LDS and how many columns there are.
struct DownChunk {
  const uint16_t *w;
  int ld;
  int meta;   // LDS offset | columns << 20
};

// A block of eight waves shares one copy of the activations; a wave owns one output row and has Q chunks in flight, each
// replaced by the chunk Q places on as soon as it has been multiplied.
constexpr int kDownWaves = 8, kDownThreads = kDownWaves * 64;
template <int Q>
__global__ void __launch_bounds__(kDownThreads) k_latent_down(LatentDownArgs a) {
  extern __shared__ __attribute__((aligned(16))) char dn_lds[];
  const int tid = threadIdx.x, lane = tid & 63;
  {   // this block's row
    const int64_t m = blockIdx.y;
    a.x0 = (const uint16_t *)a.x0 + m * a.K0;
    a.x1 = (const uint16_t *)a.x1 + m * a.top * a.K1;
    if (a.top) a.choice += m * a.top;
    a.res = a.res_f32 ? (const void *)((const float *)a.res + m * a.N) : (const void *)((const uint16_t *)a.res + m * a.H);
    a.out += m * a.N;
  }
  const int c0 = (a.K0 + 511) / 512, c1 = (a.K1 + 511) / 512, chunks = c0 + a.top * c1;
  const int Kt = a.K0 + a.top * a.K1;
  DownChunk *table = reinterpret_cast<DownChunk *>(dn_lds);
  uint16_t *xs = reinterpret_cast<uint16_t *>(table + chunks);
  const int n = blockIdx.x * kDownWaves + (tid >> 6);
  float res = 0.f;
  if (n < a.H) res = a.res_f32 ? ((const float *)a.res)[n] : bf16_bits_to_f32(((const uint16_t *)a.res)[n]);
  if (a.res_scale != 0.f) res *= a.res_scale;
  for (int c = tid; c < chunks; c += kDownThreads) {
    DownChunk d;
    if (c < c0) {
      d.w = (const uint16_t *)a.W0 + c * 512;
      d.ld = a.K0;
      d.meta = (c * 512) | ((a.K0 - c * 512 < 512 ? a.K0 - c * 512 : 512) << 20);
    } else {
      const int j = (c - c0) / c1, i = (c - c0) - j * c1;
      d.w = (const uint16_t *)a.W1 + (int64_t)a.choice[j] * a.stride1 + i * 512;
      d.ld = a.K1;
      d.meta = (a.K0 + j * a.K1 + i * 512) | ((a.K1 - i * 512 < 512 ? a.K1 - i * 512 : 512) << 20);
    }
    table[c] = d;
  }
  __syncthreads();
  ld_u32x4 w[Q];
  auto request = [&](ld_u32x4 &dst, int c) {
    if (c < chunks) {
      const DownChunk d = table[c];
      if (lane * 8 < (d.meta >> 20) && n < a.N) dst = __builtin_nontemporal_load(reinterpret_cast<const ld_u32x4 *>(d.w + (int64_t)n * d.ld + lane * 8));
    }
  };
  // the activations come from the L2 and are asked for first; they reach LDS while the weights are on their way
  constexpr int XP = 3;
  ld_u32x4 xp[XP];
  auto x_at = [&](int k) { return *reinterpret_cast<const ld_u32x4 *>(k < a.K0 ? (const uint16_t *)a.x0 + k : (const uint16_t *)a.x1 + (k - a.K0)); };
#pragma unroll
  for (int i = 0; i < XP; ++i)
    if ((tid + i * kDownThreads) * 8 < Kt) xp[i] = x_at((tid + i * kDownThreads) * 8);
#pragma unroll
  for (int u = 0; u < Q; ++u) {
    w[u] = ld_u32x4{0u, 0u, 0u, 0u};
    request(w[u], u);
  }
#pragma unroll
  for (int i = 0; i < XP; ++i)
    if ((tid + i * kDownThreads) * 8 < Kt) *reinterpret_cast<ld_u32x4 *>(xs + (tid + i * kDownThreads) * 8) = xp[i];
  for (int k = (tid + XP * kDownThreads) * 8; k < Kt; k += kDownThreads * 8) *reinterpret_cast<ld_u32x4 *>(xs + k) = x_at(k);
  __syncthreads();
  float acc = 0.f;
  for (int first = 0; first < chunks; first += Q) {
#pragma unroll
    for (int u = 0; u < Q; ++u) {
      const int c = first + u;
      if (c < chunks) {
        const int meta = table[c].meta;
        if (lane * 8 < (meta >> 20)) acc = ld_dot8(w[u], *reinterpret_cast<const ld_u32x4 *>(xs + (meta & 0xfffff) + lane * 8), acc);
        request(w[u], c + Q);
      }
    }
  }
  acc = wave_sum(acc);
  if (lane == 0 && n < a.N) a.out[n] = n < a.H ? fmaf(a.mult, acc, res) : 0.f;
}

// ---------------------------------------------------------------- launchers
bool latent_single_row_serves(int width, int groups, int max_rank, int max_experts, int64_t down_columns) {
  const char *off = getenv("RAI_HIP_NO_LATENT_FUSED");   // read per call: the tests compare both forms in one process
  if (off && *off && *off != '0') return false;
  return width % 8 == 0 && width <= 4096 && groups <= 16 && (width / groups) % 8 == 0 && max_rank <= 4096 && max_experts <= kRankedExperts && down_columns * 2 + 16 * 1024 <= 150 * 1024;
}

int launch_latent_in(hipStream_t st, LatentInArgs a) {
  const int rows = a.N1 + a.N2;
  // about eight waves per CU at least, whole pairs of rows
  int rpw = (rows + kNumCU * 16 - 1) / (kNumCU * 16);
  a.rows_per_wave = rpw < 2 ? 2 : (rpw + 1) / 2 * 2;
  a.waves1 = (a.N1 + a.rows_per_wave - 1) / a.rows_per_wave;
  const int waves = a.waves1 + (a.N2 + a.rows_per_wave - 1) / a.rows_per_wave;
  const dim3 grid((waves + 3) / 4), block(256);
  if (a.K <= 512) hipLaunchKernelGGL(k_latent_in<1>, grid, block, 0, st, a);
  else if (a.K <= 1024) hipLaunchKernelGGL(k_latent_in<2>, grid, block, 0, st, a);
  else if (a.K <= 2048) hipLaunchKernelGGL(k_latent_in<4>, grid, block, 0, st, a);
  else if (a.K <= 2560) hipLaunchKernelGGL(k_latent_in<5>, grid, block, 0, st, a);
  else hipLaunchKernelGGL(k_latent_in<8>, grid, block, 0, st, a);
  return launch_check("latent_in");
}

int launch_latent_mid(hipStream_t st, LatentMidArgs a) {
  const int rows = a.Nq + a.top * 2 * a.EFp;
  int rpw = (rows + kNumCU * 16 - 1) / (kNumCU * 16);
  a.rows_per_wave = rpw < 2 ? 2 : (rpw + 1) / 2 * 2;
  a.waves_q = (a.Nq + a.rows_per_wave - 1) / a.rows_per_wave;
  a.waves_e = a.top ? (2 * a.EFp + a.rows_per_wave - 1) / a.rows_per_wave : 1;
  const int waves = a.waves_q + a.top * a.waves_e + 1;
  int K = a.Qp > a.Rp ? a.Qp : a.Rp;
  if (a.top && a.Hp > K) K = a.Hp;
  const dim3 grid((waves + 3) / 4), block(256);
  if (K <= 512) hipLaunchKernelGGL(k_latent_mid<1>, grid, block, 0, st, a);
  else if (K <= 1024) hipLaunchKernelGGL(k_latent_mid<2>, grid, block, 0, st, a);
  else if (K <= 2048) hipLaunchKernelGGL(k_latent_mid<4>, grid, block, 0, st, a);
  else if (K <= 2560) hipLaunchKernelGGL(k_latent_mid<5>, grid, block, 0, st, a);
  else hipLaunchKernelGGL(k_latent_mid<8>, grid, block, 0, st, a);
  return launch_check("latent_mid");
}

bool moe_slots_serves(int64_t slots, int experts, int Hp, int top, int EFp) {
  const char *off = getenv("RAI_HIP_NO_LATENT_FUSED");   // read per call: the tests compare both forms in one process
  if (off && *off && *off != '0') return false;
  // more slots than experts: several tokens share an expert, whose weights the grouped tiles read once
  return slots <= 64 && slots <= experts && Hp <= 4096 && (int64_t)top * EFp * 2 + 16 * 1024 <= 150 * 1024;
}
int launch_moe_slots(hipStream_t st, MoeSlotsArgs a) {
  int rpw = (a.slots * 2 * a.EFp + kNumCU * 16 - 1) / (kNumCU * 16);
  a.rows_per_wave = rpw < 2 ? 2 : (rpw + 1) / 2 * 2;
  a.waves_e = (2 * a.EFp + a.rows_per_wave - 1) / a.rows_per_wave;
  const dim3 grid((a.slots * a.waves_e + 3) / 4), block(256);
  if (a.Hp <= 512) hipLaunchKernelGGL(k_moe_slots<1>, grid, block, 0, st, a);
  else if (a.Hp <= 1024) hipLaunchKernelGGL(k_moe_slots<2>, grid, block, 0, st, a);
  else if (a.Hp <= 2048) hipLaunchKernelGGL(k_moe_slots<4>, grid, block, 0, st, a);
  else if (a.Hp <= 2560) hipLaunchKernelGGL(k_moe_slots<5>, grid, block, 0, st, a);
  else hipLaunchKernelGGL(k_moe_slots<8>, grid, block, 0, st, a);
  return launch_check("moe_slots");
}

template <int Q> static int launch_latent_down_q(hipStream_t st, const LatentDownArgs &a, size_t lds) {
  static bool attr_set = false;
  if (!attr_set) {
    RAI_HIP_TRY(hipFuncSetAttribute((const void *)k_latent_down<Q>, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
    attr_set = true;
  }
  hipLaunchKernelGGL(k_latent_down<Q>, dim3((a.N + kDownWaves - 1) / kDownWaves, a.rows), dim3(kDownThreads), lds, st, a);
  return launch_check("latent_down");
}
int launch_latent_down(hipStream_t st, const LatentDownArgs &a) {
  const int chunks = (a.K0 + 511) / 512 + a.top * ((a.K1 + 511) / 512);
  const size_t lds = (size_t)chunks * sizeof(DownChunk) + ((size_t)a.K0 + (size_t)a.top * a.K1) * 2;
  RAI_REQUIRE(lds <= 150 * 1024 && a.K0 % 8 == 0 && a.K1 % 8 == 0, RAI_ERR_UNSUPPORTED, "latent down: %d + %d x %d columns", a.K0, a.top, a.K1);
  if (chunks <= 8) return launch_latent_down_q<8>(st, a, lds);
  if (chunks <= 16) return launch_latent_down_q<16>(st, a, lds);
  if (chunks > 16 && chunks <= 24) return launch_latent_down_q<24>(st, a, lds);
  return launch_latent_down_q<16>(st, a, lds);
}

}  // namespace rai
