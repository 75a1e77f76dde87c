// Mixture of experts: routing, the device-side plan that sorts (token, choice) slots by expert, and the scaled gather
// of the experts' input rows.  The experts' Linears are the grouped tile kernels (gemm_mfma.hip, gemm.hip); the sum of
// a token's expert outputs is part of the next residual-stream norm (norm.hip).
#include "latent.h"

namespace rai {

// One wave per token.  Lane l holds the logits of experts l, l + 64, ...; a chosen one is struck from the lane's mask.
// The sigmoid is monotonic, so the largest scores are the largest logits; the lower expert wins a tie.
__global__ void __launch_bounds__(256) k_moe_route(const float *logits, int64_t tokens, int experts, int top, int *choice, float *weight) {
  const int64_t t = blockIdx.x * 4ll + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (t >= tokens) return;
  const float *z = logits + t * experts;
  uint32_t taken = 0;
  for (int j = 0; j < top; ++j) {
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = 0; lane + i * 64 < experts; ++i) {
      const float v = z[lane + i * 64];
      if (!((taken >> i) & 1u) && (v > bv || bi == 0x7fffffff)) { bv = v; bi = lane + i * 64; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(bv, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (oi != 0x7fffffff && (bi == 0x7fffffff || ov > bv || (ov == bv && oi < bi))) { bv = ov; bi = oi; }
    }
    if ((bi & 63) == lane) taken |= 1u << (bi >> 6);
    if (lane == 0) {
      choice[t * top + j] = bi;
      weight[t * top + j] = 1.0f / (1.0f + expf(-bv));
    }
  }
}

int launch_moe_route(hipStream_t st, const float *logits, int64_t tokens, int experts, int top, int *choice, float *weight) {
  RAI_REQUIRE(tokens > 0 && experts >= 1 && experts <= 2048 && top >= 1 && top <= experts, RAI_ERR_BAD_SHAPE, "moe: top %d of %d experts",
              top, experts);
  hipLaunchKernelGGL(k_moe_route, dim3((unsigned)((tokens + 3) / 4)), dim3(256), 0, st, logits, tokens, experts, top, choice, weight);
  return launch_check("moe_route");
}

int moe_max_tiles(int64_t slots, int experts, int bm) {
  const int64_t nonempty = slots < experts ? slots : experts;
  return (int)(slots / bm + nonempty);
}

// One block per expert.  Every block counts all experts' slots (LDS), so it knows where its own rows start and which
// tiles are its own without waiting for any other; a second pass over the choices hands out the rows in slot order.
__global__ void __launch_bounds__(1024) k_moe_plan(const int *choice, int64_t slots, int experts, int bm, MoePlan plan, int *row_of_slot) {
  extern __shared__ int hist[];           // [experts]
  __shared__ int s_first, s_tile, s_count, wave_n[16];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int i = tid; i < experts; i += 1024) hist[i] = 0;
  if (tid == 0) s_count = 0;
  __syncthreads();
  for (int64_t s = tid; s < slots; s += 1024) atomicAdd(&hist[choice[s]], 1);
  __syncthreads();
  if (wave == 0) {
    int first = 0, tile = 0, all = 0;
    for (int i = lane; i < experts; i += 64) {
      const int n = hist[i], nt = (n + bm - 1) / bm;
      if (i < e) { first += n; tile += nt; }
      all += nt;
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      first += __shfl_xor(first, o, 64);
      tile += __shfl_xor(tile, o, 64);
      all += __shfl_xor(all, o, 64);
    }
    if (lane == 0) {
      s_first = first;
      s_tile = tile;
      if (e == 0) *plan.n_tiles = all;
    }
  }
  __syncthreads();
  const int mine = hist[e], first = s_first;
  for (int i = tid; i * bm < mine; i += 1024)
    plan.tiles[s_tile + i] = int4{e, first + i * bm, mine - i * bm < bm ? mine - i * bm : bm, 0};
  if (mine == 0) return;
  for (int64_t s0 = 0; s0 < slots; s0 += 1024) {
    const int64_t s = s0 + tid;
    const bool hit = s < slots && choice[s] == e;
    const unsigned long long vote = __ballot(hit);
    if (lane == 0) wave_n[wave] = __popcll(vote);
    __syncthreads();
    int base = s_count;
    for (int w = 0; w < wave; ++w) base += wave_n[w];
    if (hit) {
      const int row = first + base + __popcll(vote & ((1ull << lane) - 1ull));
      plan.slot_of[row] = (int)s;
      row_of_slot[s] = row;
    }
    __syncthreads();
    if (tid == 0) {
      int n = 0;
      for (int w = 0; w < 16; ++w) n += wave_n[w];
      s_count += n;
    }
    __syncthreads();
    if (s_count == mine) break;   // the same value for every thread
  }
}

int launch_moe_plan(hipStream_t st, const int *choice, int64_t slots, int experts, int bm, const MoePlan &plan, int *row_of_slot) {
  RAI_REQUIRE(slots > 0 && slots < (1ll << 31) && moe_max_tiles(slots, experts, bm) <= plan.cap_tiles, RAI_ERR_BAD_SHAPE, "moe: %lld slots",
              (long long)slots);
  hipLaunchKernelGGL(k_moe_plan, dim3(experts), dim3(1024), (size_t)experts * sizeof(int), st, choice, slots, experts, bm, plan, row_of_slot);
  return launch_check("moe_plan");
}

template <typename T>
__global__ void __launch_bounds__(256) k_moe_gather(const T *h, int64_t ld, int cols, const int *slot_of, const float *weight, int top,
                                                    int64_t slots, T *out) {
  constexpr int V = 16 / sizeof(T);
  struct alignas(16) Pack { T v[V]; };
  const int packs = cols / V;
  for (int64_t i = blockIdx.x * 256ll + threadIdx.x; i < slots * packs; i += (int64_t)gridDim.x * 256) {
    const int64_t r = i / packs;
    const int p = (int)(i - r * packs);
    const int slot = slot_of[r];
    const float w = weight[slot];
    Pack x = *reinterpret_cast<const Pack *>(h + (int64_t)(slot / top) * ld + p * V);
#pragma unroll
    for (int e = 0; e < V; ++e) Scalar<T>::store(&x.v[e], w * (float)Scalar<T>::load(&x.v[e]));
    *reinterpret_cast<Pack *>(out + r * cols + p * V) = x;
  }
}

int launch_moe_gather(hipStream_t st, int dtype, const void *h, int64_t ld, int cols, const MoePlan &plan, const float *weight, int top,
                      int64_t slots, void *out) {
  const int64_t packs = slots * (cols / (dtype == RAI_BF16 ? 8 : 4));
  const int64_t b = (packs + 255) / 256;
  const dim3 grid((unsigned)(b < kNumCU * 32 ? b : kNumCU * 32)), block(256);
  if (dtype == RAI_BF16)
    hipLaunchKernelGGL(k_moe_gather<bf16_raw>, grid, block, 0, st, (const bf16_raw *)h, ld, cols, plan.slot_of, weight, top, slots, (bf16_raw *)out);
  else
    hipLaunchKernelGGL(k_moe_gather<float>, grid, block, 0, st, (const float *)h, ld, cols, plan.slot_of, weight, top, slots, (float *)out);
  return launch_check("moe_gather");
}

}  // namespace rai
