// Mixture of experts: routing, the device-side plan that sorts (token, choice) slots by expert, and the scaled gather
// of the experts' input rows.  The experts' Linears are the grouped tile kernels (gemm_mfma.hip, gemm.hip); the sum of
// a token's expert outputs is part of the next residual-stream norm (norm.hip).
#include "latent.h"
#include "moe.h"

namespace rai {

// One wave per token, up to 64 N experts; the sigmoid is monotonic, so the largest scores are the largest logits.
template <int N>
__global__ void __launch_bounds__(256) k_moe_route_ranked(const float *logits, int64_t tokens, int experts, int top, int *choice, float *weight) {
  const int64_t t = blockIdx.x * 4ll + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (t >= tokens) return;
  float v[N];
  int rank[N];
  rank_experts<N>(logits + t * experts, experts, lane, v, rank);
#pragma unroll
  for (int i = 0; i < N; ++i)
    if (rank[i] < top && lane + 64 * i < experts) {
      choice[t * top + rank[i]] = lane + 64 * i;
      weight[t * top + rank[i]] = router_score(v[i]);
    }
}

// Any number of experts: one wave per token.  Lane l holds the logits of experts l, l + 64, ...; a chosen one is struck from the lane's mask.
// The lower expert wins a tie.
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
      float v = z[lane + i * 64];
      v = v == v ? v : -INFINITY;
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
      weight[t * top + j] = router_score(bv);
    }
  }
}

int launch_moe_route(hipStream_t st, const float *logits, int64_t tokens, int experts, int top, int *choice, float *weight) {
  RAI_REQUIRE(tokens > 0 && experts >= 1 && experts <= 2048 && top >= 1 && top <= experts, RAI_ERR_BAD_SHAPE, "moe: top %d of %d experts",
              top, experts);
  const dim3 grid((unsigned)((tokens + 3) / 4)), block(256);
  if (experts <= 64) hipLaunchKernelGGL(k_moe_route_ranked<1>, grid, block, 0, st, logits, tokens, experts, top, choice, weight);
  else if (experts <= 128) hipLaunchKernelGGL(k_moe_route_ranked<2>, grid, block, 0, st, logits, tokens, experts, top, choice, weight);
  else if (experts <= kRankedExperts) hipLaunchKernelGGL(k_moe_route_ranked<4>, grid, block, 0, st, logits, tokens, experts, top, choice, weight);
  else hipLaunchKernelGGL(k_moe_route, grid, block, 0, st, logits, tokens, experts, top, choice, weight);
  return launch_check("moe_route");
}

int moe_max_tiles(int64_t slots, int experts, int bm) {
  const int64_t nonempty = slots < experts ? slots : experts;
  return (int)(slots / bm + nonempty);
}

// Few slots (decode): one launch, one block per expert.  Every block counts all experts' slots (LDS), so it knows where its own rows start and which
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

// Many slots (prefill): the slots in chunks of kPlanChunk, one block each, in three launches.
//   count:  counts[chunk][expert]
//   base:   one block turns the counts into the first sorted row of every (chunk, expert), expert-major and chunks in
//           order within an expert, and writes the tile table
//   assign: a slot's row is its (chunk, expert) base plus the earlier slots of the chunk with the same expert
// All of it is counting, so the order is that of the one-launch form: by expert, then by slot.
constexpr int kPlanChunk = 256;

__global__ void __launch_bounds__(kPlanChunk) k_moe_plan_count(const int *choice, int64_t slots, int experts, int *counts) {
  extern __shared__ int hist[];
  for (int i = threadIdx.x; i < experts; i += kPlanChunk) hist[i] = 0;
  __syncthreads();
  const int64_t s = blockIdx.x * (int64_t)kPlanChunk + threadIdx.x;
  if (s < slots) atomicAdd(&hist[choice[s]], 1);
  __syncthreads();
  for (int i = threadIdx.x; i < experts; i += kPlanChunk) counts[(int64_t)blockIdx.x * experts + i] = hist[i];
}

// 1024 threads as `groups` runs of the chunks times `lanes` experts (lanes a power of two, groups * lanes = 1024; more
// experts than lanes take turns).
__global__ void __launch_bounds__(1024) k_moe_plan_base(int *counts, int chunks, int experts, int lanes, int bm, MoePlan plan) {
  extern __shared__ int mb[];                       // part[groups][experts] | first[experts] | tile[experts]
  const int groups = 1024 / lanes, tid = threadIdx.x;
  int *part = mb, *first = part + groups * experts, *tile = first + experts;
  const int g = tid / lanes, el = tid % lanes;
  const int per = (chunks + groups - 1) / groups;
  const int c0 = g * per, c1 = c0 + per < chunks ? c0 + per : chunks;
  for (int e = el; e < experts; e += lanes) {
    int n = 0;
    for (int c = c0; c < c1; ++c) n += counts[(int64_t)c * experts + e];
    part[g * experts + e] = n;
  }
  __syncthreads();
  for (int e = tid; e < experts; e += 1024) {       // exclusive sums over the groups; the total goes to first[e]
    int run = 0;
    for (int i = 0; i < groups; ++i) { const int n = part[i * experts + e]; part[i * experts + e] = run; run += n; }
    first[e] = run;
  }
  __syncthreads();
  if (tid == 0) {                                   // expert offsets, in rows and in tiles
    int row = 0, t = 0;
    for (int e = 0; e < experts; ++e) {
      const int n = first[e];
      first[e] = row;
      tile[e] = t;
      row += n;
      t += (n + bm - 1) / bm;
    }
    *plan.n_tiles = t;
  }
  __syncthreads();
  for (int e = el; e < experts; e += lanes) {
    int run = first[e] + part[g * experts + e];
    for (int c = c0; c < c1; ++c) {
      int *p = counts + (int64_t)c * experts + e;
      const int n = *p;
      *p = run;
      run += n;
    }
    if (g == groups - 1) part[g * experts + e] = run;   // end of the expert's rows
  }
  __syncthreads();
  for (int e = g; e < experts; e += groups) {           // a group of threads writes one expert's tiles
    const int r0 = first[e], n = part[(groups - 1) * experts + e] - r0;
    for (int i = el; i * bm < n; i += lanes) plan.tiles[tile[e] + i] = int4{e, r0 + i * bm, n - i * bm < bm ? n - i * bm : bm, 0};
  }
}

__global__ void __launch_bounds__(kPlanChunk) k_moe_plan_assign(const int *choice, int64_t slots, int experts, const int *base, MoePlan plan, int *row_of_slot) {
  extern __shared__ int waves[];                    // [4][experts]: slots of each expert in each wave
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int i = tid; i < 4 * experts; i += kPlanChunk) waves[i] = 0;
  __syncthreads();
  const int64_t s = blockIdx.x * (int64_t)kPlanChunk + tid;
  const int e = s < slots ? choice[s] : -1;
  // lanes with the same expert: those that agree on every bit of its number (and on having one)
  unsigned long long same = __ballot(e >= 0);
  for (int b = 0; (1 << b) < experts; ++b) {
    const unsigned long long ones = __ballot((e >> b) & 1);
    same &= (e >> b) & 1 ? ones : ~ones;
  }
  const int before = __popcll(same & ((1ull << lane) - 1ull));
  if (e >= 0 && before == 0) waves[wave * experts + e] = __popcll(same);
  __syncthreads();
  if (e < 0) return;
  int row = base[(int64_t)blockIdx.x * experts + e] + before;
  for (int w = 0; w < wave; ++w) row += waves[w * experts + e];
  plan.slot_of[row] = (int)s;
  row_of_slot[s] = row;
}

int64_t moe_plan_counts(int64_t slots, int experts) { return slots > kPlanFewSlots ? (slots + kPlanChunk - 1) / kPlanChunk * experts : 0; }

int launch_moe_plan(hipStream_t st, const int *choice, int64_t slots, int experts, int bm, const MoePlan &plan, int *row_of_slot) {
  RAI_REQUIRE(slots > 0 && slots < (1ll << 31) && moe_max_tiles(slots, experts, bm) <= plan.cap_tiles, RAI_ERR_BAD_SHAPE, "moe: %lld slots",
              (long long)slots);
  if (slots > kPlanFewSlots && experts <= kPlanExperts) {
    const int chunks = (int)((slots + kPlanChunk - 1) / kPlanChunk);
    int lanes = 1;
    while (lanes < experts && lanes < 1024) lanes *= 2;
    const size_t lds = (size_t)(1024 / lanes + 2) * experts * sizeof(int);
    hipLaunchKernelGGL(k_moe_plan_count, dim3(chunks), dim3(kPlanChunk), (size_t)experts * sizeof(int), st, choice, slots, experts, plan.counts);
    RAI_TRY(launch_check("moe_plan_count"));
    hipLaunchKernelGGL(k_moe_plan_base, dim3(1), dim3(1024), lds, st, plan.counts, chunks, experts, lanes, bm, plan);
    RAI_TRY(launch_check("moe_plan_base"));
    hipLaunchKernelGGL(k_moe_plan_assign, dim3(chunks), dim3(kPlanChunk), (size_t)4 * experts * sizeof(int), st, choice, slots, experts, plan.counts, plan, row_of_slot);
    return launch_check("moe_plan_assign");
  }
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
