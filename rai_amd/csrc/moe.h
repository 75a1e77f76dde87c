// Device-side choice of experts, shared by the routing kernel (moe.hip) and the single-row step (latent_decode.hip).
#pragma once
#include "common.h"

namespace rai {

constexpr int kRankedExperts = 256;   // the ranking holds up to four logits per lane

// Logits of experts lane, lane + 64, ... of one token (-inf past the end; a NaN counts as -inf, so that ranks stay a
// permutation) and their ranks: rank r = how many experts have a larger logit, the lower expert first among equals.
// Every value is compared with every other through a scalar register, which needs no cross-lane traffic.
template <int N>
__device__ __forceinline__ void rank_experts(const float *z, int experts, int lane, float (&v)[N], int (&rank)[N]) {
#pragma unroll
  for (int i = 0; i < N; ++i) {
    v[i] = lane + 64 * i < experts ? z[lane + 64 * i] : -INFINITY;
    v[i] = v[i] == v[i] ? v[i] : -INFINITY;
    rank[i] = 0;
  }
#pragma unroll
  for (int j = 0; j < N; ++j) {
#pragma unroll 16
    for (int l = 0; l < 64; ++l) {
      const float other = __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v[j]), l));
#pragma unroll
      for (int i = 0; i < N; ++i) rank[i] += other > v[i] || (other == v[i] && 64 * j + l < 64 * i + lane) ? 1 : 0;
    }
  }
}

__device__ __forceinline__ float router_score(float z) { return 1.0f / (1.0f + expf(-z)); }

}  // namespace rai
