// Device pieces of the gated delta rule shared by delta.hip and delta_chunk.hip.
#pragma once
#include "delta.h"

namespace rai {

__device__ __forceinline__ float dl_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float dl_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
// log(1 + exp(z)); for results that meet bf16 operands through the hardware's exp2 and log2 and a short series where the
// logarithm's argument is close to 1 (relative error below 1e-6).
template <typename T> __device__ __forceinline__ float softplus_for(float z) {
  if constexpr (sizeof(T) == 4) return dl_softplus(z);
  const float x = __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z));
  const float series = x * (1.f - x * (0.5f - x * (0.33333333f - x * (0.25f - x * 0.2f))));
  return fmaxf(z, 0.f) + (x < 0.06f ? series : 0.69314718056f * __builtin_amdgcn_logf(1.f + x));
}

template <typename T> __device__ __forceinline__ float ld(const void *p, int64_t i) { return (float)Scalar<T>::load((const T *)p + i); }

// The inputs of the last `taps` tokens of this call go to their places in the ring: the v channels of head h, and with
// the first head of a group the group's q and k channels.
template <typename T>
__device__ __forceinline__ void update_ring(const DeltaArgs &a, int b, int h, int pos0, int tid, int nt) {
  const DeltaShape &z = a.s;
  const int rep = z.heads / z.kv_heads, kd = z.kv_heads * z.Dk;
  const int nqk = h % rep == 0 ? 2 * z.Dk : 0, n = nqk + z.Vp;
  for (int i = tid; i < n; i += nt) {
    const int c = i < nqk ? (i < z.Dk ? (h / rep) * z.Dk + i : kd + (h / rep) * z.Dk + i - z.Dk) : 2 * kd + h * z.Vp + i - nqk;
    for (int s = a.S > z.taps ? a.S - z.taps : 0; s < a.S; ++s)
      ((T *)a.ring)[((int64_t)b * z.taps + (pos0 + s) % z.taps) * z.channels + c] = ((const T *)a.dn)[((int64_t)b * a.S + s) * z.ldn + c];
  }
}

}  // namespace rai
