#include "rotary.h"

#include <cmath>

namespace rai {

bool same_rotary(const RotaryParams &a, const RotaryParams &b) {
  return a.dims == b.dims && a.base == b.base && a.factor == b.factor &&
         (a.factor <= 0 || (a.low == b.low && a.high == b.high && a.original == b.original));
}

void rotary_tables(const RotaryParams &r, int positions, std::vector<float> *cs, std::vector<float> *sn) {
  const int half = r.dims / 2;
  const double two_pi = 6.283185307179586476925;
  cs->resize((size_t)positions * r.dims);
  sn->resize((size_t)positions * r.dims);
  for (int i = 0; i < half; ++i) {
    double f = pow(r.base, -2.0 * i / r.dims);
    if (r.factor > 0) {
      const double wave = two_pi / f;
      if (wave > r.original / r.low) f /= r.factor;
      else if (wave >= r.original / r.high) {
        const double s = (r.original / wave - r.low) / (r.high - r.low);
        f = (1.0 - s) * f / r.factor + s * f;
      }
    }
    for (int p = 0; p < positions; ++p) {
      const size_t e = (size_t)p * r.dims + i;
      (*cs)[e] = (*cs)[e + half] = (float)cos(p * f);
      (*sn)[e] = (*sn)[e + half] = (float)sin(p * f);
    }
  }
}

// One thread per pack of V features; a pack of the first half of the rotated features takes its partner along, so the
// update of q stays in place.
template <typename T, int V>
__global__ void __launch_bounds__(256) k_rotary_append(RotaryAppendArgs a) {
  struct alignas(sizeof(T) * V) Pack { T v[V]; };
  const int pos0 = a.state->pos, half = a.rot / 2;
  const uint32_t units = a.heads + 2 * a.kv_heads, packs = a.D / V;
  const int64_t total = (int64_t)a.B * a.S * units * packs;
  for (int64_t e = blockIdx.x * (int64_t)blockDim.x + threadIdx.x; e < total; e += (int64_t)gridDim.x * blockDim.x) {
    const int d = (int)(e % packs) * V;
    const int64_t r = e / packs;
    const int unit = (int)(r % units);
    const int64_t row = r / units;
    const int s = (int)(row % a.S), b = (int)(row / a.S), pos = pos0 + s;
    T *src = (T *)a.rows + row * a.ld + (int64_t)unit * a.D;
    T *dst = src;
    if (unit >= a.heads) {
      const bool key = unit < a.heads + a.kv_heads;
      const int kv = key ? unit - a.heads : unit - a.heads - a.kv_heads;
      dst = (T *)(key ? a.kcache : a.vcache) + (((int64_t)b * a.kv_heads + kv) * a.Tmax + pos) * a.D;
      if (!key) {
        *reinterpret_cast<Pack *>(dst + d) = *reinterpret_cast<const Pack *>(src + d);
        continue;
      }
    }
    if (d >= a.rot) {
      if (dst != src) *reinterpret_cast<Pack *>(dst + d) = *reinterpret_cast<const Pack *>(src + d);
    } else if (d < half) {
      const Pack u = *reinterpret_cast<const Pack *>(src + d), v = *reinterpret_cast<const Pack *>(src + d + half);
      const float *c = a.cos_t + (int64_t)pos * a.rot + d, *n = a.sin_t + (int64_t)pos * a.rot + d;
      Pack o1, o2;
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float x = (float)Scalar<T>::load(&u.v[j]), y = (float)Scalar<T>::load(&v.v[j]);
        Scalar<T>::store(&o1.v[j], fmaf(x, c[j], -y * n[j]));
        Scalar<T>::store(&o2.v[j], fmaf(y, c[j], x * n[j]));
      }
      *reinterpret_cast<Pack *>(dst + d) = o1;
      *reinterpret_cast<Pack *>(dst + d + half) = o2;
    }
  }
}

template <typename T, int V> static int launch_rotary_append_t(hipStream_t st, const RotaryAppendArgs &a) {
  const int64_t total = (int64_t)a.B * a.S * (a.heads + 2 * a.kv_heads) * (a.D / V);
  const int64_t blocks = (total + 255) / 256;
  hipLaunchKernelGGL((k_rotary_append<T, V>), dim3((unsigned)(blocks < 65536 ? blocks : 65536)), dim3(256), 0, st, a);
  return launch_check("rotary_append");
}

int launch_rotary_append(hipStream_t st, int dtype, const RotaryAppendArgs &a) {
  RAI_REQUIRE(a.rot >= 0 && a.rot % 2 == 0 && a.rot <= a.D, RAI_ERR_BAD_ARG, "rotary: %d of %d features", a.rot, a.D);
  const int v = dtype == RAI_BF16 ? 8 : 4;
  const bool vec = a.D % v == 0 && (a.rot / 2) % v == 0 && a.ld % v == 0 && (uintptr_t)a.rows % 16 == 0;
  if (dtype == RAI_BF16) return vec ? launch_rotary_append_t<bf16_raw, 8>(st, a) : launch_rotary_append_t<bf16_raw, 1>(st, a);
  return vec ? launch_rotary_append_t<float, 4>(st, a) : launch_rotary_append_t<float, 1>(st, a);
}

}  // namespace rai
