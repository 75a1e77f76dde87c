// Rotary positions with f32 angles (rotary.hip): tables on the host's side and the launch that rotates the queries and
// keys of packed projection rows and appends keys and values to the cache.
#pragma once
#include <vector>

#include "common.h"
#include "decode_mega.h"

namespace rai {

// Pair i of the `dims` rotated features (i with i + dims / 2) turns by p * f_i at position p, f_i = base^(-2 i / dims).
// factor > 0: waves longer than original / low positions are stretched by `factor`, those shorter than original / high
// kept, the ones between blended.
struct RotaryParams {
  int dims;
  double base, factor, low, high, original;
};
bool same_rotary(const RotaryParams &a, const RotaryParams &b);
// [positions][dims] cosines and sines, both halves of a row alike.
void rotary_tables(const RotaryParams &r, int positions, std::vector<float> *cs, std::vector<float> *sn);

// rows [q heads | k heads | v heads | ...] of `dtype`, each head D wide, ld apart: row (b, s) is position state->pos + s.
// Queries are rotated in place; rotated keys and the values go to the caches [B][kv_heads][Tmax][D].
struct RotaryAppendArgs {
  void *rows;
  int64_t ld;
  void *kcache, *vcache;
  const float *cos_t, *sin_t;
  const DevState *state;
  int B, S, heads, kv_heads, D, rot, Tmax;
};
int launch_rotary_append(hipStream_t st, int dtype, const RotaryAppendArgs &a);

}  // namespace rai
