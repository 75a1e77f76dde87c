// Launchers of the gated delta rule with a decay per key channel (delta.hip).  Per sequence and head a state S [Dk][Vp]
// in f32 is carried from token to token:
//   S <- g * S (rows),  u = beta (v - S^T k),  S <- S + k u^T,  o = S^T q.
// q, k and v pass a short causal convolution over time and silu, q and k are then made unit vectors per head.
#pragma once
#include "common.h"
#include "decode_mega.h"

namespace rai {

// The sizes of one layer.  Dk and Vp are the padded head widths (multiples of 32; padding channels have zero weights),
// dim and vdim the real ones.  Projection rows are [q (kv_heads Dk) | k (kv_heads Dk) | v (heads Vp) | ...], ldn apart;
// the first `channels` columns pass the convolution.
struct DeltaShape {
  int heads, kv_heads, dim, vdim, Dk, Vp, taps;
  int channels;
  int64_t ldn;
  int off_b, off_a1, off_g1;   // columns of beta's projection and of the two low-rank factors
};
constexpr int kDeltaMaxHead = 512;   // largest Dk or Vp

struct DeltaArgs {
  DeltaShape s;
  int B, S;
  const DevState *state;       // row (b, s) is position state->pos + s; at position 0 the carried state counts as zero
  const void *dn;              // projection rows
  const void *conv;            // [channels][taps]
  void *ring;                  // [B][taps][channels]: the inputs of the last `taps` positions, position p at p mod taps
  float *carried;              // [B][heads][Dk][Vp]
  const void *A_log, *dt_bias; // [heads], [heads Dk]
  float *decay;                // [rows, heads Dk]: the low-rank factor's output (k_delta_decay makes it log g in place)
  void *q, *k;                 // [rows, kv_heads Dk] of the model dtype, after convolution and silu
  float *qn, *kn;              // [rows, kv_heads]: what makes each a unit vector (queries: times dim^-1/2)
  float *beta;                 // [rows, heads]
  void *v;                     // [rows, heads Vp] of the model dtype
  float *o;                    // [rows + 1, heads Vp], the last row is scratch
  const void *norm_w;          // [Vp]
  float eps;
  const void *gate;            // [rows, heads Vp], before its sigmoid
  void *out;                   // rows ldo apart
  int64_t ldo;
  // step only, one row: the low-rank factors' second halves folded in (rank padded to a multiple of 8); null: decay and
  // gate were computed before
  const void *a2, *g2;         // [heads Dk, a_rank], [heads Vp, g_rank]
  int a_rank, g_rank;
  char *chunk_ws;              // delta_chunk_ws_bytes(); null: the chunked form is not used
};
// The chunked form (bf16 models): see delta_chunk.hip.
constexpr int kDeltaChunk = 64;
bool delta_chunk_serves(int dtype, const DeltaShape &s);
size_t delta_chunk_ws_bytes(const DeltaShape &s, int64_t max_batch, int64_t max_rows);
int launch_delta_chunks(hipStream_t st, const DeltaArgs &a);   // the recurrence only, after the preparation
// Any number of tokens: preparation (convolutions, unit vectors, decays), recurrence, norm and gate.
int launch_delta_tokens(hipStream_t st, int dtype, const DeltaArgs &a);
// One token per sequence in one launch, where it serves the head sizes.
bool delta_step_serves(const DeltaShape &s);
int launch_delta_step(hipStream_t st, int dtype, const DeltaArgs &a);

}  // namespace rai
