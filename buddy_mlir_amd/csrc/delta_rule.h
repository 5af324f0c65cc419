// delta_rule.h -- the gated delta rule with a decay per key channel: per head a state S
// [dim, vdim] with S <- diag(g) S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q.
// Queries, keys and values pass a short causal convolution and silu; queries and keys
// are made unit vectors; the decay and the output's gate come from low-rank projections.
// Everything behind the projections is f32.
#pragma once

#include "bf16_linear.h"

namespace bh {

struct DeltaShape {
  int heads = 0, kv_heads = 0; // head h reads query / key head h / (heads / kv_heads)
  int dim = 0, vdim = 0, taps = 0;
  int decay_rank = 0, gate_rank = 0;
  float eps = 0.f; // of the output's norm
  // where the parts lie in a row of projections: the convolution's inputs (query, key,
  // value) first, then step size, inner decay, inner gate
  int q_at = 0, k_at = 0, v_at = 0, beta_at = 0, decay_at = 0, gate_at = 0;
  int channels = 0;                // columns of the convolution: [0, channels)
  const float *conv_w = nullptr;   // [taps][channels]
  const uint16_t *decay_w = nullptr, *gate_w = nullptr; // bfloat16 [heads * dim][decay_rank], [heads * vdim][gate_rank]
  const float *decay_bias = nullptr; // [heads * dim]
  const float *decay_speed = nullptr; // [heads]: log g = decay_speed * softplus(. + bias)
  const float *norm_w = nullptr;      // [vdim]
  Bf16Matrix decay, gate;             // the same two matrices for many rows
  int dim32() const { return (int)round_up(dim, 32); }
  int vdim16() const { return (int)round_up(vdim, 16); }
};

struct DeltaRows {
  DeltaShape s;
  const float *proj = nullptr; // [rows][ld]
  int ld = 0, rows = 0, start = 0; // rows hold positions start .. start + rows - 1
  const int *pos = nullptr;        // device: in place of `start`, for one row
  float *ring = nullptr;           // [taps][channels], position p in slot p % taps
  float *state = nullptr;          // [heads][dim][vdim]
  float *o = nullptr, *gate = nullptr; // launch_delta_scan: [rows][heads * vdim], outputs ahead of norm and gate
  void *out = nullptr;             // launch_delta_chunks: [rows][out_ld], normed and gated
  int out_ld = 0;
  bool act_f32 = true;             // type of out: f32 or bfloat16
};
// Token by token: a step of decoding, short portions.
int launch_delta_scan(const DeltaRows &a, hipStream_t stream);

// out = per head o / rms(o) * norm_w * sigmoid(gate)
int launch_delta_gate(const DeltaShape &s, const float *o, const float *gate, int ld_gate, int rows, void *out,
                      int out_ld, bool act_f32, hipStream_t stream);

// A prompt in chunks of kDeltaChunk tokens.  Within a chunk the writes are solved for as
// one triangular system; the state goes from chunk to chunk.
constexpr int kDeltaChunk = 64;
// floats of scratch for `rows` tokens; 0: the state's size is not one the chunks take
size_t delta_workspace(const DeltaShape &s, int rows);
int launch_delta_chunks(const DeltaRows &a, float *workspace, hipStream_t stream);

} // namespace bh
