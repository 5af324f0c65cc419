// linear_attn.h -- linear attention with a constant decay per head: the state
// S <- decay * S + k v^T and its readout S^T q.  The state and everything that
// enters it are f32.
#pragma once

#include "common.h"

namespace bh {

constexpr int kLinearChunk = 64; // tokens a prompt's chunked form takes at a time

struct LinearShape {
  int heads = 0, dim = 0, vdim = 0;
};
struct LinearStep {
  LinearShape s;
  const float *q = nullptr, *k = nullptr, *v = nullptr; // head by head
  const float *powers = nullptr; // [heads][kLinearChunk + 1]: decay^j
  float *state = nullptr;        // [heads][dim][vdim]
  float *out = nullptr;          // [heads * vdim]
};
int launch_linear_step(const LinearStep &a, hipStream_t stream);

struct LinearRows {
  LinearShape s;
  const float *proj = nullptr; // [rows][ld] with q, k, v at their offsets
  int ld = 0, q_at = 0, k_at = 0, v_at = 0;
  int rows = 0;
  const float *powers = nullptr;
  float *state = nullptr;
  float *chunk_states = nullptr; // [chunks][heads][dim][vdim]
  float *out = nullptr;          // [rows][heads * vdim]
};
inline int linear_chunks(int rows) { return (rows + kLinearChunk - 1) / kLinearChunk; }
int launch_linear_rows(const LinearRows &a, hipStream_t stream);

} // namespace bh
