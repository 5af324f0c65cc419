// head_attn.h -- attention over a cache of per-head keys and values, causal or through a
// sliding window: grouped query heads, rotary positions on a part of a head, and as
// parameters a sink in the softmax's denominator, two maps per head that are subtracted
// (differential attention), and a gate on the output.
#pragma once

#include "common.h"

namespace bh {

constexpr int kHeadKeyTile = 64; // positions of a cache are laid out in tiles of this many

struct HeadShape {
  int heads = 0, kv_heads = 0; // query head h reads key / value head h / (heads / kv_heads)
  int maps = 1;                // 1 or 2: query and key parts of a head, over the same values
  int dim = 0, vdim = 0, rot_dims = 0;
  int window = 0; // keys a position sees, itself included; 0: all before it
  float scale = 0.f;
  float rot_gain = 1.f;
  // maps == 2: (a1 - lambda * a2), over its root mean square, times out_gain
  float lambda = 0.f, eps = 0.f, out_gain = 1.f;
  const float *sink = nullptr;   // [heads]: one more score without a value, or null
  const double *turns = nullptr; // [rot_dims / 2]: turns per position
  bool gated = false;            // times sigmoid(gate)
  // cache: position p in row p & ring_mask of `rows` (a multiple of kHeadKeyTile)
  int rows = 0, ring_mask = 0;
  bool f32 = false; // element type of the cache and of the activations: f32 or bfloat16
  int dim32() const { return (int)round_up(dim, 32); }
  int vdim16() const { return (int)round_up(vdim, 16); }
  int map_heads() const { return heads * maps; }
  size_t elem_bytes() const { return f32 ? 4 : 2; }
  // keys: [kv_heads * maps][rows][dim32], zeros past dim; values: [kv_heads][vdim16][rows]
  size_t key_bytes() const { return elem_bytes() * kv_heads * maps * (size_t)rows * dim32(); }
  size_t value_bytes() const { return elem_bytes() * kv_heads * (size_t)vdim16() * rows; }
};

// Sizes the cache: a ring for windows that fit one below max_len positions, else a row
// per position.  `block`: the most tokens that are added at once.
void head_cache_rows(HeadShape &s, int max_len, int block);

// ---- one token -----------------------------------------------------------------------
struct HeadStep {
  HeadShape s;
  const float *proj = nullptr; // q, k, v and the gate at their offsets
  int q_at = 0, k_at = 0, v_at = 0, gate_at = 0;
  const int *pos = nullptr; // device
  void *keys = nullptr, *values_t = nullptr;
  float *part_acc = nullptr; // [chunks][map_heads][vdim16]
  float *part_ml = nullptr;  // [chunks][map_heads][2]
  float *out = nullptr;      // [heads * vdim]
};
int head_max_chunks(const HeadShape &s, int max_len);
// `span`: visible keys the launch must cover
int launch_head_step(const HeadStep &a, int span, hipStream_t stream);

// ---- many tokens ---------------------------------------------------------------------
struct HeadRows {
  HeadShape s;
  const float *proj = nullptr; // [rows][ld]
  int ld = 0, q_at = 0, k_at = 0, v_at = 0, gate_at = 0;
  int rows = 0, start = 0; // rows hold positions start .. start + rows - 1
  void *keys = nullptr, *values_t = nullptr;
  void *queries = nullptr; // [rows][map_heads][dim32]
  float *maps_out = nullptr; // [rows][map_heads][vdim]: needed with two maps or a gate
  void *out = nullptr;       // [rows][out_ld]
  int out_ld = 0;
};
// rotations, cache, attention, and what stands behind it
int launch_head_rows(const HeadRows &a, hipStream_t stream);

} // namespace bh
