// latent_attn.h -- attention over a cache of latents: a row per position holds one
// rotated key part and one normed latent that all heads share, in a ring of
// positions, seen through a sliding window.
#pragma once

#include "bf16_linear.h"

namespace bh {

struct LatentShape {
  int heads = 0, dim = 0, rot_dim = 0, vdim = 0, rank = 0;
  int window = 0;
  float scale = 0.f, eps = 0.f;
  // cache: ring_mask + 1 (a power of two) rows of row_elems() elements
  int ring_mask = 0;
  bool f32 = false; // element type of the cache and of the activations: f32 or bfloat16
  // a row: the rotated part from element 0, the latent from element rot8(), zeros
  int rot8() const { return (int)round_up(rot_dim, 8); }
  int row_elems() const { return (int)round_up(rot8() + rank16(), 32); }
  // a query or key of a head in a prompt's attention: the unrotated part, padded, then
  // the rotated one
  int key_elems() const { return (int)round_up(dim16() + rot8(), 32); }
  int rank16() const { return (int)round_up(rank, 16); }
  int heads16() const { return (int)round_up(heads, 16); }
  int dim16() const { return (int)round_up(dim, 16); }
  int vdim16() const { return (int)round_up(vdim, 16); }
};

// ---- one token ---------------------------------------------------------------
// Attention in the latent space: the query goes through the key matrix once, the
// window's latents are read once for all heads, and the folded latent of a head
// goes through the value matrix.
struct LatentStep {
  LatentShape s;
  const float *proj = nullptr;   // [q | dkv | gate] as the projections leave them
  int dkv_at = 0, gate_at = 0;
  const float *norm_w = nullptr; // [rank]
  const double *turns = nullptr; // [rot_dim / 2]: turns per position
  const int *pos = nullptr;      // device
  Bf16Matrix uk_t;               // per head, one behind the other: [rank16] x dim
  Bf16Matrix uv;                 // per head: [vdim16] x rank
  void *cache = nullptr;
  float *query = nullptr;        // [heads16][row_elems]
  float *part_acc = nullptr;     // [chunks][heads16][rank16]
  float *part_ml = nullptr;      // [chunks][heads16][2]
  float *out = nullptr;          // [heads * vdim], gated
};
// How a step cuts its window: positions per workgroup and workgroups.  `span`: keys
// the launch must cover.
struct LatentCut {
  int key_tiles, chunks; // chunks of 16 * key_tiles positions
};
LatentCut latent_step_cut(const LatentShape &s, int span);
int latent_max_chunks(const LatentShape &s);
int launch_latent_step(const LatentStep &a, int span, hipStream_t stream);

// ---- many tokens ---------------------------------------------------------------
constexpr int kLatentKeyTile = 64; // keys and values are padded to this many positions
struct LatentRows {
  LatentShape s;
  const float *proj = nullptr; // [rows][ld]: q | dkv | gate at their offsets
  int ld = 0, dkv_at = 0, gate_at = 0;
  int rows = 0, start = 0; // rows hold positions start .. start + rows - 1
  const float *norm_w = nullptr;
  const double *turns = nullptr;
  void *cache = nullptr;
  void *queries = nullptr; // [rows][heads][key_elems], rotated and scaled
  // keys and values of the visible positions first .. start + rows - 1, made from
  // the cache: [keys][heads * dim16] and, transposed, [heads * vdim16][value_ld];
  // both with room for a multiple of kLatentKeyTile positions
  const void *keys = nullptr, *values_t = nullptr;
  int value_ld = 0;
  int first = 0;
  void *out = nullptr; // [rows][out_ld], gated
  int out_ld = 0;
};
int latent_first_visible(const LatentShape &s, int start);
// latent norm, rotations, cache rows, queries
int launch_latent_rows(const LatentRows &a, hipStream_t stream);
int launch_latent_attention(const LatentRows &a, hipStream_t stream);

} // namespace bh
