// row_ops.h -- what a decoder layer does to whole rows between its matrix products
// when it runs many tokens: residual sums, norms, the input convolution, routing.
#pragma once

#include "common.h"

namespace bh {

// x[r] = scale * table[token[r]] (bfloat16 table); with norm_w ([width]) then
// x[r] / rms(x[r]) * norm_w
int launch_embed_rows(const uint16_t *table, const int *tokens, int rows, int width, int vocab,
                      float scale, const float *norm_w, float eps, float *x, hipStream_t stream);

// Per row: x' = x + y * (out_gain / rms(y)), then x' * (gain / rms(x')).  y may be
// missing, a row, or a row plus the weighted outputs of the row's experts.  `plain_y`:
// x' = x + y.  `add`: one row that is added to every x' as well.  `norm_w`: a weight
// per channel on the normed row.
struct NormRows {
  float *x = nullptr;            // [rows][width]
  bool write_x = false;          // x' goes back into x
  const float *y = nullptr;      // [rows][ldy], or null
  int ldy = 0;
  const float *expert_out = nullptr; // [rows * top][lde]
  const float *expert_w = nullptr;   // [rows][top]
  int lde = 0, top = 0;
  float out_gain = 1.f, gain = 1.f, eps = 0.f;
  bool plain_y = false;
  const float *add = nullptr, *norm_w = nullptr; // [width]
  int rows = 0, width = 0;
  const int *pick = nullptr;     // output row r is made from row pick[r]; `rows` counts outputs
  float *out_f32 = nullptr;      // [rows][width]
  void *out_act = nullptr;       // [rows][ld_act], f32 or bfloat16
  int ld_act = 0;
  bool act_f32 = false;
};
int launch_norm_rows(const NormRows &a, hipStream_t stream);

// out[r] = h[r] + causal convolution over time per channel; rows before the first
// come from the ring ([taps][width], position p in slot p % taps).  Afterwards the
// ring holds the last rows, and conv_next ([2][width], position p in slot p % 2) what
// they add at the position that follows.
struct ConvRows {
  const float *h = nullptr; // [rows][width]
  const float *w = nullptr; // [taps][width]
  float *ring = nullptr, *next = nullptr;
  int taps = 0, width = 0, rows = 0, start = 0;
  void *out = nullptr;
  int ld = 0;
  bool act_f32 = false;
};
int launch_conv_rows(const ConvRows &a, hipStream_t stream); 

// out[r] = (x[r] / rms(x[r])) * w * sigmoid(gate[r])
struct GatedNormRows {
  const float *x = nullptr; // [rows][width]
  const float *w = nullptr;
  const float *gate = nullptr; // [rows][ld_gate]
  int ld_gate = 0, rows = 0, width = 0;
  float eps = 0.f;
  void *out = nullptr;
  int ld = 0;
  bool act_f32 = false;
};
int launch_gated_norm_rows(const GatedNormRows &a, hipStream_t stream);

// The `top` largest logits of every row (equal ones by index), their softmax, and
// for each expert the list of assignments row * top + rank, rows ascending.
struct RouteRows {
  const float *logits = nullptr; // [rows][ld]
  int ld = 0, rows = 0, experts = 0, top = 0;
  int *chosen = nullptr;   // [rows][top]
  float *weights = nullptr; // [rows][top]
  int *counts = nullptr;   // [experts]
  int *lists = nullptr;    // [experts][list_cap]
  int list_cap = 0;
};
int launch_route_rows(const RouteRows &a, hipStream_t stream);

} // namespace bh
