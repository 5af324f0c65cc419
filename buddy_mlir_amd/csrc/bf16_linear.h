// bf16_linear.h -- products with resident bfloat16 matrices: one row (decode) and
// many rows (prefill), and the forms that pick expert matrices by a router.
//
// "bf16 wave tiles": a matrix of N output channels x K inputs is padded to
// Kp = ceil64(K), Np = ceil16(N) and cut into tiles of 16 channels x 32 k, 1 KiB
// each.  Tile (g, c) is at byte ((g * Kp / 32) + c) * 1024; lane L owns the 16
// bytes holding k = c*32 + (L/16)*8 + 0..7 of channel g*16 + L%16: as it lies,
// the A operand of v_mfma_f32_16x16x32_bf16, and with the k of a tile taken in
// the order (j, L/16) the A operands of eight v_mfma_f32_16x16x4_f32.
#pragma once

#include "bf16_dev.h"

namespace bh {

constexpr int kBfTileK = 32;

// A packed matrix, or several packed one behind the other, each padded to 16
// channels.
struct Bf16Matrix {
  const uint4 *tiles = nullptr;
  int N = 0;      // channels including padding (a multiple of 16)
  int K = 0;      // inputs without padding
  int ktiles = 0; // 2 * ceil64(K) / 64
  int groups() const { return N / 16; }
};
inline int bf16_ktiles(int64_t K) { return (int)(2 * ceil_div(K, 64)); }
inline size_t bf16_tiles_bytes(int64_t K, int64_t N) {
  return (size_t)ceil_div(N, 16) * bf16_ktiles(K) * 1024;
}
// element (n, k) is at src[n * stride_n + k * stride_k]
int launch_pack_bf16(const uint16_t *src, int64_t stride_n, int64_t stride_k, int64_t N, int64_t K,
                     void *tiles, hipStream_t stream);

// ---- one row -------------------------------------------------------------------
// What a launch multiplies.
enum RowInput {
  kRowPlain = 0,   // src
  kRowNorm = 1,    // x' = src + y * (out_gain / rms(y)) (src alone without y), then
                   // x' * (gain / rms(x')), then, with conv_w, itself plus its
                   // causal convolution over the ring of earlier rows
  kRowGated = 2,   // (src / rms(src)) * weight * sigmoid(gate)
  kRowResidual = 3, // x' = src + y + add (each may be missing), then x' / rms(x') * norm_w
  kRowHeadGated = 4 // like kRowGated with the mean over heads of head_dim values each,
                    // which share the weight [head_dim]
};
struct RowGemv {
  Bf16Matrix W;
  RowInput input = kRowPlain;
  const float *src = nullptr;
  bool src_padded = false; // src has (finite) values up to a multiple of 64
  float eps = 0.f;
  // kRowNorm
  const float *y = nullptr;
  float out_gain = 1.f, gain = 1.f;
  float *x_out = nullptr;         // x' (must not be src)
  float *row_out = nullptr;       // the finished input row
  const float *conv_w = nullptr;  // [taps][K]
  float *conv_ring = nullptr;     // [taps][K], row of position p in slot p % taps
  float *conv_next = nullptr;     // [2][K]: what earlier rows add at position p, in slot p % 2
  int taps = 0;
  const int *pos = nullptr;       // device: position of the row
  // kRowGated, kRowHeadGated
  const float *weight = nullptr, *gate = nullptr;
  int head_dim = 0;
  // kRowResidual (also eps, y, x_out, row_out)
  const float *add = nullptr, *norm_w = nullptr;
  // kRowResidual: W holds two matrices of N / 2 channels, the second one behind the
  // first; out [N / 2] = gated activation of the two
  bool gated = false;
  GatedAct act = kActGeluTanh;
  // output: channels below silu_channels go through silu
  float *out = nullptr;
  int silu_channels = 0;
  // first maximum of every group of 16 channels, channels below `valid` only
  float *max_v = nullptr;
  int *max_i = nullptr;
  int valid = 0;
};
int launch_row_gemv(const RowGemv &a, hipStream_t stream);

// Expert matrices: expert e's gate | up are two packed matrices behind each
// other, down is one.
struct ExpertSet {
  const uint4 *gate_up = nullptr, *down = nullptr;
  int count = 0, ff = 0;
  float limit = 0.f;
};
// Clamped gated activation of an expert: g = min(g, limit), u = clamp(u, +-limit),
// g * sigmoid(1.702 g) * (u + 1).
struct RowMoe {
  const float *h = nullptr;       // [width]
  const float *logits = nullptr;  // router logits [experts]
  int width = 0, top = 0;
  ExpertSet experts, shared;      // shared.count 0 or 1
  float *act = nullptr;           // [top + 1][max ceil64(ff)]
  int act_stride = 0;
  int *chosen = nullptr;          // [top], written by the first launch
  float *weights = nullptr;       // [top]
  float *out = nullptr;           // [ceil16(width)]
};
constexpr int kMaxExperts = 512;
int launch_row_moe(const RowMoe &a, hipStream_t stream);

// ---- many rows -----------------------------------------------------------------
// C[rows, N] = A[rows, K] . W^T on the matrix cores with f32 sums.  A is bfloat16
// (bf16 products) or f32 (f32 products: nothing is rounded below 32 bits).
enum GemmOut {
  kOutF32 = 0,       // C f32 [rows][ldc]
  kOutAct = 1,       // C in A's type [rows][ldc]
  kOutActTrans = 2,  // C in A's type [N][ldc], a row per channel
  kOutExpertAct = 3  // two matrices: the gated activation of both, A's type [rows][ldc]
};
struct RowsGemm {
  Bf16Matrix W;               // kOutExpertAct: N channels each, second one behind the first
  const void *A = nullptr;    // row r at A + r * lda elements
  int lda = 0;                // a multiple of 8
  bool f32 = false;
  int rows = 0;
  // rows of A in a ring: row r is at ((ring_base + r) & ring_mask)
  int ring_base = 0, ring_mask = -1;
  GemmOut out = kOutF32;
  void *C = nullptr;
  int ldc = 0;
  int silu_channels = 0;      // kOutF32: these first channels go through silu
  GatedAct act = kActClamped; // kOutExpertAct
  float limit = 0.f;
  // Grouped form: matrix e applies to the rows listed for it.  lists[e][i] is an
  // assignment id; it reads A row id / list_div and writes C row id.
  int experts = 0;
  const int *counts = nullptr; // [experts]
  const int *lists = nullptr;  // [experts][list_cap]
  int list_cap = 0, list_div = 1, list_total = 0; // total: assignments over all experts
  int64_t expert_tiles = 0;    // 1 KiB tiles from one expert's matrix to the next
};
int launch_rows_gemm(const RowsGemm &a, hipStream_t stream);

} // namespace bh
