// flash_tile.h -- attention of a prompt, tile by tile: what a wavefront does with a tile
// of keys and values that lies in LDS.
#pragma once

#include "bf16_dev.h"

namespace bh {

// Keys of a tile: 128 bytes of a V^T row.
template <typename T> struct KeyTile {
  static constexpr int kKeys = 128 / (int)sizeof(T);
};

#if defined(__HIPCC__)
// A wavefront owns 16 queries.  S^T = K . Q^T leaves a lane with keys of one query, which
// is the B operand of O^T += V^T . P^T as it lies (of 32 keys in bfloat16: a lane's eight
// are keys 4q .. 4q + 3 of both halves, and V^T rows are stored in that order).  NK:
// 32-element steps of a key, NV: 16-channel groups of a value.
//
// The running maximum a lane subtracts follows the scores only when one exceeds it by
// more than kSlack: the weights stay below e^kSlack, and the sums are rescaled a few
// times per query instead of once per tile.  The softmax weights of the bfloat16 form
// are multiplied as two bfloat16 terms each (17 bits).
template <typename T, int NK, int NV> struct Flash {
  static constexpr int E = 16 / (int)sizeof(T), KEYS = KeyTile<T>::kKeys, SUB = KEYS / 16;
  static constexpr int kKeyRow = NK * 32 + E, kValueRow = KEYS + E; // rows start 4 banks apart
  static constexpr float kSlack = 8.0f;

  f32x4 o[NV];
  float m = -INFINITY, l = 0.f; // l: this lane's share
  __device__ __forceinline__ Flash() {
#pragma unroll
    for (int v = 0; v < NV; ++v)
      o[v] = f32x4{0.f, 0.f, 0.f, 0.f};
  }

  // where run c (16 bytes) of channel r of a V^T tile goes, and its store
  static __device__ __forceinline__ int value_at(int r, int c) {
    return r * kValueRow + (sizeof(T) == 2 ? (c >> 2) * 32 + (c & 1) * 16 + ((c >> 1) & 1) * 4 : c * E);
  }
  static __device__ __forceinline__ void store_value(T *vt, int at, u32x4 v) {
    if constexpr (sizeof(T) == 2) {
      *reinterpret_cast<uint2 *>(vt + at) = uint2{v[0], v[1]};
      *reinterpret_cast<uint2 *>(vt + at + 8) = uint2{v[2], v[3]};
    } else {
      *reinterpret_cast<u32x4 *>(vt + at) = v;
    }
  }

  // kt: [KEYS][kKeyRow], vt: [16 * NV][kValueRow].  gap0: this lane's query minus the
  // tile's first key; a key is seen when 0 <= gap < window.  `whole`: all of them are.
  __device__ __forceinline__ void tile(const T *kt, const T *vt, const Frag<T> (&qf)[NK], bool whole,
                                       int gap0, int window) {
    const int lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
    f32x4 s[SUB];
#pragma unroll
    for (int b = 0; b < SUB; ++b)
      s[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    // the fragments of the next step are read while this one is multiplied
    const T *kp = kt + col * kKeyRow + quad * 8;
    Frag<T> kf[2][SUB];
#pragma unroll
    for (int b = 0; b < SUB; ++b)
      kf[0][b].load(kp + b * 16 * kKeyRow);
#pragma unroll
    for (int t = 0; t < NK; ++t) {
      if (t + 1 < NK) {
#pragma unroll
        for (int b = 0; b < SUB; ++b)
          kf[(t + 1) & 1][b].load(kp + b * 16 * kKeyRow + (t + 1) * 32);
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int b = 0; b < SUB; ++b)
        s[b] = mfma32(kf[t & 1][b], qf[t], s[b]);
      __builtin_amdgcn_sched_barrier(0);
    }
    if (!whole) {
#pragma unroll
      for (int b = 0; b < SUB; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int gap = gap0 - (b * 16 + quad * 4 + r);
          s[b][r] = gap >= 0 && gap < window ? s[b][r] : -INFINITY;
        }
    }
    float mt = s[0][0];
#pragma unroll
    for (int b = 0; b < SUB; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        mt = fmaxf(mt, s[b][r]);
    float x, y;
    lane_pair<16>(mt, x, y);
    mt = fmaxf(x, y);
    lane_pair<32>(mt, x, y);
    mt = fmaxf(x, y);
    if (__any(mt > m + kSlack)) { // -inf + kSlack stays below every score
      mt = fmaxf(mt, m);
      const float alpha = mt == -INFINITY ? 1.f : fast_exp(m - mt);
      m = mt;
      l *= alpha;
#pragma unroll
      for (int v = 0; v < NV; ++v)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          o[v][r] *= alpha;
    }
    const float base = m == -INFINITY ? 0.f : m; // nothing visible so far
#pragma unroll
    for (int b = 0; b < SUB; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[b][r] = fast_exp(s[b][r] - base);
        l += s[b][r];
      }
    if constexpr (sizeof(T) == 2) {
      // the weights as two bfloat16 terms
      uint4 hi[SUB / 2], lo[SUB / 2];
#pragma unroll
        for (int b = 0; b < SUB / 2; ++b) {
          unsigned ph[4], pl[4];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const f32x4 &x = s[2 * b + (j >> 1)];
            const float x0 = x[2 * (j & 1)], x1 = x[2 * (j & 1) + 1];
            ph[j] = pack_bf(x0, x1);
            pl[j] = pack_bf(x0 - bf_lo(ph[j]), x1 - bf_hi(ph[j]));
          }
          hi[b] = uint4{ph[0], ph[1], ph[2], ph[3]};
          lo[b] = uint4{pl[0], pl[1], pl[2], pl[3]};
        }
      constexpr int G = NV < 4 ? NV : 4; // value tiles read ahead
      const T *vp = vt + col * kValueRow + quad * 8;
      Frag<T> vf[2][G][SUB / 2];
#pragma unroll
      for (int v = 0; v < G; ++v)
#pragma unroll
        for (int b = 0; b < SUB / 2; ++b)
          vf[0][v][b].load(vp + v * 16 * kValueRow + b * 32);
#pragma unroll
      for (int v0 = 0; v0 < NV; v0 += G) {
        if (v0 + G < NV) {
#pragma unroll
          for (int v = 0; v < G; ++v)
#pragma unroll
            for (int b = 0; b < SUB / 2; ++b)
              vf[(v0 / G + 1) & 1][v][b].load(vp + (v0 + G + v) * 16 * kValueRow + b * 32);
        }
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int b = 0; b < SUB / 2; ++b) {
#pragma unroll
          for (int v = 0; v < G; ++v)
            o[v0 + v] = mfma_bf16(vf[(v0 / G) & 1][v][b].v, hi[b], o[v0 + v]);
#pragma unroll
          for (int v = 0; v < G; ++v)
            o[v0 + v] = mfma_bf16(vf[(v0 / G) & 1][v][b].v, lo[b], o[v0 + v]);
        }
        __builtin_amdgcn_sched_barrier(0);
      }
    } else {
#pragma unroll
      for (int v = 0; v < NV; ++v)
#pragma unroll
        for (int b = 0; b < SUB; ++b) {
          const f32x4 vv = *reinterpret_cast<const f32x4 *>(vt + (v * 16 + col) * kValueRow + b * 16 + quad * 4);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[v] = mfma_f32(vv[r], s[b][r], o[v]);
        }
    }
  }
};
#endif

} // namespace bh
