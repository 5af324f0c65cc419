// bf16_gemv.hip -- one activation row times resident bfloat16 matrices: the
// matrix products of a decode step.
//
// The activations stay f32 and every product is an f32 multiply-add (a bfloat16
// weight widens to f32 exactly), in both number formats: the launch is bound by
// the two bytes of each weight, not by its arithmetic.  What a decoder layer does
// between two products is the prologue of the second one: every workgroup repeats
// it on the few KiB of the row while its first weight tiles are on their way.
#include "bf16_linear.h"
#include "bf16_dev.h"

#include <algorithm>

namespace bh {
namespace {

constexpr int kRowThreads = 512, kRowWaves = kRowThreads / 64;
constexpr int kAhead = 8; // weight tiles a wavefront keeps in flight

__global__ void __launch_bounds__(256)
pack_bf16_kernel(const uint16_t *__restrict__ src, int64_t sn, int64_t sk, int N, int K, int ktiles,
                 int64_t total, uint4 *__restrict__ tiles) {
  const int64_t id = (int64_t)blockIdx.x * 256 + threadIdx.x; // one 16-byte run
  if (id >= total)
    return;
  const int lane = (int)(id & 63);
  const int64_t tile = id >> 6;
  const int64_t g = tile / ktiles;
  const int c = (int)(tile - g * ktiles);
  const int64_t n = g * 16 + (lane & 15);
  const int k0 = c * kBfTileK + (lane >> 4) * 8;
  unsigned short v[8];
  for (int j = 0; j < 8; ++j)
    v[j] = n < N && k0 + j < K ? src[n * sn + (int64_t)(k0 + j) * sk] : (unsigned short)0;
  uint4 o;
  o.x = v[0] | ((unsigned)v[1] << 16);
  o.y = v[2] | ((unsigned)v[3] << 16);
  o.z = v[4] | ((unsigned)v[5] << 16);
  o.w = v[6] | ((unsigned)v[7] << 16);
  tiles[id] = o;
}

__device__ __forceinline__ float dot_tile(const uint4 w, const float *a, float acc) {
  const f32x4 lo = *reinterpret_cast<const f32x4 *>(a), hi = *reinterpret_cast<const f32x4 *>(a + 4);
  acc = fmaf(bf_lo(w.x), lo[0], acc);
  acc = fmaf(bf_hi(w.x), lo[1], acc);
  acc = fmaf(bf_lo(w.y), lo[2], acc);
  acc = fmaf(bf_hi(w.y), lo[3], acc);
  acc = fmaf(bf_lo(w.z), hi[0], acc);
  acc = fmaf(bf_hi(w.z), hi[1], acc);
  acc = fmaf(bf_lo(w.w), hi[2], acc);
  acc = fmaf(bf_hi(w.w), hi[3], acc);
  return acc;
}

// sum over the workgroup; `red` is used once per call site
__device__ __forceinline__ float block_sum(float v, float *red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0)
    red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int w = 0; w < kRowWaves; ++w)
    s += red[w];
  return s;
}

struct RowTail { // arguments a wavefront needs only behind its first loads
  float *x_out, *row_out;
  const float *conv_w;
  float *conv_ring, *conv_next;
  const int *pos;
  const float *weight, *gate;
  float *out;
  float *max_v;
  int *max_i;
  float eps, out_gain, gain;
  int taps, silu_channels, valid;
  const float *add, *norm_w;
  GatedAct act;
  int head_dim;
};

__device__ __forceinline__ f32x4 load4(const float *p) { return *reinterpret_cast<const f32x4 *>(p); }
__device__ __forceinline__ void save4(float *p, f32x4 v) { *reinterpret_cast<f32x4 *>(p) = v; }

// What the row of this position leaves for later ones: itself in the ring, and what
// it and the rows before it will add to the next one.
__device__ __forceinline__ void keep_row(const RowTail &a, int K, int p, int i, float h) {
  a.conv_ring[(int64_t)(p % a.taps) * K + i] = h;
  float c = 0.f;
  for (int b = a.taps - 1; b >= 1; --b) {
    const int q = p + 1 - b;
    if (q < 0)
      continue;
    const float e = b == 1 ? h : a.conv_ring[(int64_t)(q % a.taps) * K + i];
    c = fmaf(a.conv_w[(int64_t)(a.taps - 1 - b) * K + i], e, c);
  }
  a.conv_next[(int64_t)((p + 1) & 1) * K + i] = c;
}

// The finished input row into act[0 .. Kp).  R > 0: K is a multiple of 4 and at most
// 2048 * R, and every thread keeps its 4 * R values in registers from one trip to
// memory.  R = 0: any K.  `keeper`: this workgroup stores what the row leaves behind.
template <int INPUT, int R>
struct RowPrologue {
  f32x4 x[R], y[R], c[2][R], w[R];
  const float *yp;
  int at[R];
  bool in[R];
  __device__ __forceinline__ void request(const float *src, const float *ysrc, const float *conv_next,
                                          int K, const RowTail &a) {
    yp = ysrc;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      at[r] = (r * kRowThreads + (int)threadIdx.x) * 4;
      in[r] = at[r] < K;
      const int i = in[r] ? at[r] : 0;
      x[r] = load4(src + i);
      if constexpr (INPUT == kRowNorm) {
        if (yp)
          y[r] = load4(yp + i);
        if (conv_next) { // both slots: which one counts depends on the position
          c[0][r] = load4(conv_next + i);
          c[1][r] = load4(conv_next + K + i);
          w[r] = load4(a.conv_w + (int64_t)(a.taps - 1) * K + i);
        }
      } else if constexpr (INPUT == kRowGated) {
        w[r] = load4(a.weight + i);
        c[0][r] = load4(a.gate + i);
      } else if constexpr (INPUT == kRowHeadGated) {
        w[r] = load4(a.weight + i % a.head_dim);
        c[0][r] = load4(a.gate + i);
      } else if constexpr (INPUT == kRowResidual) {
        if (yp)
          y[r] = load4(yp + i);
        if (a.add)
          c[0][r] = load4(a.add + i);
        w[r] = load4(a.norm_w + i);
      }
    }
  }
  __device__ __forceinline__ float squares(const f32x4 (&v)[R]) const {
    float s = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (in[r])
#pragma unroll
        for (int j = 0; j < 4; ++j)
          s = fmaf(v[r][j], v[r][j], s);
    return s;
  }
  __device__ __forceinline__ void finish(float *act, int K, int Kp, const RowTail &a, bool keeper,
                                         float (*red)[kRowWaves]) {
    if constexpr (INPUT == kRowGated) {
      const float g = 1.0f / sqrtf(block_sum(squares(x), red[0]) / (float)K + a.eps);
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          x[r][j] = x[r][j] * g * w[r][j] * sigmoid_f(c[0][r][j]);
    } else if constexpr (INPUT == kRowHeadGated) {
      // the squares of four values each meet in LDS, where the row goes afterwards
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (in[r])
          act[at[r] >> 2] = fmaf(x[r][0], x[r][0], x[r][1] * x[r][1]) + fmaf(x[r][2], x[r][2], x[r][3] * x[r][3]);
      __syncthreads();
      const int per = a.head_dim >> 2;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const float *sq = act + (in[r] ? at[r] / a.head_dim * per : 0);
        float ss = 0.f;
        for (int i = 0; i < per; ++i)
          ss += sq[i];
        const float g = 1.0f / sqrtf(ss / (float)a.head_dim + a.eps);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          x[r][j] = x[r][j] * g * w[r][j] * sigmoid_f(c[0][r][j]);
      }
      __syncthreads();
    } else if constexpr (INPUT == kRowResidual) {
#pragma unroll
      for (int r = 0; r < R; ++r) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if (yp)
            x[r][j] += y[r][j];
          if (a.add)
            x[r][j] += c[0][r][j];
        }
        if (keeper && a.x_out && in[r])
          save4(a.x_out + at[r], x[r]);
      }
      const float g = 1.0f / sqrtf(block_sum(squares(x), red[1]) / (float)K + a.eps);
#pragma unroll
      for (int r = 0; r < R; ++r) {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          x[r][j] = x[r][j] * g * w[r][j];
        if (keeper && a.row_out && in[r])
          save4(a.row_out + at[r], x[r]);
      }
    } else if constexpr (INPUT == kRowNorm) {
      if (yp) {
        const float ry = a.out_gain / sqrtf(block_sum(squares(y), red[0]) / (float)K + a.eps);
#pragma unroll
        for (int r = 0; r < R; ++r) {
#pragma unroll
          for (int j = 0; j < 4; ++j)
            x[r][j] = fmaf(y[r][j], ry, x[r][j]);
          if (keeper && a.x_out && in[r])
            save4(a.x_out + at[r], x[r]);
        }
      }
      const float g = a.gain / sqrtf(block_sum(squares(x), red[1]) / (float)K + a.eps);
      const int p = a.conv_w ? *a.pos : 0;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        f32x4 h;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          h[j] = x[r][j] * g;
        x[r] = h;
        if (a.conv_w) {
#pragma unroll
          for (int j = 0; j < 4; ++j)
            x[r][j] += fmaf(w[r][j], h[j], p == 0 ? 0.f : p & 1 ? c[1][r][j] : c[0][r][j]);
          if (keeper && in[r])
#pragma unroll
            for (int j = 0; j < 4; ++j)
              keep_row(a, K, p, at[r] + j, h[j]);
        }
        if (keeper && a.row_out && in[r])
          save4(a.row_out + at[r], x[r]);
      }
    }
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (at[r] < Kp)
        save4(act + at[r], in[r] ? x[r] : f32x4{0.f, 0.f, 0.f, 0.f});
  }
};
template <int INPUT>
struct RowPrologue<INPUT, 0> {
  const float *src, *yp;
  __device__ __forceinline__ void request(const float *s, const float *ysrc, const float *, int,
                                          const RowTail &) {
    src = s;
    yp = ysrc;
  }
  __device__ __forceinline__ void finish(float *act, int K, int Kp, const RowTail &a, bool keeper,
                                         float (*red)[kRowWaves]) {
    const int tid = threadIdx.x;
    float scale = 1.f;
    if constexpr (INPUT == kRowPlain) {
      for (int i = tid; i < K; i += kRowThreads)
        act[i] = src[i];
    } else if constexpr (INPUT == kRowHeadGated) {
      float *scales = act + Kp; // [heads]
      for (int h = tid >> 6; h * a.head_dim < K; h += kRowWaves) {
        float ss = 0.f;
        for (int i = tid & 63; i < a.head_dim; i += 64)
          ss = fmaf(src[h * a.head_dim + i], src[h * a.head_dim + i], ss);
        ss = wave_sum(ss);
        if ((tid & 63) == 0)
          scales[h] = 1.0f / sqrtf(ss / (float)a.head_dim + a.eps);
      }
      __syncthreads();
      for (int i = tid; i < K; i += kRowThreads)
        act[i] = src[i] * scales[i / a.head_dim] * a.weight[i % a.head_dim];
    } else {
      float ry = 0.f, ss = 0.f;
      if (INPUT == kRowNorm && yp) {
        for (int i = tid; i < K; i += kRowThreads)
          ss = fmaf(yp[i], yp[i], ss);
        ry = a.out_gain / sqrtf(block_sum(ss, red[0]) / (float)K + a.eps);
      }
      ss = 0.f;
      for (int i = tid; i < K; i += kRowThreads) {
        float v = src[i];
        if (INPUT == kRowNorm && yp) {
          v = fmaf(yp[i], ry, v);
          if (keeper && a.x_out)
            a.x_out[i] = v;
        }
        if constexpr (INPUT == kRowResidual) {
          if (yp)
            v += yp[i];
          if (a.add)
            v += a.add[i];
          if (keeper && a.x_out)
            a.x_out[i] = v;
        }
        act[i] = v;
        ss = fmaf(v, v, ss);
      }
      scale = (INPUT == kRowNorm ? a.gain : 1.0f) / sqrtf(block_sum(ss, red[1]) / (float)K + a.eps);
    }
    const int p = INPUT == kRowNorm && a.conv_w ? *a.pos : 0;
    for (int i = tid; i < Kp; i += kRowThreads) {
      float h = 0.f;
      if (i < K) {
        h = act[i] * scale;
        if constexpr (INPUT == kRowGated)
          h *= a.weight[i] * sigmoid_f(a.gate[i]);
        if constexpr (INPUT == kRowHeadGated)
          h *= sigmoid_f(a.gate[i]);
        if constexpr (INPUT == kRowResidual) {
          h *= a.norm_w[i];
          if (keeper && a.row_out)
            a.row_out[i] = h;
        }
        if constexpr (INPUT == kRowNorm) {
          if (a.conv_w) {
            const float raw = h;
            h += fmaf(a.conv_w[(int64_t)(a.taps - 1) * K + i], raw,
                      p > 0 ? a.conv_next[(int64_t)(p & 1) * K + i] : 0.f);
            if (keeper)
              keep_row(a, K, p, i, raw);
          }
          if (keeper && a.row_out)
            a.row_out[i] = h;
        }
      }
      act[i] = h;
    }
  }
};

// Grid: workgroups of 8 wavefronts = (8 >> ks_shift) channel groups x (1 <<
// ks_shift) slices of k that meet in LDS in slice order.  kRowNorm, kRowResidual: one
// workgroup more, which multiplies nothing and stores what the row leaves behind.
// GATED: neighbouring channel groups are group i of one matrix and of the other.
template <int INPUT, int R, bool GATED>
__global__ void __launch_bounds__(kRowThreads)
row_gemv_kernel(const uint4 *__restrict__ W, const float *__restrict__ src,
                const float *__restrict__ y, const float *conv_next, int K, int ktiles, int groups,
                int ks_shift, int slice_tiles, RowTail a) {
  extern __shared__ __attribute__((aligned(16))) float act[]; // [Kp]
  __shared__ float red[2][kRowWaves];
  __shared__ float part[kRowWaves][16];
  const int Kp = ktiles * kBfTileK;
  const int tid = threadIdx.x, lane = tid & 63;
  // the row's values first: loads return in order, and these come from the L2
  RowPrologue<INPUT, R> row;
  row.request(src, y, conv_next, K, a);
  if ((INPUT == kRowNorm || INPUT == kRowResidual) && blockIdx.x == gridDim.x - 1) {
    row.finish(act, K, Kp, a, true, red);
    return;
  }
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int slice = wave & ((1 << ks_shift) - 1);
  const int g = blockIdx.x * (kRowWaves >> ks_shift) + (wave >> ks_shift);
  const int gl = min(g, groups - 1); // a wavefront past the last group repeats it and stores nothing
  const int t0 = slice * slice_tiles, t1 = min(t0 + slice_tiles, ktiles);
  const uint4 *wp = W + (int64_t)(GATED ? (gl & 1) * (groups >> 1) + (gl >> 1) : gl) * ktiles * 64 + lane;
  uint4 w[kAhead];
#pragma unroll
  for (int u = 0; u < kAhead; ++u)
    w[u] = wp[(int64_t)min(t0 + u, ktiles - 1) * 64];
  row.finish(act, K, Kp, a, false, red);
  __syncthreads();

  const float *ap = act + (lane >> 4) * 8;
  float acc = 0.f;
  for (int t = t0; t < t1; t += kAhead) {
    uint4 n[kAhead];
    const bool more = t + kAhead < t1;
    if (more) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        n[u] = wp[(int64_t)min(t + kAhead + u, ktiles - 1) * 64];
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u)
      if (t + u < t1)
        acc = dot_tile(w[u], ap + (t + u) * kBfTileK, acc);
    if (more) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        w[u] = n[u];
    }
  }
  acc = sum_rows(acc);
  if (lane < 16)
    part[wave][lane] = acc;
  __syncthreads();
  const int gi = tid >> 4;
  if constexpr (GATED) {
    if (gi < (kRowWaves >> ks_shift) / 2) {
      const int go = blockIdx.x * ((kRowWaves >> ks_shift) / 2) + gi;
      float vg = 0.f, vu = 0.f;
      for (int s = 0; s < (1 << ks_shift); ++s) {
        vg += part[((2 * gi) << ks_shift) + s][tid & 15];
        vu += part[((2 * gi + 1) << ks_shift) + s][tid & 15];
      }
      if (go < groups / 2)
        a.out[go * 16 + (tid & 15)] = gated_act(a.act, vg, vu, 0.f);
    }
    return;
  }
  if (gi < (kRowWaves >> ks_shift)) {
    const int go = blockIdx.x * (kRowWaves >> ks_shift) + gi;
    float v = 0.f;
    for (int s = 0; s < (1 << ks_shift); ++s)
      v += part[(gi << ks_shift) + s][tid & 15];
    const int n = go * 16 + (tid & 15);
    if (n < a.silu_channels)
      v = silu_f(v);
    if (go < groups)
      a.out[n] = v;
    if (a.max_v) {
      const bool ok = go < groups && n < a.valid;
      const float m = row16_max(ok ? v : -INFINITY);
      const unsigned long long hit = __ballot(ok && v == m);
      const unsigned mine = (unsigned)(hit >> (lane & 48)) & 0xffffu;
      if ((tid & 15) == 0 && go < groups) {
        a.max_v[go] = mine ? m : -INFINITY;
        a.max_i[go] = mine ? go * 16 + __builtin_ctz(mine) : 0x7fffffff;
      }
    }
  }
}

// ---- experts of one row ----------------------------------------------------------

__device__ __forceinline__ unsigned order_key(float f) {
  const unsigned u = __float_as_uint(f);
  return u & 0x80000000u ? ~u : u | 0x80000000u;
}

// The `rank`-th largest of `count` logits (0 = the largest; equal ones by index),
// found by every wavefront for itself: R values per lane.
template <int R>
__device__ __forceinline__ int pick_expert(const float *__restrict__ logits, int count, int rank,
                                           float &value) {
  const int lane = threadIdx.x & 63;
  unsigned key[R];
  float val[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = r * 64 + lane;
    val[r] = logits[min(i, count - 1)];
    key[r] = i < count ? max(order_key(val[r]), 1u) : 0u;
  }
  int idx = 0;
  for (int it = 0; it <= rank; ++it) {
    unsigned best = key[0];
#pragma unroll
    for (int r = 1; r < R; ++r)
      best = max(best, key[r]);
    const unsigned m = wave_max_u32(best);
    idx = -1;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const unsigned long long b = __ballot(key[r] == m);
      if (idx < 0 && b) {
        const int l = __builtin_ctzll(b);
        idx = r * 64 + l;
        value = lane_f(val[r], l);
        if (lane == l)
          key[r] = 0;
      }
    }
  }
  return idx;
}

struct MoeGateUp {
  const uint4 *gate_up, *shared_gate_up;
  int ktiles, groups, shared_groups; // of one matrix
  int experts, top, width;
  float limit, shared_limit;
  float *act;
  int act_stride;
  int *chosen;
  float *chosen_logit;
};

// Grid (channel groups, top + shared): 8 wavefronts = gate and up of
// (4 >> ks_shift) channel groups x (1 << ks_shift) slices of k.
template <int R>
__global__ void __launch_bounds__(kRowThreads)
moe_gate_up_kernel(const float *__restrict__ h, const float *__restrict__ logits, int ks_shift,
                   int slice_tiles, MoeGateUp a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float part[kRowWaves][16];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int per = (kRowWaves / 2) >> ks_shift;
  const int slot = blockIdx.y;
  const bool is_shared = slot >= a.top;
  const int groups = is_shared ? a.shared_groups : a.groups;
  if ((int)blockIdx.x * per >= groups)
    return;
  const int Kp = a.ktiles * kBfTileK;
  for (int i = tid; i < Kp; i += kRowThreads)
    lds[i] = i < a.width ? h[i] : 0.f;
  const uint4 *W = a.shared_gate_up;
  if (!is_shared) {
    float z = 0.f;
    const int e = __builtin_amdgcn_readfirstlane(pick_expert<R>(logits, a.experts, slot, z));
    W = a.gate_up + (int64_t)e * 2 * a.groups * a.ktiles * 64;
    if (blockIdx.x == 0 && tid == 0) {
      a.chosen[slot] = e;
      a.chosen_logit[slot] = z;
    }
  }
  const int mat = wave & 1, slice = (wave >> 1) & ((1 << ks_shift) - 1);
  const int g = blockIdx.x * per + (wave >> (1 + ks_shift)), gl = min(g, groups - 1);
  const int t0 = slice * slice_tiles, t1 = min(t0 + slice_tiles, a.ktiles);
  const uint4 *wp = W + (int64_t)(mat * groups + gl) * a.ktiles * 64 + lane;
  uint4 w[kAhead];
#pragma unroll
  for (int u = 0; u < kAhead; ++u)
    w[u] = wp[(int64_t)min(t0 + u, a.ktiles - 1) * 64];
  __syncthreads();
  const float *ap = lds + (lane >> 4) * 8;
  float acc = 0.f;
  for (int t = t0; t < t1; t += kAhead) {
    uint4 n[kAhead];
    const bool more = t + kAhead < t1;
    if (more) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        n[u] = wp[(int64_t)min(t + kAhead + u, a.ktiles - 1) * 64];
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u)
      if (t + u < t1)
        acc = dot_tile(w[u], ap + (t + u) * kBfTileK, acc);
    if (more) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        w[u] = n[u];
    }
  }
  acc = sum_rows(acc);
  if (lane < 16)
    part[wave][lane] = acc;
  __syncthreads();
  const int gi = tid >> 4;
  if (gi < per) {
    const int go = blockIdx.x * per + gi;
    float vg = 0.f, vu = 0.f;
    for (int s = 0; s < (1 << ks_shift); ++s) {
      const int wv = (gi << (1 + ks_shift)) + 2 * s;
      vg += part[wv][tid & 15];
      vu += part[wv + 1][tid & 15];
    }
    if (go < groups)
      a.act[(int64_t)slot * a.act_stride + go * 16 + (tid & 15)] =
          expert_act(vg, vu, is_shared ? a.shared_limit : a.limit);
  }
}

struct MoeDown {
  const uint4 *shared_down;
  int groups;                  // channel groups of the output
  int top, ktiles, shared_ktiles;
  int act_stride;
  const float *chosen_logit;
  float *out;
};

// Grid: one channel group (HALF: 8 of its 16 channels) per workgroup; its wavefronts
// cut the concatenation of the chosen experts' k (and the shared expert's) into
// slices.  With HALF a load covers the 8 channels of two consecutive tiles, so it
// still moves whole 128-byte lines; every expert has an even number of tiles.
template <int WAVES, bool HALF>
__global__ void __launch_bounds__(WAVES * 64)
moe_down_kernel(const uint4 *__restrict__ down, const float *__restrict__ act,
                const int *__restrict__ chosen, int slice_tiles, MoeDown a) {
  __shared__ float part[WAVES][16];
  constexpr int kStep = HALF ? 2 : 1; // tiles per load
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int g = HALF ? blockIdx.x >> 1 : blockIdx.x, half = HALF ? blockIdx.x & 1 : 0;
  // this lane's 16 bytes of a load and the k they hold
  const int run = HALF ? (lane >> 5) * 64 + ((lane >> 3) & 3) * 16 + half * 8 + (lane & 7) : lane;
  const int k_at = HALF ? (lane >> 5) * kBfTileK + ((lane >> 3) & 3) * 8 : (lane >> 4) * 8;
  // lane j: the j-th chosen expert and its softmax weight
  const int cj = a.top > 0 ? chosen[min(lane, a.top - 1)] : 0;
  const float zj = lane < a.top ? a.chosen_logit[lane] : -INFINITY;
  const float most = wave_max(zj); // with all lanes, not under the condition below
  const float ej = lane < a.top ? expf(zj - most) : 0.f;
  const float wj = ej / wave_sum(ej);

  const int routed = a.top * a.ktiles, total = routed + a.shared_ktiles;
  const int t0 = min(wave * slice_tiles, total), t1 = min(t0 + slice_tiles, total);
  // walks the tiles of the concatenation: segment, tile inside it
  int seg = t0 < routed ? t0 / a.ktiles : a.top;
  int off = t0 < routed ? t0 - seg * a.ktiles : t0 - routed;
  int left = t1 - t0;
  float acc = 0.f;
  while (left > 0) {
    const bool sh = seg >= a.top;
    const int kt = sh ? a.shared_ktiles : a.ktiles;
    const int n = min(left, kt - off);
    const int e = sh ? 0 : __builtin_amdgcn_readlane(cj, min(seg, 63));
    const float wt = sh ? 1.0f : lane_f(wj, min(seg, 63));
    const uint4 *wp = (sh ? a.shared_down : down + (int64_t)e * a.groups * kt * 64) +
                      ((int64_t)g * kt + off) * 64 + run;
    const float *ap = act + (int64_t)seg * a.act_stride + off * kBfTileK + k_at;
    float s = 0.f;
    for (int t = 0; t < n; t += kAhead * kStep) {
      uint4 w[kAhead];
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        w[u] = wp[(int64_t)min(t + u * kStep, n - kStep) * 64];
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        if (t + u * kStep < n)
          s = dot_tile(w[u], ap + (t + u * kStep) * kBfTileK, s);
    }
    acc = fmaf(wt, s, acc);
    left -= n;
    off = 0;
    ++seg;
  }
  acc = sum_rows(acc);
  if constexpr (HALF)
    acc += __shfl_xor(acc, 8, 64);
  if (lane < (HALF ? 8 : 16))
    part[wave][lane] = acc;
  __syncthreads();
  if (tid < (HALF ? 8 : 16)) {
    float v = 0.f;
#pragma unroll
    for (int s = 0; s < WAVES; ++s)
      v += part[s][tid];
    a.out[g * 16 + half * 8 + tid] = v;
  }
}

// slices start at even tiles
int down_slice(int total, int waves) { return (int)round_up(ceil_div(total, waves), 2); }

int shift_for(int v) {
  int s = 0;
  while ((1 << (s + 1)) <= v)
    ++s;
  return s;
}

} // namespace

int launch_pack_bf16(const uint16_t *src, int64_t stride_n, int64_t stride_k, int64_t N, int64_t K,
                     void *tiles, hipStream_t stream) {
  BH_REQUIRE(src && tiles && N > 0 && K > 0, "pack_bf16: bad argument");
  const int64_t total = (int64_t)bf16_tiles_bytes(K, N) / 16;
  hipLaunchKernelGGL(pack_bf16_kernel, dim3((unsigned)ceil_div(total, 256)), dim3(256), 0, stream,
                     src, stride_n, stride_k, (int)N, (int)K, bf16_ktiles(K), total,
                     static_cast<uint4 *>(tiles));
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_row_gemv(const RowGemv &a, hipStream_t stream) {
  const Bf16Matrix &W = a.W;
  BH_REQUIRE(W.tiles && W.K > 0 && W.N > 0 && W.N % 16 == 0 && W.ktiles == bf16_ktiles(W.K) &&
                 a.src && a.out,
             "row_gemv: bad argument");
  BH_REQUIRE(!a.conv_w || (a.conv_ring && a.conv_next && a.pos && a.taps > 0),
             "row_gemv: convolution operands");
  BH_REQUIRE((a.input != kRowGated && a.input != kRowHeadGated) || (a.weight && a.gate), "row_gemv: gate operands");
  BH_REQUIRE(a.input != kRowHeadGated || (a.head_dim > 0 && W.K % a.head_dim == 0), "row_gemv: heads of %d values",
             a.head_dim);
  BH_REQUIRE(a.x_out == nullptr || a.x_out != a.src, "row_gemv: the row is read by every workgroup");
  BH_REQUIRE(!a.max_v || a.max_i, "row_gemv: maxima without indices");
  BH_REQUIRE(a.input != kRowResidual || a.norm_w, "row_gemv: no norm weight");
  BH_REQUIRE(!a.gated || (a.input == kRowResidual && W.N % 32 == 0 && !a.max_v && a.act == kActGeluTanh),
             "row_gemv: gated form");
  if (a.input == kRowPlain && a.src_padded && !a.silu_channels && !a.max_v && ((uintptr_t)a.src & 15) == 0 &&
      W.ktiles >= 64 && (W.groups() < 192 || W.ktiles > 256)) {
    // a long row and few channels: as many slices of k as the experts' down product takes
    MoeDown d{W.tiles, W.groups(), 0, 1, W.ktiles, 0, nullptr, a.out};
    if (W.groups() < 192)
      hipLaunchKernelGGL((moe_down_kernel<16, true>), dim3(2 * W.groups()), dim3(1024), 0, stream,
                         (const uint4 *)nullptr, a.src, (const int *)nullptr, down_slice(W.ktiles, 16), d);
    else
      hipLaunchKernelGGL((moe_down_kernel<16, false>), dim3(W.groups()), dim3(1024), 0, stream,
                         (const uint4 *)nullptr, a.src, (const int *)nullptr, down_slice(W.ktiles, 16), d);
    BH_CHECK_HIP(hipGetLastError());
    return BUDDY_HIP_OK;
  }
  // slices of k: doubled while the launch has fewer than 2048 wavefronts and each
  // keeps four tiles
  const int groups = W.groups();
  int ks = 1;
  while (ks < (a.gated ? kRowWaves / 2 : kRowWaves) && (int64_t)groups * ks < 2048 && W.ktiles / (2 * ks) >= 4)
    ks *= 2;
  const int shift = shift_for(ks), per = kRowWaves >> shift;
  const int slice_tiles = (int)ceil_div(W.ktiles, ks);
  const size_t lds = sizeof(float) * ((size_t)W.ktiles * kBfTileK + (a.head_dim ? W.K / a.head_dim : 0));
  BH_REQUIRE(lds <= 150 * 1024, "row_gemv: a row of %d values does not fit LDS", W.K);
  RowTail t{a.x_out, a.row_out, a.conv_w, a.conv_ring, a.conv_next, a.pos, a.weight, a.gate,
            a.out, a.max_v, a.max_i, a.eps, a.out_gain, a.gain, a.taps, a.silu_channels, a.valid,
            a.add, a.norm_w, a.act, a.head_dim};
  const bool keeper = a.input == kRowNorm || a.input == kRowResidual;
  const dim3 grid((unsigned)(ceil_div(groups, per) + keeper)), block(kRowThreads);
  bool quads = W.K % 4 == 0 && a.head_dim % 4 == 0;
  for (const void *p : {(const void *)a.src, (const void *)a.y, (const void *)a.x_out,
                        (const void *)a.row_out, (const void *)a.conv_w, (const void *)a.conv_next,
                        (const void *)a.weight, (const void *)a.gate, (const void *)a.add,
                        (const void *)a.norm_w})
    quads = quads && ((uintptr_t)p & 15) == 0;
  const int span = W.ktiles * kBfTileK; // the padding is written too
  const int regs = !quads || span > 8192 ? 0 : span <= 2048 ? 1 : span <= 4096 ? 2 : 4;
#define BH_ROW(I, R, G)                                                                          \
  do {                                                                                           \
    static DynLdsOnce once;                                                                      \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)row_gemv_kernel<I, R, G>, 150 * 1024));       \
    hipLaunchKernelGGL((row_gemv_kernel<I, R, G>), grid, block, lds, stream, W.tiles, a.src, a.y,\
                       a.conv_w ? a.conv_next : nullptr, W.K, W.ktiles, groups, shift,           \
                       slice_tiles, t);                                                          \
  } while (0)
#define BH_ROWS(I, G)                                                                            \
  do {                                                                                           \
    if (regs == 1)                                                                               \
      BH_ROW(I, 1, G);                                                                           \
    else if (regs == 2)                                                                          \
      BH_ROW(I, 2, G);                                                                           \
    else if (regs == 4)                                                                          \
      BH_ROW(I, 4, G);                                                                           \
    else                                                                                         \
      BH_ROW(I, 0, G);                                                                           \
  } while (0)
  if (a.input == kRowPlain)
    BH_ROWS(kRowPlain, false);
  else if (a.input == kRowNorm)
    BH_ROWS(kRowNorm, false);
  else if (a.input == kRowGated)
    BH_ROWS(kRowGated, false);
  else if (a.input == kRowHeadGated)
    BH_ROWS(kRowHeadGated, false);
  else if (a.gated)
    BH_ROWS(kRowResidual, true);
  else
    BH_ROWS(kRowResidual, false);
#undef BH_ROWS
#undef BH_ROW
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_row_moe(const RowMoe &a, hipStream_t stream) {
  BH_REQUIRE(a.h && a.logits && a.width > 0 && a.act && a.chosen && a.weights && a.out &&
                 a.experts.gate_up && a.experts.down && a.experts.count > 0 &&
                 a.experts.count <= kMaxExperts && a.top > 0 && a.top <= 64 &&
                 a.top <= a.experts.count && a.experts.ff > 0,
             "row_moe: bad argument");
  const bool shared = a.shared.count > 0;
  BH_REQUIRE(!shared || (a.shared.gate_up && a.shared.down && a.shared.ff > 0),
             "row_moe: shared expert");
  MoeGateUp u{};
  u.gate_up = a.experts.gate_up;
  u.shared_gate_up = a.shared.gate_up;
  u.ktiles = bf16_ktiles(a.width);
  u.groups = (int)ceil_div(a.experts.ff, 16);
  u.shared_groups = shared ? (int)ceil_div(a.shared.ff, 16) : 0;
  u.experts = a.experts.count;
  u.top = a.top;
  u.width = a.width;
  u.limit = a.experts.limit;
  u.shared_limit = a.shared.limit;
  u.act = a.act;
  u.act_stride = a.act_stride;
  u.chosen = a.chosen;
  u.chosen_logit = a.weights;
  BH_REQUIRE(a.act_stride >= 64 * ceil_div(std::max(a.experts.ff, shared ? a.shared.ff : 0), 64),
             "row_moe: activation rows too short");
  int ks = 1;
  while (ks < kRowWaves / 2 && u.ktiles / (2 * ks) >= 4)
    ks *= 2;
  const int shift = shift_for(ks), per = (kRowWaves / 2) >> shift;
  const size_t lds = sizeof(float) * (size_t)u.ktiles * kBfTileK;
  BH_REQUIRE(lds <= 150 * 1024, "row_moe: a row of %d values does not fit LDS", a.width);
  const dim3 grid((unsigned)ceil_div(std::max(u.groups, u.shared_groups), per),
                  (unsigned)(a.top + (shared ? 1 : 0)));
  const int slice_tiles = (int)ceil_div(u.ktiles, ks);
#define BH_GU(R)                                                                                \
  do {                                                                                          \
    static DynLdsOnce once;                                                                     \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)moe_gate_up_kernel<R>, 150 * 1024));        \
    hipLaunchKernelGGL(moe_gate_up_kernel<R>, grid, dim3(kRowThreads), lds, stream, a.h,        \
                       a.logits, shift, slice_tiles, u);                                        \
  } while (0)
  if (a.experts.count <= 64)
    BH_GU(1);
  else
    BH_GU(kMaxExperts / 64);
#undef BH_GU
  BH_CHECK_HIP(hipGetLastError());
  MoeDown d{};
  d.shared_down = a.shared.down;
  d.groups = (int)ceil_div(a.width, 16);
  d.top = a.top;
  d.ktiles = bf16_ktiles(a.experts.ff);
  d.shared_ktiles = shared ? bf16_ktiles(a.shared.ff) : 0;
  d.act_stride = a.act_stride;
  d.chosen_logit = a.weights;
  d.out = a.out;
  const int total = a.top * d.ktiles + d.shared_ktiles;
  auto slice = [&](int waves) { return down_slice(total, waves); };
  if (total >= 64 && d.groups < 192) // fewer workgroups than compute units: halves
    hipLaunchKernelGGL((moe_down_kernel<16, true>), dim3(2 * d.groups), dim3(1024), 0, stream,
                       a.experts.down, a.act, a.chosen, slice(16), d);
  else if (total >= 64)
    hipLaunchKernelGGL((moe_down_kernel<16, false>), dim3(d.groups), dim3(1024), 0, stream,
                       a.experts.down, a.act, a.chosen, slice(16), d);
  else
    hipLaunchKernelGGL((moe_down_kernel<4, false>), dim3(d.groups), dim3(256), 0, stream,
                       a.experts.down, a.act, a.chosen, slice(4), d);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

} // namespace bh

extern "C" {

size_t buddy_hip_bf16_tiles_bytes(int64_t K, int64_t N) {
  return K > 0 && N > 0 ? bh::bf16_tiles_bytes(K, N) : 0;
}

int buddy_hip_pack_bf16_tiles(const uint16_t *W, int64_t K, int64_t N, void *tiles,
                              buddy_hip_stream stream) try {
  BH_REQUIRE(K < (1 << 30) && N < (1 << 30), "pack_bf16_tiles: bad size");
  return bh::launch_pack_bf16(W, K, 1, N, K, tiles, bh::as_stream(stream));
} BH_CATCH_INT("buddy_hip_pack_bf16_tiles")

int buddy_hip_gemv_bf16(const float *x, const void *tiles, float *y, int64_t K, int64_t N,
                        buddy_hip_stream stream) try {
  BH_REQUIRE(K > 0 && N > 0 && K < (1 << 30) && N < (1 << 30), "gemv_bf16: bad size");
  bh::RowGemv g;
  g.W.tiles = static_cast<const uint4 *>(tiles);
  g.W.K = (int)K;
  g.W.N = (int)bh::round_up(N, 16);
  g.W.ktiles = bh::bf16_ktiles(K);
  g.src = x;
  g.out = y;
  return bh::launch_row_gemv(g, bh::as_stream(stream));
} BH_CATCH_INT("buddy_hip_gemv_bf16")
}
