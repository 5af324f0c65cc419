// head_attn.hip -- attention over per-head keys and values.  A token: partials over
// chunks of the visible keys, then their fold; a prompt: cache rows and queries, a flash
// attention over tiles of keys, and for two maps or a gate a pass that combines them.
//
// Scores, softmax and sums are f32.  A token's products are f32 throughout.  Of a prompt
// the products take their operands in the cache's format.
#include "head_attn.h"
#include "bf16_dev.h"
#include "flash_tile.h"
#include "rotary.h"

#include <algorithm>
#include <climits>

namespace bh {
namespace {

constexpr int kTile = kHeadKeyTile;

// coordinate i of the rotated head that lies at v; cs: [cos | sin] of the pairs
__device__ __forceinline__ float turned(const float *v, int i, int half, const float *cs) {
  if (i >= 2 * half)
    return v[i];
  const int f = i < half ? i : i - half;
  const float u = v[f], w = v[f + half], c = cs[f], s = cs[half + f];
  return i < half ? u * c - w * s : w * c + u * s;
}
template <typename T> __device__ __forceinline__ float as_stored(float v) {
  return sizeof(T) == 2 ? bf_f(f_bf(v)) : v;
}
template <typename T> __device__ __forceinline__ Frag<float> widened(const Frag<T> &f) {
  if constexpr (sizeof(T) == 2)
    return widen(f.v);
  else
    return f;
}
__device__ __forceinline__ void store_quad(float *p, f32x4 v) { *reinterpret_cast<f32x4 *>(p) = v; }
__device__ __forceinline__ void store_quad(bf16_bits *p, f32x4 v) {
  *reinterpret_cast<uint2 *>(p) = uint2{pack_bf(v[0], v[1]), pack_bf(v[2], v[3])};
}
__device__ __forceinline__ void set_elem(Frag<float> &f, int j, float v) {
  if (j < 4)
    f.lo[j] = v;
  else
    f.hi[j - 4] = v;
}

struct HeadPartArgs {
  int group, maps, dim, vdim, half; // group: query heads per key / value head
  int window, ring_mask, rows, tiles; // tiles: key tiles of a chunk
  int q_at, k_at, v_at, map_heads;
  float scale, rot_gain;
  float *acc, *ml;
};

// Grid (chunks, kv_heads * maps, query heads of a group / 16).  Four wavefronts: each
// scores 16 of a tile's 64 keys against up to 16 query heads, then takes its share of
// the value channels.  S^T = K . Q^T and O^T = V^T . P^T on the f32 matrix cores.  The
// workgroups that hold the new position's tile take its key and value from the
// projections, and one of them stores them.  NV: channel groups per wavefront, at most.
template <typename T, int NV>
__global__ void __launch_bounds__(256)
head_part_kernel(const float *__restrict__ proj, T *__restrict__ keys, T *__restrict__ values_t,
                 const double *__restrict__ turns, const int *__restrict__ pos, int dim32, int vdim16,
                 HeadPartArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int qrow = dim32 + 4;
  float *qs = lds;                  // [16][qrow]: queries, rotated and scaled
  float *nk = qs + 16 * qrow;       // [dim32]: the new key
  float *nv = nk + dim32;           // [vdim16]: the new value
  float *cs = nv + vdim16;          // [2 * half]
  float *sp = cs + ((2 * a.half + 3) & ~3); // [64][17]: scores
  const int gm = blockIdx.y, g = gm / a.maps, map = gm - g * a.maps;
  const int q0 = blockIdx.z * 16, nq = min(16, a.group - q0);
  T *kc = keys + (int64_t)gm * a.rows * dim32;
  T *vc = values_t + (int64_t)g * vdim16 * a.rows;
  const int p = *pos;
  const int lo = max(0, p - a.window + 1);
  const int first = (lo & ~(kTile - 1)) + blockIdx.x * a.tiles * kTile;
  if (first > p) { // nothing visible: an empty partial
    if (tid < nq) {
      const int hm = (g * a.group + q0 + tid) * a.maps + map;
      float *ml = a.ml + ((int64_t)blockIdx.x * a.map_heads + hm) * 2;
      ml[0] = -INFINITY;
      ml[1] = 0.f;
    }
    return;
  }
  const int last = min(first + a.tiles * kTile, (p & ~(kTile - 1)) + kTile); // end of the chunk's tiles
  const bool has_new = p < last;

  // the first tile, asked for ahead of the queries
  constexpr int kAhead = 4;
  const int steps = dim32 / 32;
  Frag<T> kf[kAhead], vf[NV][2];
  auto key_at = [&](int k0) { return kc + (int64_t)((k0 + wave * 16 + col) & a.ring_mask) * dim32 + quad * 8; };
  auto fetch_keys = [&](int k0) {
    const T *kp = key_at(k0);
#pragma unroll
    for (int t = 0; t < kAhead; ++t)
      kf[t].load(kp + min(t, steps - 1) * 32);
  };
  auto fetch_values = [&](int k0) {
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int ct = min(wave + i * 4, vdim16 / 16 - 1);
      const T *vp = vc + (int64_t)(ct * 16 + col) * a.rows + (k0 & a.ring_mask) + quad * 8;
      vf[i][0].load(vp);
      vf[i][1].load(vp + 32);
    }
  };
  fetch_keys(first);
  fetch_values(first);

  for (int f = tid; f < a.half; f += 256) {
    float c, s;
    rotation(turns[f], p, c, s);
    cs[f] = c * a.rot_gain;
    cs[a.half + f] = s * a.rot_gain;
  }
  __syncthreads();
  for (int i = tid; i < 16 * dim32; i += 256) {
    const int h = i / dim32, d = i - h * dim32;
    float v = 0.f;
    if (h < nq && d < a.dim)
      v = turned(proj + a.q_at + (int64_t)((g * a.group + q0 + h) * a.maps + map) * a.dim, d, a.half, cs) * a.scale;
    qs[h * qrow + d] = v;
  }
  if (has_new) {
    const bool keeper = blockIdx.z == 0;
    for (int d = tid; d < dim32; d += 256) {
      const float v = d < a.dim ? turned(proj + a.k_at + (int64_t)gm * a.dim, d, a.half, cs) : 0.f;
      nk[d] = as_stored<T>(v);
      if (keeper)
        store_act<T>(kc + (int64_t)(p & a.ring_mask) * dim32 + d, v);
    }
    for (int c = tid; c < vdim16; c += 256) {
      const float v = c < a.vdim ? proj[a.v_at + (int64_t)g * a.vdim + c] : 0.f;
      nv[c] = as_stored<T>(v);
      if (keeper && map == 0)
        store_act<T>(vc + (int64_t)c * a.rows + (p & a.ring_mask), v);
    }
  }
  __syncthreads();

  f32x4 o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i)
    o[i] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  for (int k0 = first; k0 < last; k0 += kTile) {
    if (k0 > first) {
      fetch_keys(k0);
      fetch_values(k0);
    }
    f32x4 s{0.f, 0.f, 0.f, 0.f};
    const bool mine = k0 + wave * 16 + col == p;
    const float *qp = qs + col * qrow + quad * 8;
    auto score = [&](int t, const Frag<T> &stored) {
      Frag<float> k = widened(stored), q;
      if (mine)
        k.load(nk + t * 32 + quad * 8);
      q.load(qp + t * 32);
      s = mfma32(k, q, s);
    };
#pragma unroll
    for (int t = 0; t < kAhead; ++t)
      if (t < steps)
        score(t, kf[t]);
    for (int t = kAhead; t < steps; ++t) {
      Frag<T> k;
      k.load(key_at(k0) + t * 32);
      score(t, k);
    }
    if (k0 > first)
      __syncthreads(); // the previous tile's scores have been read
#pragma unroll
    for (int r = 0; r < 4; ++r)
      sp[(wave * 16 + quad * 4 + r) * 17 + col] = s[r];
    __syncthreads();
    // all 64 keys of this lane's head, in the order of the value operand
    float w[2][8], mt = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int key = t * 32 + quad * 8 + j, at = k0 + key;
        w[t][j] = at <= p && at >= lo ? sp[key * 17 + col] : -INFINITY;
        mt = fmaxf(mt, w[t][j]);
      }
    float x, y;
    lane_pair<16>(mt, x, y);
    mt = fmaxf(x, y);
    lane_pair<32>(mt, x, y);
    mt = fmaxf(fmaxf(x, y), m); // every tile has a visible key: finite
    const float alpha = fast_exp(m - mt);
    m = mt;
    l *= alpha;
    Frag<float> pw[2];
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float e = fast_exp(w[t][j] - m);
        l += e;
        set_elem(pw[t], j, e);
      }
    const int fresh = p - k0; // the new position within this tile
#pragma unroll
    for (int i = 0; i < NV; ++i) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        o[i][r] *= alpha;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        Frag<float> v = widened(vf[i][t]);
        if (fresh < kTile) {
          const float n = nv[min(wave + i * 4, vdim16 / 16 - 1) * 16 + col];
#pragma unroll
          for (int j = 0; j < 8; ++j)
            set_elem(v, j, t * 32 + quad * 8 + j == fresh ? n : j < 4 ? v.lo[j & 3] : v.hi[j & 3]);
        }
        o[i] = mfma32(v, pw[t], o[i]);
      }
    }
  }
  l = sum_rows(l);
  if (col >= nq)
    return;
  const int hm = (g * a.group + q0 + col) * a.maps + map;
  const int64_t at = (int64_t)blockIdx.x * a.map_heads + hm;
  if (wave == 0 && quad == 0) {
    a.ml[at * 2] = m;
    a.ml[at * 2 + 1] = l;
  }
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (wave + i * 4 < vdim16 / 16)
      *reinterpret_cast<f32x4 *>(a.acc + at * vdim16 + (wave + i * 4) * 16 + quad * 4) = o[i];
}

struct HeadFoldArgs {
  int maps, vdim, gated;
  float lambda, eps, out_gain;
  const float *sink, *gate;
  float *out;
};

// A workgroup per head: its wavefronts share out the chunks, lanes take four value
// channels each; then the maps are combined.
__global__ void __launch_bounds__(256)
head_fold_kernel(const float *__restrict__ acc, const float *__restrict__ ml, int chunks, int map_heads,
                 int vdim16, HeadFoldArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[4];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x;
  float *wt = lds, *fold = lds + ((a.maps * chunks + 3) & ~3); // [maps][chunks], [maps][4][vdim16]
  // a wavefront per map finds the chunks' weights
  if (wave < a.maps) {
    const int hm = h * a.maps + wave;
    const float sink = a.sink ? a.sink[h] : -INFINITY;
    float m = sink;
    for (int c = lane; c < chunks; c += 64)
      m = fmaxf(m, ml[((int64_t)c * map_heads + hm) * 2]);
    m = wave_max(m);
    float l = 0.f;
    for (int c = lane; c < chunks; c += 64) {
      const float2 v = *reinterpret_cast<const float2 *>(ml + ((int64_t)c * map_heads + hm) * 2);
      const float e = v.y > 0.f ? fast_exp(v.x - m) : 0.f;
      wt[wave * chunks + c] = e;
      l = fmaf(e, v.y, l);
    }
    l = wave_sum(l) + (a.sink ? fast_exp(sink - m) : 0.f);
    const float inv = 1.0f / l;
    for (int c = lane; c < chunks; c += 64)
      wt[wave * chunks + c] *= inv;
  }
  __syncthreads();
  for (int mp = 0; mp < a.maps; ++mp)
    for (int i = lane * 4; i < vdim16; i += 256) {
      const float *src = acc + (int64_t)(h * a.maps + mp) * vdim16 + i;
      f32x4 o{0.f, 0.f, 0.f, 0.f};
      for (int c = wave; c < chunks; c += 32) {
        f32x4 v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u)
          v[u] = *reinterpret_cast<const f32x4 *>(src + (int64_t)min(c + u * 4, chunks - 1) * map_heads * vdim16);
#pragma unroll
        for (int u = 0; u < 8; ++u) {
          const float e = c + u * 4 < chunks ? wt[mp * chunks + min(c + u * 4, chunks - 1)] : 0.f;
#pragma unroll
          for (int j = 0; j < 4; ++j) // an empty partial's accumulators were never written
            o[j] = e != 0.f ? fmaf(e, v[u][j], o[j]) : o[j];
        }
      }
      *reinterpret_cast<f32x4 *>(fold + (mp * 4 + wave) * vdim16 + i) = o;
    }
  __syncthreads();
  auto folded = [&](int mp, int i) {
    const float *f = fold + mp * 4 * vdim16 + i;
    return (f[0] + f[vdim16]) + (f[2 * vdim16] + f[3 * vdim16]);
  };
  float scale = 1.f;
  if (a.maps == 2) {
    float ss = 0.f;
    for (int i = tid; i < a.vdim; i += 256) {
      const float d = folded(0, i) - a.lambda * folded(1, i);
      ss = fmaf(d, d, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0)
      red[wave] = ss;
    __syncthreads();
    scale = a.out_gain / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)a.vdim + a.eps);
  }
  for (int i = tid; i < a.vdim; i += 256) {
    float v = folded(0, i);
    if (a.maps == 2)
      v = (v - a.lambda * folded(1, i)) * scale;
    if (a.gated)
      v *= sigmoid_f(a.gate[(int64_t)h * a.vdim + i]);
    a.out[(int64_t)h * a.vdim + i] = v;
  }
}

// ---- many tokens -----------------------------------------------------------------

struct HeadRowsArgs {
  int map_heads, kv_maps, kv_heads, dim, vdim, vdim16, half;
  int ld, q_at, k_at, v_at, rows, start;
  int cache_rows, ring_mask;
  int quads; // whole heads are rotated, and moved four pairs at a time
  float scale, rot_gain;
};

constexpr int kValueSlice = 32; // channels of a value head that are turned round at once

// The first `rows` workgroups: a token's queries and keys.  The others: 64 positions of
// a slice of a value head, turned round in LDS.
template <typename T>
__global__ void __launch_bounds__(256)
head_rows_kernel(const float *__restrict__ proj, T *__restrict__ keys, T *__restrict__ values_t,
                 T *__restrict__ queries, const double *__restrict__ turns, int dim32, HeadRowsArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x;
  if ((int)blockIdx.x < a.rows) {
    const int p = a.start + blockIdx.x;
    const float *row = proj + (int64_t)blockIdx.x * a.ld;
    for (int f = tid; f < a.half; f += 256) {
      float c, s;
      rotation(turns[f], p, c, s);
      lds[f] = c * a.rot_gain;
      lds[a.half + f] = s * a.rot_gain;
    }
    __syncthreads();
    T *qo = queries + (int64_t)blockIdx.x * a.map_heads * dim32;
    const int slot = p & a.ring_mask;
    if (a.quads) {
      const int per = a.half / 4;
      for (int i = tid; i < (a.map_heads + a.kv_maps) * per; i += 256) {
        const int h = i / per, f = (i - h * per) * 4, g = h - a.map_heads;
        const float *src = row + (g < 0 ? a.q_at + h * a.dim : a.k_at + g * a.dim) + f;
        T *dst = (g < 0 ? qo + (int64_t)h * dim32 : keys + ((int64_t)g * a.cache_rows + slot) * dim32) + f;
        const f32x4 u = *reinterpret_cast<const f32x4 *>(src), v = *reinterpret_cast<const f32x4 *>(src + a.half);
        const float m = g < 0 ? a.scale : 1.0f;
        f32x4 x, y;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float c = lds[f + j] * m, s = lds[a.half + f + j] * m;
          x[j] = u[j] * c - v[j] * s;
          y[j] = v[j] * c + u[j] * s;
        }
        store_quad(dst, x);
        store_quad(dst + a.half, y);
      }
      const int pad = dim32 - a.dim;
      for (int i = tid; i < (a.map_heads + a.kv_maps) * pad; i += 256) {
        const int h = i / pad, d = a.dim + i - h * pad, g = h - a.map_heads;
        store_act<T>((g < 0 ? qo + (int64_t)h * dim32 : keys + ((int64_t)g * a.cache_rows + slot) * dim32) + d, 0.f);
      }
      return;
    }
    for (int h = tid >> 6; h < a.map_heads + a.kv_maps; h += 4) {
      const int g = h - a.map_heads;
      const float *src = row + (g < 0 ? a.q_at + h * a.dim : a.k_at + g * a.dim);
      T *dst = g < 0 ? qo + (int64_t)h * dim32 : keys + ((int64_t)g * a.cache_rows + slot) * dim32;
      const float f = g < 0 ? a.scale : 1.0f;
      for (int d = tid & 63; d < dim32; d += 64)
        store_act<T>(dst + d, d < a.dim ? turned(src, d, a.half, lds) * f : 0.f);
    }
    return;
  }
  int b = blockIdx.x - a.rows;
  const int slices = (a.vdim16 + kValueSlice - 1) / kValueSlice, c0 = b % slices * kValueSlice;
  b /= slices;
  const int g = b % a.kv_heads;
  const int t0 = (a.start & ~(kTile - 1)) + b / a.kv_heads * kTile; // aligned positions
  const int p0 = max(t0, a.start), p1 = min(t0 + kTile, a.start + a.rows);
  constexpr int vrow = kValueSlice + 1;
#pragma unroll
  for (int i0 = 0; i0 < kTile * kValueSlice; i0 += 256) {
    const int i = i0 + tid, r = i / kValueSlice, x = i % kValueSlice, c = c0 + x, p = t0 + r;
    lds[r * vrow + x] = p >= p0 && p < p1 && c < a.vdim
                            ? proj[(int64_t)(p - a.start) * a.ld + a.v_at + g * a.vdim + c] : 0.f;
  }
  __syncthreads();
  const int r = tid & 63, p = t0 + r;
  if (p < p0 || p >= p1)
    return;
  for (int x = tid >> 6; x < kValueSlice && c0 + x < a.vdim16; x += 4)
    store_act<T>(values_t + ((int64_t)g * a.vdim16 + c0 + x) * a.cache_rows + (p & a.ring_mask), lds[r * vrow + x]);
}

struct HeadAttnArgs {
  int map_heads, group, maps, vdim, nv, kd, window;
  int rows, start, cache_rows, ring_mask, out_ld;
  const float *sink;
};

// Grid (map heads, query blocks).  A wavefront owns 16 queries, the workgroup's four
// share tiles of keys through LDS; the next tile is on its way in registers meanwhile.
// NK: 32-element steps of a key, NV: 16-channel groups of a value, at most; smaller
// heads are padded with zeros (keys) or with rows whose results are not stored (values).
// Tiles start at multiples of their size, so none is cut by the end of a ring.  OUT: f32
// or the activations' type.
template <typename T, typename OUT, int NK, int NV>
__global__ void __launch_bounds__(256, NV <= 8 ? 2 : 1)
head_attention_kernel(const T *__restrict__ queries, const T *__restrict__ keys,
                      const T *__restrict__ values_t, OUT *__restrict__ out, HeadAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char raw[];
  using F = Flash<T, NK, NV>;
  constexpr int E = F::E, KEYS = F::KEYS, kBlock = 64;
  constexpr int KL = NK, VL = (NV + 1) / 2; // 16-byte loads per thread and tile
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int hm = blockIdx.x, h = hm / a.maps, g = h / a.group, gm = g * a.maps + hm % a.maps;
  const int q0 = (gridDim.y - 1 - blockIdx.y) * kBlock; // long blocks first
  T *kt = reinterpret_cast<T *>(raw); // [KEYS][kKeyRow]
  T *vt = kt + KEYS * F::kKeyRow;     // [16 * NV][kValueRow]

  const int qi = q0 + wave * 16 + col, my_q = a.start + qi; // this lane's query
  Frag<T> qf[NK];
  const T *q = queries + ((int64_t)min(qi, a.rows - 1) * a.map_heads + hm) * a.kd + quad * 8;
#pragma unroll
  for (int t = 0; t < NK; ++t) {
    if (t * 32 < a.kd)
      qf[t].load(q + t * 32);
    else
      qf[t] = Frag<T>{};
  }
  const int key_hi = a.start + min(q0 + kBlock, a.rows) - 1;                // last visible
  const int key_lo = max(0, a.start + q0 - a.window + 1) & ~(KEYS - 1);     // tile of the first
  const int wave_q0 = a.start + q0 + wave * 16, wave_q1 = wave_q0 + 15;

  // the 16-byte runs this thread moves
  const int runs = a.kd / E;
  const T *kc = keys + (int64_t)gm * a.cache_rows * a.kd;
  int ksrc[KL], kdst[KL];
#pragma unroll
  for (int i = 0; i < KL; ++i) {
    const int id = min(i * 256 + tid, KEYS * runs - 1); // past the end: the last one again
    const int r = id / runs, c = id - r * runs;
    ksrc[i] = r * a.kd + c * E;
    kdst[i] = r * F::kKeyRow + c * E;
  }
  const T *vsrc[VL];
  int vdst[VL];
#pragma unroll
  for (int i = 0; i < VL; ++i) {
    const int id = min(i * 256 + tid, 16 * a.nv * 8 - 1), r = id >> 3, c = id & 7;
    vsrc[i] = values_t + ((int64_t)g * 16 * a.nv + r) * a.cache_rows + c * E;
    vdst[i] = F::value_at(r, c);
  }
  u32x4 kr[KL], vr[VL];
  auto fetch = [&](int k0) { // positions past the last query's are masked
    const int slot = k0 & a.ring_mask;
    const T *kp = kc + (int64_t)slot * a.kd;
#pragma unroll
    for (int i = 0; i < KL; ++i)
      kr[i] = *reinterpret_cast<const u32x4 *>(kp + ksrc[i]);
#pragma unroll
    for (int i = 0; i < VL; ++i)
      vr[i] = *reinterpret_cast<const u32x4 *>(vsrc[i] + slot);
  };
  fetch(key_lo);
  if (a.kd < NK * 32) { // the padding of the keys
    const int pad = NK * 32 - a.kd;
    for (int i = tid; i < KEYS * pad; i += 256)
      kt[(i / pad) * F::kKeyRow + a.kd + i % pad] = 0;
  }

  F flash;
  for (int k0 = key_lo; k0 <= key_hi; k0 += KEYS) {
    __syncthreads(); // the previous tile has been read
#pragma unroll
    for (int i = 0; i < KL; ++i)
      *reinterpret_cast<u32x4 *>(kt + kdst[i]) = kr[i];
#pragma unroll
    for (int i = 0; i < VL; ++i)
      F::store_value(vt, vdst[i], vr[i]);
    __syncthreads();
    fetch(min(k0 + KEYS, key_hi & ~(KEYS - 1)));
    if (k0 > wave_q1 || k0 + KEYS - 1 <= wave_q0 - a.window)
      continue; // nothing of this tile is visible to this wavefront
    const bool whole = k0 + KEYS - 1 <= wave_q0 && wave_q1 - k0 < a.window;
    flash.tile(kt, vt, qf, whole, my_q - k0, a.window);
  }
  float sum = sum_rows(flash.l);
  if (qi >= a.rows)
    return;
  float f;
  if (a.sink) {
    const float sink = a.sink[h], m = fmaxf(flash.m, sink), e = fast_exp(flash.m - m);
    f = e / fmaf(sum, e, fast_exp(sink - m));
  } else {
    f = 1.0f / sum;
  }
  OUT *dst = out + (int64_t)qi * a.out_ld + (int64_t)hm * a.vdim;
#pragma unroll
  for (int v = 0; v < NV; ++v)
    if (v < a.nv) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = v * 16 + quad * 4 + r;
        if (c < a.vdim)
          store_act<OUT>(dst + c, flash.o[v][r] * f);
      }
    }
}

struct HeadCombineArgs {
  int heads, maps, vdim, rows, ld, gate_at, out_ld, gated;
  float lambda, eps, out_gain;
};

// A wavefront per row and head.
template <typename T>
__global__ void __launch_bounds__(256)
head_combine_kernel(const float *__restrict__ maps_out, const float *__restrict__ proj, T *__restrict__ out,
                    HeadCombineArgs a) {
  const int lane = threadIdx.x & 63;
  const int64_t id = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (id >= (int64_t)a.rows * a.heads)
    return;
  const int64_t row = id / a.heads;
  const int h = (int)(id - row * a.heads);
  const float *o = maps_out + id * a.maps * a.vdim;
  auto value = [&](int i) { return a.maps == 2 ? o[i] - a.lambda * o[a.vdim + i] : o[i]; };
  float scale = 1.f;
  if (a.maps == 2) {
    float ss = 0.f;
    for (int i = lane; i < a.vdim; i += 64) {
      const float d = value(i);
      ss = fmaf(d, d, ss);
    }
    scale = a.out_gain / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
  }
  const float *gate = proj + row * a.ld + a.gate_at + (int64_t)h * a.vdim;
  for (int i = lane; i < a.vdim; i += 64) {
    float v = value(i) * scale;
    if (a.gated)
      v *= sigmoid_f(gate[i]);
    store_act<T>(out + row * a.out_ld + (int64_t)h * a.vdim + i, v);
  }
}

constexpr size_t kLdsLimit = 156 * 1024;

bool shape_ok(const HeadShape &s) {
  return s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && (s.maps == 1 || s.maps == 2) &&
         s.dim > 0 && s.vdim > 0 && s.rot_dims >= 0 && s.rot_dims % 2 == 0 && s.rot_dims <= s.dim &&
         (s.rot_dims == 0 || s.turns) && s.window >= 0 && s.rows > 0 && s.rows % kTile == 0 &&
         (s.ring_mask == INT_MAX || (s.ring_mask == s.rows - 1 && (s.rows & (s.rows - 1)) == 0));
}
int window_of(const HeadShape &s) { return s.window ? s.window : INT_MAX; }
// key tiles a step may touch, and how they are cut: chunks of `tiles` tiles
int step_tiles(const HeadShape &s, int span) {
  if (s.window)
    span = std::min(span, s.window);
  return (int)ceil_div(span, kTile) + (s.window ? 1 : 0);
}
int chunk_tiles(int tiles) { return (int)ceil_div(tiles, 64); }

} // namespace

void head_cache_rows(HeadShape &s, int max_len, int block) {
  const int64_t all = round_up(max_len, kTile), ring = (int64_t)s.window - 1 + block;
  int64_t p = kTile;
  while (p < ring)
    p *= 2;
  if (s.window && p < all) {
    s.rows = (int)p;
    s.ring_mask = s.rows - 1;
  } else {
    s.rows = (int)all;
    s.ring_mask = INT_MAX;
  }
}

int head_max_chunks(const HeadShape &s, int max_len) {
  // the number of chunks falls where a chunk gets another tile
  const int tiles = step_tiles(s, (int)round_up(max_len, kTile) * 2);
  return std::min(tiles, 64);
}

int launch_head_step(const HeadStep &a, int span, hipStream_t stream) {
  const HeadShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.pos && a.keys && a.values_t && a.part_acc && a.part_ml && a.out &&
                 span > 0,
             "head_step: bad argument");
  const int tiles = step_tiles(s, span), per = chunk_tiles(tiles), chunks = (int)ceil_div(tiles, per);
  const int group = s.heads / s.kv_heads, d32 = s.dim32(), v16 = s.vdim16();
  HeadPartArgs p{group, s.maps, s.dim, s.vdim, s.rot_dims / 2, window_of(s), s.ring_mask, s.rows, per,
                 a.q_at, a.k_at, a.v_at, s.map_heads(), s.scale, s.rot_gain, a.part_acc, a.part_ml};
  const size_t lds = sizeof(float) * ((size_t)16 * (d32 + 4) + d32 + v16 + round_up(s.rot_dims, 4) + 64 * 17);
  BH_REQUIRE(lds <= kLdsLimit && v16 <= 512, "head_step: heads of %d and %d values", s.dim, s.vdim);
  const dim3 grid((unsigned)chunks, (unsigned)(s.kv_heads * s.maps), (unsigned)ceil_div(group, 16));
#define BH_PART(T, NV)                                                                             \
  do {                                                                                             \
    static DynLdsOnce once;                                                                        \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)head_part_kernel<T, NV>, (int)kLdsLimit));     \
    hipLaunchKernelGGL((head_part_kernel<T, NV>), grid, dim3(256), lds, stream, a.proj,            \
                       static_cast<T *>(a.keys), static_cast<T *>(a.values_t), s.turns, a.pos,     \
                       d32, v16, p);                                                               \
  } while (0)
#define BH_PARTS(T)                                                                                \
  do {                                                                                             \
    if (v16 <= 64)                                                                                 \
      BH_PART(T, 1);                                                                               \
    else if (v16 <= 128)                                                                           \
      BH_PART(T, 2);                                                                               \
    else if (v16 <= 256)                                                                           \
      BH_PART(T, 4);                                                                               \
    else                                                                                           \
      BH_PART(T, 8);                                                                               \
  } while (0)
  if (s.f32)
    BH_PARTS(float);
  else
    BH_PARTS(bf16_bits);
#undef BH_PARTS
#undef BH_PART
  BH_CHECK_HIP(hipGetLastError());
  HeadFoldArgs f{s.maps, s.vdim, s.gated ? 1 : 0, s.lambda, s.eps, s.out_gain, s.sink,
                 a.proj + a.gate_at, a.out};
  const size_t fold_lds = sizeof(float) * ((size_t)round_up((int64_t)s.maps * chunks, 4) + (size_t)s.maps * 4 * v16);
  hipLaunchKernelGGL(head_fold_kernel, dim3((unsigned)s.heads), dim3(256), fold_lds, stream, a.part_acc,
                     a.part_ml, chunks, s.map_heads(), v16, f);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

namespace {
template <typename T, typename OUT, int NK, int NV>
int launch_attention(const HeadRows &a, OUT *out, const HeadAttnArgs &p, hipStream_t stream) {
  using F = Flash<T, NK, NV>;
  constexpr size_t lds = sizeof(T) * ((size_t)F::KEYS * F::kKeyRow + (size_t)16 * NV * F::kValueRow);
  static_assert(lds <= kLdsLimit, "the tiles must fit LDS");
  static DynLdsOnce once;
  BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)head_attention_kernel<T, OUT, NK, NV>, (int)kLdsLimit));
  hipLaunchKernelGGL((head_attention_kernel<T, OUT, NK, NV>),
                     dim3((unsigned)p.map_heads, (unsigned)ceil_div(a.rows, 64)), dim3(256), lds, stream,
                     static_cast<const T *>(a.queries), static_cast<const T *>(a.keys),
                     static_cast<const T *>(a.values_t), out, p);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}
template <typename T, typename OUT>
int launch_attention_any(const HeadRows &a, OUT *out, const HeadAttnArgs &p, hipStream_t stream) {
  const int nk = p.kd / 32;
  BH_REQUIRE(nk <= 16 && p.nv <= 32, "head_attention: heads of %d and %d values", a.s.dim, a.s.vdim);
  if (nk <= 2 && p.nv <= 4)
    return launch_attention<T, OUT, 2, 4>(a, out, p, stream);
  if (nk <= 2 && p.nv <= 8)
    return launch_attention<T, OUT, 2, 8>(a, out, p, stream);
  if (nk <= 4 && p.nv <= 8)
    return launch_attention<T, OUT, 4, 8>(a, out, p, stream);
  if (nk <= 8 && p.nv <= 16)
    return launch_attention<T, OUT, 8, 16>(a, out, p, stream);
  return launch_attention<T, OUT, 16, 32>(a, out, p, stream);
}

template <typename T> int launch_rows(const HeadRows &a, hipStream_t stream) {
  const HeadShape &s = a.s;
  HeadRowsArgs r{s.map_heads(), s.kv_heads * s.maps, s.kv_heads, s.dim, s.vdim, s.vdim16(), s.rot_dims / 2,
                 a.ld, a.q_at, a.k_at, a.v_at, a.rows, a.start, s.rows, s.ring_mask, 0, s.scale, s.rot_gain};
  r.quads = s.rot_dims == s.dim && s.dim % 8 == 0 && a.ld % 4 == 0 && a.q_at % 4 == 0 && a.k_at % 4 == 0 &&
            (((uintptr_t)a.proj | (uintptr_t)a.queries | (uintptr_t)a.keys) & 15) == 0;
  const int value_tiles = (a.start + a.rows - 1) / kTile - a.start / kTile + 1;
  const int value_groups = value_tiles * s.kv_heads * (int)ceil_div(s.vdim16(), kValueSlice);
  const size_t lds = sizeof(float) * std::max((size_t)s.rot_dims, (size_t)kTile * (kValueSlice + 1));
  hipLaunchKernelGGL(head_rows_kernel<T>, dim3((unsigned)(a.rows + value_groups)), dim3(256), lds, stream, a.proj, static_cast<T *>(a.keys), static_cast<T *>(a.values_t),
                     static_cast<T *>(a.queries), s.turns, s.dim32(), r);
  BH_CHECK_HIP(hipGetLastError());
  HeadAttnArgs p{s.map_heads(), s.heads / s.kv_heads, s.maps, s.vdim, s.vdim16() / 16, s.dim32(), window_of(s),
                 a.rows, a.start, s.rows, s.ring_mask, a.out_ld, s.sink};
  if (s.maps == 1 && !s.gated)
    return launch_attention_any<T, T>(a, static_cast<T *>(a.out), p, stream);
  p.out_ld = s.map_heads() * s.vdim;
  if (int rc = launch_attention_any<T, float>(a, a.maps_out, p, stream))
    return rc;
  HeadCombineArgs c{s.heads, s.maps, s.vdim, a.rows, a.ld, a.gate_at, a.out_ld, s.gated ? 1 : 0,
                    s.lambda, s.eps, s.out_gain};
  hipLaunchKernelGGL(head_combine_kernel<T>, dim3((unsigned)ceil_div((int64_t)a.rows * s.heads, 4)), dim3(256), 0,
                     stream, a.maps_out, a.proj, static_cast<T *>(a.out), c);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}
} // namespace

int launch_head_rows(const HeadRows &a, hipStream_t stream) {
  const HeadShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.keys && a.values_t && a.queries && a.out && a.rows > 0 && a.start >= 0 &&
                 s.vdim <= 512 && ((s.maps == 1 && !s.gated) || a.maps_out),
             "head_rows: bad argument");
  // the new rows must not take the place of visible ones
  BH_REQUIRE(s.ring_mask == INT_MAX ? a.start + a.rows <= s.rows
                                    : a.rows + std::min(a.start, s.window - 1) <= s.rows,
             "head_rows: %d rows from %d leave the cache (%d rows)", a.rows, a.start, s.rows);
  return s.f32 ? launch_rows<float>(a, stream) : launch_rows<bf16_bits>(a, stream);
}

} // namespace bh
