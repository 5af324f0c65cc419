// latent_attn.hip -- latent attention over a ring of cached latents: three launches
// for a token (queries and the cache row, attention partials, fold + values), and
// for a prompt the cache rows and a flash attention over expanded keys and values.
//
// Scores, softmax and sums are f32.  A token's products are f32 throughout.  Of a
// prompt the products take the operands in the cache's format: f32 on the f32
// matrix cores, or bfloat16 keys, queries and values with the softmax weights as
// two bfloat16 terms each (17 bits), all summed in f32.
#include "latent_attn.h"
#include "bf16_dev.h"

#include <algorithm>

namespace bh {
namespace {

// cos and sin of position * turns (turns of the full circle per position); the
// product is reduced to a fraction of a turn in double, so a far position keeps
// its 32-bit angle
__device__ __forceinline__ void rotation(double turns, int p, float &c, float &s) {
  double t = turns * (double)p;
  t -= rint(t);
  sincospif(2.0f * (float)t, &s, &c);
}

constexpr int kStepThreads = 512, kStepWaves = 8;

struct LatentQueryArgs {
  int heads, dim, rot_dim, rank, row_elems, ring_mask, dkv_at, uk_groups, uk_ktiles;
  float scale, eps;
  const float *norm_w;
  const double *turns;
  const int *pos;
  void *cache;
  float *query;
};

// Grid (heads + 1, parts): the last row of workgroups writes the token's cache
// row, the others a head's query in the space of a cache row.
template <typename T>
__global__ void __launch_bounds__(kStepThreads)
latent_query_kernel(const uint4 *__restrict__ uk, const float *__restrict__ proj, LatentQueryArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, half = a.rot_dim / 2;
  const int p = *a.pos;
  if (h == a.heads) {
    if (blockIdx.y)
      return;
    __shared__ float red[kStepWaves];
    const float *d = proj + a.dkv_at;
    float ss = 0.f;
    for (int i = tid; i < a.rank; i += kStepThreads)
      ss = fmaf(d[i], d[i], ss);
    ss = wave_sum(ss);
    if (lane == 0)
      red[wave] = ss;
    __syncthreads();
    ss = 0.f;
    for (int w = 0; w < kStepWaves; ++w)
      ss += red[w];
    const float r = 1.0f / sqrtf(ss / (float)a.rank + a.eps);
    T *row = static_cast<T *>(a.cache) + (int64_t)(p & a.ring_mask) * a.row_elems;
    for (int i = tid; i < a.row_elems; i += kStepThreads) {
      float v = 0.f;
      if (i < a.rank) {
        v = d[i] * r * a.norm_w[i];
      } else if (i < a.rank + a.rot_dim) {
        const int j = i - a.rank, f = j < half ? j : j - half;
        float c, s;
        rotation(a.turns[f], p, c, s);
        const float u = d[a.rank + f], w = d[a.rank + f + half];
        v = j < half ? u * c - w * s : w * c + u * s;
      }
      store_act<T>(row + i, v);
    }
    return;
  }
  const float *q = proj + (int64_t)h * (a.dim + a.rot_dim);
  float *out = a.query + (int64_t)h * a.row_elems;
  const int Kp = a.uk_ktiles * kBfTileK;
  for (int i = tid; i < Kp; i += kStepThreads)
    lds[i] = i < a.dim ? q[i] : 0.f;
  if (blockIdx.y == 0)
    for (int i = a.rank + tid; i < a.row_elems; i += kStepThreads) {
      float v = 0.f;
      const int j = i - a.rank;
      if (j < a.rot_dim) {
        const int f = j < half ? j : j - half;
        float c, s;
        rotation(a.turns[f], p, c, s);
        const float u = q[a.dim + f], w = q[a.dim + f + half];
        v = (j < half ? u * c - w * s : w * c + u * s) * a.scale;
      }
      out[i] = v;
    }
  __syncthreads();
  for (int g = blockIdx.y * kStepWaves + wave; g < a.uk_groups; g += gridDim.y * kStepWaves) {
    const uint4 *wp = uk + ((int64_t)h * a.uk_groups + g) * a.uk_ktiles * 64 + lane;
    float acc = 0.f;
#pragma unroll 4
    for (int t = 0; t < a.uk_ktiles; ++t) {
      const uint4 w = wp[(int64_t)t * 64];
      const float *x = lds + t * kBfTileK + (lane >> 4) * 8;
      acc = fmaf(bf_lo(w.x), x[0], acc);
      acc = fmaf(bf_hi(w.x), x[1], acc);
      acc = fmaf(bf_lo(w.y), x[2], acc);
      acc = fmaf(bf_hi(w.y), x[3], acc);
      acc = fmaf(bf_lo(w.z), x[4], acc);
      acc = fmaf(bf_hi(w.z), x[5], acc);
      acc = fmaf(bf_lo(w.w), x[6], acc);
      acc = fmaf(bf_hi(w.w), x[7], acc);
    }
    acc = sum_rows(acc);
    const int l = g * 16 + lane;
    if (lane < 16 && l < a.rank)
      out[l] = acc * a.scale;
  }
}

struct LatentPartArgs {
  int heads, heads16, rank16, row_elems, window, ring_mask, lds_stride;
  const int *pos;
  float *acc, *ml;
};

// Grid (chunks, heads16 / 16).  Four wavefronts per key tile of 16 positions: each
// takes a quarter of the score's k, then all share out the latent dimensions.
// S^T = C . Q^T leaves a lane with 4 keys of one head, which is the B operand of
// O^T += C^T . P^T as it lies.
template <typename T, int KT>
__global__ void __launch_bounds__(KT * 256)
latent_part_kernel(const T *__restrict__ cache, const float *__restrict__ query, LatentPartArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char raw[];
  constexpr int kThreads = KT * 256, kKeys = KT * 16;
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int qs = a.row_elems + 4;
  T *ck = reinterpret_cast<T *>(raw);                                            // [kKeys][lds_stride]
  float *qq = reinterpret_cast<float *>(raw + sizeof(T) * kKeys * a.lds_stride); // [16][qs]
  float *sp = qq + 16 * qs;                                                      // [KT][4][16][16]
  const int p = *a.pos;
  const int lo = max(0, p - a.window + 1), n = p - lo + 1;
  const int k0 = blockIdx.x * kKeys, head0 = blockIdx.y * 16;
  float *ml = a.ml + ((int64_t)blockIdx.x * a.heads16 + head0) * 2;
  if (k0 >= n) { // nothing visible: an empty partial
    if (tid < 16) {
      ml[tid * 2] = -INFINITY;
      ml[tid * 2 + 1] = 0.f;
    }
    return;
  }
  constexpr int E = 16 / (int)sizeof(T);
  const int runs = a.row_elems / E;
  for (int i = tid; i < kKeys * runs; i += kThreads) {
    const int r = i / runs, c = i - r * runs;
    uint4 v{0, 0, 0, 0};
    if (k0 + r < n)
      v = *reinterpret_cast<const uint4 *>(cache + (int64_t)((lo + k0 + r) & a.ring_mask) * a.row_elems + c * E);
    *reinterpret_cast<uint4 *>(ck + r * a.lds_stride + c * E) = v;
  }
  const int qruns = a.row_elems / 4;
  for (int i = tid; i < 16 * qruns; i += kThreads) {
    const int r = i / qruns, c = i - r * qruns;
    f32x4 v{0.f, 0.f, 0.f, 0.f};
    if (head0 + r < a.heads)
      v = *reinterpret_cast<const f32x4 *>(query + (int64_t)(head0 + r) * a.row_elems + c * 4);
    *reinterpret_cast<f32x4 *>(qq + r * qs + c * 4) = v;
  }
  __syncthreads();
  {
    const int kt = wave >> 2, quarter = wave & 3;
    f32x4 s{0.f, 0.f, 0.f, 0.f};
    const T *kr = ck + (kt * 16 + col) * a.lds_stride + quad * 8;
    const float *qr = qq + col * qs + quad * 8;
    for (int t = quarter; t < a.row_elems / 32; t += 4) {
      Frag<T> kf;
      Frag<float> qf, kw;
      kf.load(kr + t * 32);
      qf.load(qr + t * 32);
      if constexpr (sizeof(T) == 2)
        kw = widen(kf.v);
      else
        kw = kf;
      s = mfma32(kw, qf, s);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
      sp[((wave * 16) + quad * 4 + r) * 16 + col] = s[r];
  }
  __syncthreads();
  f32x4 pr[KT];
  float m = -INFINITY;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int key = quad * 4 + r;
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w)
        s += sp[(((kt * 4 + w) * 16) + key) * 16 + col];
      s = k0 + kt * 16 + key < n ? s : -INFINITY;
      pr[kt][r] = s;
      m = fmaxf(m, s);
    }
  {
    float x, y;
    lane_pair<16>(m, x, y);
    m = fmaxf(x, y);
    lane_pair<32>(m, x, y);
    m = fmaxf(x, y);
  }
  float l = 0.f;
#pragma unroll
  for (int kt = 0; kt < KT; ++kt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = fast_exp(pr[kt][r] - m); // the chunk's first key is visible: m is finite
      pr[kt][r] = e;
      l += e;
    }
  l = sum_rows(l);
  if (wave == 0 && lane < 16) {
    ml[lane * 2] = m;
    ml[lane * 2 + 1] = l;
  }
  float *acc = a.acc + ((int64_t)blockIdx.x * a.heads16 + head0 + col) * a.rank16;
  for (int lt = wave; lt < a.rank16 / 16; lt += KT * 4) {
    f32x4 o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        o = mfma_f32(load_act<T>(ck + (kt * 16 + quad * 4 + r) * a.lds_stride + lt * 16 + col),
                     pr[kt][r], o);
    *reinterpret_cast<f32x4 *>(acc + lt * 16 + quad * 4) = o;
  }
}

struct LatentFoldArgs {
  int heads16, rank, rank16, vdim, groups, ktiles, chunks;
  const float *acc, *ml, *gate;
  float *out;
};

// Grid (heads, parts of the value channels): folds the partials of a head, then
// four channel groups of its value matrix, k in two slices.
__global__ void __launch_bounds__(kStepThreads)
latent_value_kernel(const uint4 *__restrict__ uv, LatentFoldArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float part[kStepWaves][16];
  __shared__ float red[2][kStepWaves];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x;
  const int Kp = a.ktiles * kBfTileK;
  float *x = lds, *wt = lds + Kp; // [Kp], [chunks]
  const int gi = wave >> 1, slice = wave & 1;
  const int g = blockIdx.y * 4 + gi, gl = min(g, a.groups - 1);
  const int half = (a.ktiles + 1) / 2;
  const int t0 = slice * half, t1 = min(t0 + half, a.ktiles);
  const uint4 *wp = uv + ((int64_t)h * a.groups + gl) * a.ktiles * 64 + lane;
  constexpr int kAhead = 8;
  uint4 w[kAhead];
#pragma unroll
  for (int u = 0; u < kAhead; ++u)
    w[u] = wp[(int64_t)min(t0 + u, a.ktiles - 1) * 64];
  float m = -INFINITY;
  for (int c = tid; c < a.chunks; c += kStepThreads)
    m = fmaxf(m, a.ml[((int64_t)c * a.heads16 + h) * 2]);
  m = wave_max(m);
  if (lane == 0)
    red[0][wave] = m;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < kStepWaves; ++i)
    m = fmaxf(m, red[0][i]);
  float l = 0.f;
  for (int c = tid; c < a.chunks; c += kStepThreads) {
    const float *q = a.ml + ((int64_t)c * a.heads16 + h) * 2;
    const float e = q[1] > 0.f ? fast_exp(q[0] - m) : 0.f;
    wt[c] = e;
    l = fmaf(e, q[1], l);
  }
  l = wave_sum(l);
  if (lane == 0)
    red[1][wave] = l;
  __syncthreads();
  l = 0.f;
#pragma unroll
  for (int i = 0; i < kStepWaves; ++i)
    l += red[1][i];
  const float inv = 1.0f / l;
  const int64_t step = (int64_t)a.heads16 * a.rank16;
  for (int i = tid; i < Kp; i += kStepThreads) {
    float o = 0.f;
    if (i < a.rank) {
      const float *q = a.acc + (int64_t)h * a.rank16 + i;
      int c = 0;
      for (; c + 8 <= a.chunks; c += 8) {
        float v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u)
          v[u] = q[(c + u) * step];
#pragma unroll
        for (int u = 0; u < 8; ++u) // an empty partial's accumulators were never written
          o = wt[c + u] != 0.f ? fmaf(wt[c + u], v[u], o) : o;
      }
      for (; c < a.chunks; ++c)
        o = wt[c] != 0.f ? fmaf(wt[c], q[c * step], o) : o;
      o *= inv;
    }
    x[i] = o;
  }
  __syncthreads();
  float acc = 0.f;
  const float *xp = x + (lane >> 4) * 8;
  for (int t = t0; t < t1; t += kAhead) {
    if (t > t0) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        w[u] = wp[(int64_t)min(t + u, a.ktiles - 1) * 64];
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u)
      if (t + u < t1) {
        const float *v = xp + (t + u) * kBfTileK;
        acc = fmaf(bf_lo(w[u].x), v[0], acc);
        acc = fmaf(bf_hi(w[u].x), v[1], acc);
        acc = fmaf(bf_lo(w[u].y), v[2], acc);
        acc = fmaf(bf_hi(w[u].y), v[3], acc);
        acc = fmaf(bf_lo(w[u].z), v[4], acc);
        acc = fmaf(bf_hi(w[u].z), v[5], acc);
        acc = fmaf(bf_lo(w[u].w), v[6], acc);
        acc = fmaf(bf_hi(w[u].w), v[7], acc);
      }
  }
  acc = sum_rows(acc);
  if (lane < 16)
    part[wave][lane] = acc;
  __syncthreads();
  if (tid < 64) {
    const int gg = blockIdx.y * 4 + (tid >> 4), v = gg * 16 + (tid & 15);
    if (gg < a.groups && v < a.vdim)
      a.out[(int64_t)h * a.vdim + v] =
          (part[(tid >> 4) * 2][tid & 15] + part[(tid >> 4) * 2 + 1][tid & 15]) *
          sigmoid_f(a.gate[h]);
  }
}

// ---- many tokens -----------------------------------------------------------------

struct LatentRowsArgs {
  int heads, dim, rot_dim, rank, row_elems, ring_mask, dkv_at, ld, start;
  float scale, eps;
  const float *norm_w;
  const double *turns;
};

// One workgroup per token: the cache row, and the queries rotated and scaled in place.
template <typename T>
__global__ void __launch_bounds__(256)
latent_rows_kernel(float *__restrict__ proj, T *__restrict__ cache, LatentRowsArgs a) {
  extern __shared__ float lds[]; // cos, sin of this position
  __shared__ float red[4];
  const int tid = threadIdx.x, half = a.rot_dim / 2;
  const int p = a.start + blockIdx.x;
  float *row = proj + (int64_t)blockIdx.x * a.ld;
  const float *d = row + a.dkv_at;
  for (int f = tid; f < half; f += 256)
    rotation(a.turns[f], p, lds[f], lds[half + f]);
  float ss = 0.f;
  for (int i = tid; i < a.rank; i += 256)
    ss = fmaf(d[i], d[i], ss);
  ss = wave_sum(ss);
  if ((tid & 63) == 0)
    red[tid >> 6] = ss;
  __syncthreads();
  const float r = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.rank + a.eps);
  T *out = cache + (int64_t)(p & a.ring_mask) * a.row_elems;
  for (int i = tid; i < a.row_elems; i += 256) {
    float v = 0.f;
    if (i < a.rank) {
      v = d[i] * r * a.norm_w[i];
    } else if (i < a.rank + a.rot_dim) {
      const int j = i - a.rank, f = j < half ? j : j - half;
      const float u = d[a.rank + f], w = d[a.rank + f + half];
      v = j < half ? u * lds[f] - w * lds[half + f] : w * lds[f] + u * lds[half + f];
    }
    store_act<T>(out + i, v);
  }
  const int per = a.dim + half; // work items per head: unrotated values, then pairs
  for (int i = tid; i < a.heads * per; i += 256) {
    const int h = i / per, j = i - h * per;
    float *q = row + (int64_t)h * (a.dim + a.rot_dim);
    if (j < a.dim) {
      q[j] *= a.scale;
    } else {
      const int f = j - a.dim;
      const float u = q[a.dim + f], w = q[a.dim + f + half];
      q[a.dim + f] = (u * lds[f] - w * lds[half + f]) * a.scale;
      q[a.dim + f + half] = (w * lds[f] + u * lds[half + f]) * a.scale;
    }
  }
}

struct LatentAttnArgs {
  int heads, dim, dim16, rot_dim, vdim, vdim16, rank, row_elems, window, ring_mask;
  int ld, gate_at, rows, start, first, value_ld, out_ld;
  int kd, k_stride, v_stride; // LDS: padded key size, row strides of the K / Q and V^T tiles
};

constexpr int kTileKeys = 32;

// Grid (query blocks, heads).  A wavefront owns 16 queries; the workgroup's share
// tiles of 32 keys through LDS.  S^T = K . Q^T leaves a lane with keys of one
// query, which is the B operand of O^T += V^T . P^T as it lies.
template <typename T, int NV>
__global__ void __launch_bounds__(256)
latent_attention_kernel(const float *__restrict__ proj, const T *__restrict__ keys,
                        const T *__restrict__ values_t, const T *__restrict__ cache,
                        T *__restrict__ out, LatentAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char raw[];
  constexpr int E = 16 / (int)sizeof(T);
  const int threads = blockDim.x, waves = threads >> 6, block = waves * 16;
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.y;
  // long blocks first
  const int qb = gridDim.x - 1 - blockIdx.x, q0 = qb * block;
  T *qt = reinterpret_cast<T *>(raw);                // [block][k_stride]
  T *kt = qt + block * a.k_stride;                   // [32][k_stride]
  T *vt = kt + kTileKeys * a.k_stride;               // [vdim16][v_stride]
  for (int i = tid; i < block * a.kd; i += threads) {
    const int r = i / a.kd, k = i - r * a.kd;
    float v = 0.f;
    if (q0 + r < a.rows) {
      const float *q = proj + (int64_t)(q0 + r) * a.ld + (int64_t)h * (a.dim + a.rot_dim);
      if (k < a.dim)
        v = q[k];
      else if (k >= a.dim16 && k < a.dim16 + a.rot_dim)
        v = q[a.dim + k - a.dim16];
    }
    store_act<T>(qt + r * a.k_stride + k, v);
  }
  const int last_q = min(q0 + block, a.rows) - 1;
  const int key_hi = a.start + last_q - a.first;                                      // last visible
  const int key_lo = max(0, a.start + q0 - a.window + 1 - a.first) & ~(kTileKeys - 1); // tile of the first
  const int nkeys = a.start + a.rows - a.first;
  const int my_q = a.start + q0 + wave * 16 + col - a.first; // this lane's query as a key index

  f32x4 o[NV];
#pragma unroll
  for (int v = 0; v < NV; ++v)
    o[v] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;
  const int nv = a.vdim16 / 16;
  const int64_t kld = (int64_t)a.heads * a.dim16;
  for (int k0 = key_lo; k0 <= key_hi; k0 += kTileKeys) {
    __syncthreads(); // the previous tile has been read (and the queries are staged)
    const int kruns = a.dim16 / E;
    for (int i = tid; i < kTileKeys * kruns; i += threads) {
      const int r = i / kruns, c = i - r * kruns;
      uint4 v{0, 0, 0, 0};
      if (k0 + r < nkeys)
        v = *reinterpret_cast<const uint4 *>(keys + (k0 + r) * kld + h * a.dim16 + c * E);
      *reinterpret_cast<uint4 *>(kt + r * a.k_stride + c * E) = v;
    }
    const int tail = a.kd - a.dim16; // the shared rotated part and the padding
    for (int i = tid; i < kTileKeys * tail; i += threads) {
      const int r = i / tail, c = i - r * tail;
      T v = 0;
      if (k0 + r < nkeys && c < a.rot_dim)
        v = cache[(int64_t)((a.first + k0 + r) & a.ring_mask) * a.row_elems + a.rank + c];
      kt[r * a.k_stride + a.dim16 + c] = v;
    }
    constexpr int vruns = kTileKeys / E;
    for (int i = tid; i < a.vdim16 * vruns; i += threads) {
      const int r = i / vruns, c = i - r * vruns;
      uint4 v = *reinterpret_cast<const uint4 *>(values_t + (int64_t)(h * a.vdim16 + r) * a.value_ld + k0 + c * E);
      if (k0 + c * E + E > nkeys) { // columns past the last key hold anything
        T e[E];
        __builtin_memcpy(e, &v, 16);
#pragma unroll
        for (int j = 0; j < E; ++j)
          if (k0 + c * E + j >= nkeys)
            e[j] = 0;
        __builtin_memcpy(&v, e, 16);
      }
      *reinterpret_cast<uint4 *>(vt + r * a.v_stride + c * E) = v;
    }
    __syncthreads();
    f32x4 s0{0.f, 0.f, 0.f, 0.f}, s1 = s0;
    const T *qr = qt + (wave * 16 + col) * a.k_stride + quad * 8;
    const T *kr = kt + col * a.k_stride + quad * 8;
    for (int t = 0; t < a.kd; t += 32) {
      Frag<T> q, ka, kb;
      q.load(qr + t);
      ka.load(kr + t);
      kb.load(kr + 16 * a.k_stride + t);
      s0 = mfma32(ka, q, s0);
      s1 = mfma32(kb, q, s1);
    }
    float mt = m;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int ka = k0 + quad * 4 + r, kb = ka + 16;
      s0[r] = ka <= my_q && my_q - ka < a.window ? s0[r] : -INFINITY;
      s1[r] = kb <= my_q && my_q - kb < a.window ? s1[r] : -INFINITY;
      mt = fmaxf(mt, fmaxf(s0[r], s1[r]));
    }
    {
      float x, y;
      lane_pair<16>(mt, x, y);
      mt = fmaxf(x, y);
      lane_pair<32>(mt, x, y);
      mt = fmaxf(x, y);
    }
    const float base = mt == -INFINITY ? 0.f : mt; // nothing visible so far
    const float alpha = fast_exp(m - base);
    m = mt;
    float sum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s0[r] = fast_exp(s0[r] - base);
      s1[r] = fast_exp(s1[r] - base);
      sum += s0[r] + s1[r];
    }
    l = fmaf(l, alpha, sum);
    if constexpr (sizeof(T) == 2) {
      uint4 hi, lo;
      unsigned *ph = reinterpret_cast<unsigned *>(&hi), *pl = reinterpret_cast<unsigned *>(&lo);
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        ph[j] = pack_bf(s0[2 * j], s0[2 * j + 1]);
        pl[j] = pack_bf(s0[2 * j] - bf_lo(ph[j]), s0[2 * j + 1] - bf_hi(ph[j]));
        ph[2 + j] = pack_bf(s1[2 * j], s1[2 * j + 1]);
        pl[2 + j] = pack_bf(s1[2 * j] - bf_lo(ph[2 + j]), s1[2 * j + 1] - bf_hi(ph[2 + j]));
      }
#pragma unroll
      for (int v = 0; v < NV; ++v)
        if (v < nv) {
          const T *vr = vt + (v * 16 + col) * a.v_stride + quad * 4;
          const uint2 va = *reinterpret_cast<const uint2 *>(vr), vb = *reinterpret_cast<const uint2 *>(vr + 16);
          const uint4 vv{va.x, va.y, vb.x, vb.y};
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[v][r] *= alpha;
          o[v] = mfma_bf16(vv, hi, o[v]);
          o[v] = mfma_bf16(vv, lo, o[v]);
        }
    } else {
#pragma unroll
      for (int v = 0; v < NV; ++v)
        if (v < nv) {
          const float *vr = reinterpret_cast<const float *>(vt) + (v * 16 + col) * a.v_stride + quad * 4;
          const f32x4 va = *reinterpret_cast<const f32x4 *>(vr), vb = *reinterpret_cast<const f32x4 *>(vr + 16);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[v][r] *= alpha;
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[v] = mfma_f32(va[r], s0[r], o[v]);
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[v] = mfma_f32(vb[r], s1[r], o[v]);
        }
    }
  }
  l = sum_rows(l);
  const int qi = q0 + wave * 16 + col;
  if (qi >= a.rows)
    return;
  const float f = sigmoid_f(proj[(int64_t)qi * a.ld + a.gate_at + h]) / l;
  T *dst = out + (int64_t)qi * a.out_ld + (int64_t)h * a.vdim;
#pragma unroll
  for (int v = 0; v < NV; ++v)
    if (v < nv) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = v * 16 + quad * 4 + r;
        if (c < a.vdim)
          store_act<T>(dst + c, o[v][r] * f);
      }
    }
}

bool shape_ok(const LatentShape &s) {
  return s.heads > 0 && s.dim > 0 && s.rot_dim >= 0 && s.rot_dim % 2 == 0 && s.vdim > 0 &&
         s.rank > 0 && s.window > 0 && s.ring_mask > 0 && ((s.ring_mask + 1) & s.ring_mask) == 0;
}

size_t part_lds(const LatentShape &s, int kt, int *stride) {
  // rows of the tile start 4 banks apart
  *stride = s.row_elems() + (s.f32 ? 4 : 8);
  return (size_t)(s.f32 ? 4 : 2) * 16 * kt * *stride + 4 * (size_t)16 * (s.row_elems() + 4) +
         4 * (size_t)kt * 4 * 256;
}
constexpr size_t kLdsLimit = 156 * 1024;

} // namespace

LatentCut latent_step_cut(const LatentShape &s, int span) {
  span = std::min(span, s.window);
  int kt = span <= 1024 ? 1 : span <= 4096 ? 2 : 4, stride;
  while (kt > 1 && part_lds(s, kt, &stride) > kLdsLimit)
    kt /= 2;
  return {kt, (int)ceil_div(span, 16 * kt)};
}

int latent_max_chunks(const LatentShape &s) {
  int most = 1; // the cuts change at these spans
  for (int span : {1024, 4096, s.window})
    most = std::max(most, latent_step_cut(s, span).chunks);
  return most;
}

int launch_latent_step(const LatentStep &a, int span, hipStream_t stream) {
  const LatentShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.norm_w && a.turns && a.pos && a.cache && a.query &&
                 a.part_acc && a.part_ml && a.out && span > 0,
             "latent_step: bad argument");
  BH_REQUIRE(a.uk_t.K == s.dim && a.uk_t.N == s.heads * s.rank16() && a.uv.K == s.rank &&
                 a.uv.N == s.heads * s.vdim16(),
             "latent_step: matrix shapes");
  const int re = s.row_elems();
  {
    LatentQueryArgs q{s.heads, s.dim, s.rot_dim, s.rank, re, s.ring_mask, a.dkv_at,
                      s.rank16() / 16, a.uk_t.ktiles, s.scale, s.eps, a.norm_w, a.turns, a.pos,
                      a.cache, a.query};
    const dim3 grid((unsigned)(s.heads + 1), (unsigned)ceil_div(q.uk_groups, kStepWaves));
    const size_t lds = sizeof(float) * (size_t)q.uk_ktiles * kBfTileK;
    BH_REQUIRE(lds <= 60 * 1024, "latent_step: head of %d values", s.dim);
    if (s.f32)
      hipLaunchKernelGGL(latent_query_kernel<float>, grid, dim3(kStepThreads), lds, stream,
                         a.uk_t.tiles, a.proj, q);
    else
      hipLaunchKernelGGL(latent_query_kernel<bf16_bits>, grid, dim3(kStepThreads), lds, stream,
                         a.uk_t.tiles, a.proj, q);
    BH_CHECK_HIP(hipGetLastError());
  }
  const LatentCut cut = latent_step_cut(s, span);
  {
    LatentPartArgs p{s.heads, s.heads16(), s.rank16(), re, s.window, s.ring_mask, 0, a.pos,
                     a.part_acc, a.part_ml};
    const size_t lds = part_lds(s, cut.key_tiles, &p.lds_stride);
    BH_REQUIRE(lds <= kLdsLimit, "latent_step: a cache row of %d values does not fit LDS", re);
    const dim3 grid((unsigned)cut.chunks, (unsigned)(s.heads16() / 16));
#define BH_PART(T, KT)                                                                           \
  do {                                                                                           \
    static DynLdsOnce once;                                                                      \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)latent_part_kernel<T, KT>, (int)kLdsLimit)); \
    hipLaunchKernelGGL((latent_part_kernel<T, KT>), grid, dim3(KT * 256), lds, stream,           \
                       static_cast<const T *>(a.cache), a.query, p);                             \
  } while (0)
    if (s.f32) {
      if (cut.key_tiles == 1) BH_PART(float, 1);
      else if (cut.key_tiles == 2) BH_PART(float, 2);
      else BH_PART(float, 4);
    } else {
      if (cut.key_tiles == 1) BH_PART(bf16_bits, 1);
      else if (cut.key_tiles == 2) BH_PART(bf16_bits, 2);
      else BH_PART(bf16_bits, 4);
    }
#undef BH_PART
    BH_CHECK_HIP(hipGetLastError());
  }
  {
    LatentFoldArgs f{s.heads16(), s.rank, s.rank16(), s.vdim, s.vdim16() / 16, a.uv.ktiles,
                     cut.chunks, a.part_acc, a.part_ml, a.proj + a.gate_at, a.out};
    const size_t lds = sizeof(float) * ((size_t)a.uv.ktiles * kBfTileK + (size_t)cut.chunks);
    BH_REQUIRE(lds <= kLdsLimit, "latent_step: %d partials do not fit LDS", cut.chunks);
    static DynLdsOnce once;
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)latent_value_kernel, (int)kLdsLimit));
    hipLaunchKernelGGL(latent_value_kernel, dim3((unsigned)s.heads, (unsigned)ceil_div(f.groups, 4)),
                       dim3(kStepThreads), lds, stream, a.uv.tiles, f);
    BH_CHECK_HIP(hipGetLastError());
  }
  return BUDDY_HIP_OK;
}

int latent_first_visible(const LatentShape &s, int start) { return std::max(0, start - s.window + 1); }

int launch_latent_rows(const LatentRows &a, hipStream_t stream) {
  const LatentShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.norm_w && a.turns && a.cache && a.rows > 0 && a.start >= 0 &&
                 a.rows + std::min(a.start, s.window - 1) <= s.ring_mask + 1,
             "latent_rows: bad argument (%d rows from %d)", a.rows, a.start);
  LatentRowsArgs r{s.heads, s.dim, s.rot_dim, s.rank, s.row_elems(), s.ring_mask, a.dkv_at, a.ld,
                   a.start, s.scale, s.eps, a.norm_w, a.turns};
  const size_t lds = sizeof(float) * (size_t)std::max(2, s.rot_dim);
  if (s.f32)
    hipLaunchKernelGGL(latent_rows_kernel<float>, dim3(a.rows), dim3(256), lds, stream, a.proj,
                       static_cast<float *>(a.cache), r);
  else
    hipLaunchKernelGGL(latent_rows_kernel<bf16_bits>, dim3(a.rows), dim3(256), lds, stream, a.proj,
                       static_cast<bf16_bits *>(a.cache), r);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

namespace {
template <typename T, int NV>
int launch_attention(const LatentRows &a, const LatentAttnArgs &p, int waves, size_t lds,
                     hipStream_t stream) {
  static DynLdsOnce once;
  BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)latent_attention_kernel<T, NV>, (int)kLdsLimit));
  hipLaunchKernelGGL((latent_attention_kernel<T, NV>),
                     dim3((unsigned)ceil_div(a.rows, 16 * waves), (unsigned)a.s.heads),
                     dim3(waves * 64), lds, stream, a.proj, static_cast<const T *>(a.keys),
                     static_cast<const T *>(a.values_t), static_cast<const T *>(a.cache),
                     static_cast<T *>(a.out), p);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}
template <typename T>
int launch_attention_any(const LatentRows &a, const LatentAttnArgs &p, int waves, size_t lds,
                         hipStream_t stream) {
  const int nv = p.vdim16 / 16;
  if (nv <= 4)
    return launch_attention<T, 4>(a, p, waves, lds, stream);
  if (nv <= 8)
    return launch_attention<T, 8>(a, p, waves, lds, stream);
  if (nv <= 16)
    return launch_attention<T, 16>(a, p, waves, lds, stream);
  BH_REQUIRE(nv <= 32, "latent_attention: value heads of %d", a.s.vdim);
  return launch_attention<T, 32>(a, p, waves, lds, stream);
}
} // namespace

int launch_latent_attention(const LatentRows &a, hipStream_t stream) {
  const LatentShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.cache && a.keys && a.values_t && a.out && a.rows > 0 &&
                 a.start >= 0 && a.first == latent_first_visible(s, a.start) &&
                 a.value_ld % kTileKeys == 0 && a.value_ld >= a.start + a.rows - a.first,
             "latent_attention: bad argument");
  const int esz = s.f32 ? 4 : 2, pad = 16 / esz;
  LatentAttnArgs p{s.heads, s.dim, s.dim16(), s.rot_dim, s.vdim, s.vdim16(), s.rank, s.row_elems(),
                   s.window, s.ring_mask, a.ld, a.gate_at, a.rows, a.start, a.first, a.value_ld,
                   a.out_ld, 0, 0, 0};
  p.kd = (int)round_up(s.dim16() + s.rot_dim, 32);
  p.k_stride = p.kd + pad;
  p.v_stride = kTileKeys + pad;
  int waves = 4;
  auto lds_bytes = [&](int w) {
    return (size_t)esz * ((size_t)(16 * w + kTileKeys) * p.k_stride + (size_t)s.vdim16() * p.v_stride);
  };
  while (waves > 1 && (lds_bytes(waves) > kLdsLimit || a.rows <= 16 * (waves / 2)))
    waves /= 2;
  const size_t lds = lds_bytes(waves);
  BH_REQUIRE(lds <= kLdsLimit, "latent_attention: heads of %d + %d values do not fit LDS", p.kd,
             s.vdim);
  return s.f32 ? launch_attention_any<float>(a, p, waves, lds, stream)
               : launch_attention_any<bf16_bits>(a, p, waves, lds, stream);
}

} // namespace bh
