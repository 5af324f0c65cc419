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
#include "flash_tile.h"
#include "rotary.h"

#include <algorithm>

namespace bh {
namespace {

constexpr int kStepThreads = 512, kStepWaves = 8;

// eight bfloat16 weights times eight values in LDS
__device__ __forceinline__ float dot_run(const uint4 w, const float *x, float acc) {
  acc = fmaf(bf_lo(w.x), x[0], acc);
  acc = fmaf(bf_hi(w.x), x[1], acc);
  acc = fmaf(bf_lo(w.y), x[2], acc);
  acc = fmaf(bf_hi(w.y), x[3], acc);
  acc = fmaf(bf_lo(w.z), x[4], acc);
  acc = fmaf(bf_hi(w.z), x[5], acc);
  acc = fmaf(bf_lo(w.w), x[6], acc);
  acc = fmaf(bf_hi(w.w), x[7], acc);
  return acc;
}

struct LatentQueryArgs {
  int heads, rot8, rank, row_elems, ring_mask, dkv_at;
  float scale, eps;
  const float *norm_w;
  const double *turns;
  void *cache;
  float *query;
};

// Grid (heads + 1, parts): the last row of workgroups writes the token's cache
// row, the others a head's query in the space of a cache row.
template <typename T>
__global__ void __launch_bounds__(kStepThreads)
latent_query_kernel(const uint4 *__restrict__ uk, const float *__restrict__ proj,
                    const int *__restrict__ pos, int uk_groups, int uk_ktiles, int dim, int rot_dim,
                    LatentQueryArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, half = rot_dim / 2;
  const int p = *pos;
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
      if (i < rot_dim) {
        const int f = i < half ? i : i - half;
        float c, s;
        rotation(a.turns[f], p, c, s);
        const float u = d[a.rank + f], w = d[a.rank + f + half];
        v = i < half ? u * c - w * s : w * c + u * s;
      } else if (i >= a.rot8 && i < a.rot8 + a.rank) {
        v = d[i - a.rot8] * r * a.norm_w[i - a.rot8];
      }
      store_act<T>(row + i, v);
    }
    return;
  }
  const float *q = proj + (int64_t)h * (dim + rot_dim);
  float *out = a.query + (int64_t)h * a.row_elems;
  const int Kp = uk_ktiles * kBfTileK;
  // one channel group per wavefront, its first tiles asked for ahead of the query
  const int g = blockIdx.y * kStepWaves + wave, gl = min(g, uk_groups - 1);
  const uint4 *wp = uk + ((int64_t)h * uk_groups + gl) * uk_ktiles * 64 + lane;
  constexpr int kAhead = 4;
  uint4 w[kAhead];
#pragma unroll
  for (int u = 0; u < kAhead; ++u)
    w[u] = wp[(int64_t)min(u, uk_ktiles - 1) * 64];
  for (int i = tid; i < Kp; i += kStepThreads)
    lds[i] = i < dim ? q[i] : 0.f;
  if (blockIdx.y == 0)
    for (int i = tid; i < a.row_elems; i += kStepThreads) {
      if (i >= a.rot8 && i < a.rot8 + a.rank)
        continue; // the latent part, below
      float v = 0.f;
      if (i < rot_dim) {
        const int f = i < half ? i : i - half;
        float c, s;
        rotation(a.turns[f], p, c, s);
        const float u = q[dim + f], x = q[dim + f + half];
        v = (i < half ? u * c - x * s : x * c + u * s) * a.scale;
      }
      out[i] = v;
    }
  __syncthreads();
  float acc = 0.f;
  for (int t = 0; t < uk_ktiles; t += kAhead) {
    if (t > 0) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        w[u] = wp[(int64_t)min(t + u, uk_ktiles - 1) * 64];
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u)
      if (t + u < uk_ktiles)
        acc = dot_run(w[u], lds + (t + u) * kBfTileK + (lane >> 4) * 8, acc);
  }
  acc = sum_rows(acc);
  const int l = g * 16 + lane;
  if (lane < 16 && l < a.rank)
    out[a.rot8 + l] = acc * a.scale;
}

struct LatentPartArgs {
  int heads16, rank16, rot8;
  float *acc, *ml;
};

// Grid (chunks, heads16 / 16).  WK wavefronts per key tile of 16 positions: each
// takes its share of the score's k, then all share out the latent dimensions.
// S^T = C . Q^T leaves a lane with 4 keys of one head, which is the B operand of
// O^T += C^T . P^T as it lies.
template <typename T, int KT, int WK>
__global__ void __launch_bounds__(KT * WK * 64)
latent_part_kernel(const T *__restrict__ cache, const float *__restrict__ query,
                   const int *__restrict__ pos, int row_elems, int window, int ring_mask,
                   int lds_stride, LatentPartArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char raw[];
  constexpr int kKeys = KT * 16;
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  T *ck = reinterpret_cast<T *>(raw);                                            // [kKeys][lds_stride]
  float *sp = reinterpret_cast<float *>(raw + sizeof(T) * kKeys * lds_stride); // [KT][WK][16][16]
  const int head0 = blockIdx.y * 16;
  // this lane's query values: a step of 32 k in every WK-th, the first kQSteps of them
  // in flight together, asked for before the position is known
  constexpr int E = 16 / (int)sizeof(T), kQSteps = 20 / WK + (20 % WK != 0), kRows = 16 / WK;
  const int kt = wave / WK, share = wave % WK, steps = row_elems / 32;
  const int runs = row_elems / E;
  // (what columns of heads past the last compute is not used)
  const float *qr = query + (int64_t)(head0 + col) * row_elems + quad * 8;
  Frag<float> qf[kQSteps];
#pragma unroll
  for (int i = 0; i < kQSteps; ++i)
    qf[i].load(qr + min(share + i * WK, steps - 1) * 32);
  const int p = *pos;
  const int lo = max(0, p - window + 1), n = p - lo + 1;
  const int k0 = blockIdx.x * kKeys;
  float *ml = a.ml + ((int64_t)blockIdx.x * a.heads16 + head0) * 2;
  if (k0 >= n) { // nothing visible: an empty partial
    if (tid < 16) {
      ml[tid * 2] = -INFINITY;
      ml[tid * 2 + 1] = 0.f;
    }
    return;
  }
  for (int c0 = 0; c0 < runs; c0 += 128) {
    u32x4 v[kRows][2];
    const int ca = min(c0 + lane, runs - 1), cb = min(c0 + 64 + lane, runs - 1);
#pragma unroll
    for (int r = 0; r < kRows; ++r) { // a row past the last key repeats it, masked below
      const T *row = cache + (int64_t)((lo + min(k0 + wave * kRows + r, n - 1)) & ring_mask) * row_elems;
      v[r][0] = *reinterpret_cast<const u32x4 *>(row + ca * E);
      v[r][1] = *reinterpret_cast<const u32x4 *>(row + cb * E);
    }
#pragma unroll
    for (int r = 0; r < kRows; ++r) {
      T *row = ck + (wave * kRows + r) * lds_stride;
      *reinterpret_cast<u32x4 *>(row + ca * E) = v[r][0];
      *reinterpret_cast<u32x4 *>(row + cb * E) = v[r][1];
    }
  }
  __syncthreads();
  {
    f32x4 s{0.f, 0.f, 0.f, 0.f};
    const T *kr = ck + (kt * 16 + col) * lds_stride + quad * 8;
    auto score = [&](int t, const Frag<float> &q) {
      Frag<T> kf;
      kf.load(kr + t * 32);
      Frag<float> kw;
      if constexpr (sizeof(T) == 2)
        kw = widen(kf.v);
      else
        kw = kf;
      s = mfma32(kw, q, s);
    };
#pragma unroll
    for (int i = 0; i < kQSteps; ++i)
      if (share + i * WK < steps)
        score(share + i * WK, qf[i]);
    for (int t = share + kQSteps * WK; t < steps; t += WK) {
      Frag<float> q;
      q.load(qr + t * 32);
      score(t, q);
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
      for (int w = 0; w < WK; ++w)
        s += sp[(((kt * WK + w) * 16) + key) * 16 + col];
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
  for (int lt = wave; lt < a.rank16 / 16; lt += KT * WK) {
    f32x4 o{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kt = 0; kt < KT; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        o = mfma_f32(load_act<T>(ck + (kt * 16 + quad * 4 + r) * lds_stride + a.rot8 + lt * 16 + col),
                     pr[kt][r], o);
    *reinterpret_cast<f32x4 *>(acc + lt * 16 + quad * 4) = o;
  }
}

struct LatentFoldArgs {
  int rank, vdim;
  const float *gate;
  float *out;
};

// Grid (heads, parts of the value channels): folds the partials of a head, then
// four channel groups of its value matrix, k in two slices.
__global__ void __launch_bounds__(kStepThreads)
latent_value_kernel(const uint4 *__restrict__ uv, const float *__restrict__ part_acc,
                    const float *__restrict__ part_ml, int groups, int ktiles, int chunks, int heads16,
                    int rank16, LatentFoldArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float part[kStepWaves][16];
  __shared__ float red[2][kStepWaves];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x;
  const int Kp = ktiles * kBfTileK;
  float *x = lds, *wt = lds + Kp; // [Kp], [chunks]
  const int gi = wave >> 1, slice = wave & 1;
  const int g = blockIdx.y * 4 + gi, gl = min(g, groups - 1);
  const int half = (ktiles + 1) / 2;
  const int t0 = slice * half, t1 = min(t0 + half, ktiles);
  const uint4 *wp = uv + ((int64_t)h * groups + gl) * ktiles * 64 + lane;
  // loads return in order: what is needed first is asked for first
  float2 ml{-INFINITY, 0.f}; // (maximum, sum) of this thread's first chunk
  if (tid < chunks)
    ml = *reinterpret_cast<const float2 *>(part_ml + ((int64_t)tid * heads16 + h) * 2);
  // the partials in four parts: 128 threads take four latent dimensions each of every
  // fourth chunk, eight in flight, the first eight before their weights are known
  const int64_t step = (int64_t)heads16 * rank16;
  const int part4 = tid >> 7, i0 = (tid & 127) * 4;
  auto partials = [&](int i, int c, f32x4 (&v)[8]) {
    const float *q = part_acc + (int64_t)h * rank16 + i;
#pragma unroll
    for (int u = 0; u < 8; ++u)
      v[u] = *reinterpret_cast<const f32x4 *>(q + min(c + u * 4, chunks - 1) * step);
  };
  f32x4 v[8];
  partials(min(i0, rank16 - 4), part4, v);
  constexpr int kAhead = 8;
  uint4 w[kAhead];
#pragma unroll
  for (int u = 0; u < kAhead; ++u)
    w[u] = wp[(int64_t)min(t0 + u, ktiles - 1) * 64];
  float m = ml.x;
  for (int c = tid + kStepThreads; c < chunks; c += kStepThreads)
    m = fmaxf(m, part_ml[((int64_t)c * heads16 + h) * 2]);
  m = wave_max(m);
  if (lane == 0)
    red[0][wave] = m;
  __syncthreads();
#pragma unroll
  for (int i = 0; i < kStepWaves; ++i)
    m = fmaxf(m, red[0][i]);
  float l = 0.f;
  for (int c = tid; c < chunks; c += kStepThreads) {
    if (c != tid)
      ml = *reinterpret_cast<const float2 *>(part_ml + ((int64_t)c * heads16 + h) * 2);
    const float e = ml.y > 0.f ? fast_exp(ml.x - m) : 0.f;
    wt[c] = e;
    l = fmaf(e, ml.y, l);
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
  float *fold = wt + ((chunks + 3) & ~3); // [4][Kp]
  for (int i = i0; i < Kp; i += 512) {
    f32x4 o{0.f, 0.f, 0.f, 0.f};
    if (i < rank16) {
      for (int c = part4; c < chunks; c += 32) {
        if (i != i0 || c != part4)
          partials(i, c, v);
#pragma unroll
        for (int u = 0; u < 8; ++u) {
          const float e = c + u * 4 < chunks ? wt[min(c + u * 4, chunks - 1)] : 0.f;
#pragma unroll
          for (int j = 0; j < 4; ++j) // an empty partial's accumulators were never written
            o[j] = e != 0.f ? fmaf(e, v[u][j], o[j]) : o[j];
        }
      }
    }
    *reinterpret_cast<f32x4 *>(fold + part4 * Kp + i) = o;
  }
  __syncthreads();
  for (int i = tid; i < Kp; i += kStepThreads)
    x[i] = i < a.rank ? ((fold[i] + fold[Kp + i]) + (fold[2 * Kp + i] + fold[3 * Kp + i])) * inv : 0.f;
  __syncthreads();
  float acc = 0.f;
  const float *xp = x + (lane >> 4) * 8;
  for (int t = t0; t < t1; t += kAhead) {
    if (t > t0) {
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        w[u] = wp[(int64_t)min(t + u, ktiles - 1) * 64];
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u)
      if (t + u < t1)
        acc = dot_run(w[u], xp + (t + u) * kBfTileK, acc);
  }
  acc = sum_rows(acc);
  if (lane < 16)
    part[wave][lane] = acc;
  __syncthreads();
  if (tid < 64) {
    const int gg = blockIdx.y * 4 + (tid >> 4), v = gg * 16 + (tid & 15);
    if (gg < groups && v < a.vdim)
      a.out[(int64_t)h * a.vdim + v] =
          (part[(tid >> 4) * 2][tid & 15] + part[(tid >> 4) * 2 + 1][tid & 15]) *
          sigmoid_f(a.gate[h]);
  }
}

// ---- many tokens -----------------------------------------------------------------

struct LatentRowsArgs {
  int heads, dim, dim16, rot_dim, rot8, rank, row_elems, key_elems, ring_mask, dkv_at, ld, start;
  float scale, eps;
  const float *norm_w;
  const double *turns;
};

// One workgroup per token: its cache row and its queries.
template <typename T>
__global__ void __launch_bounds__(256)
latent_rows_kernel(const float *__restrict__ proj, T *__restrict__ cache, T *__restrict__ queries,
                   LatentRowsArgs a) {
  extern __shared__ float lds[]; // cos, sin of this position
  __shared__ float red[4];
  const int tid = threadIdx.x, half = a.rot_dim / 2;
  const int p = a.start + blockIdx.x;
  const float *row = proj + (int64_t)blockIdx.x * a.ld;
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
  // value j of the rotated vector that starts at v
  auto turned = [&](const float *v, int j) {
    const int f = j < half ? j : j - half;
    const float u = v[f], w = v[f + half], c = lds[f], s = lds[half + f];
    return j < half ? u * c - w * s : w * c + u * s;
  };
  T *out = cache + (int64_t)(p & a.ring_mask) * a.row_elems;
  for (int i = tid; i < a.row_elems; i += 256) {
    float v = 0.f;
    if (i < a.rot_dim)
      v = turned(d + a.rank, i);
    else if (i >= a.rot8 && i < a.rot8 + a.rank)
      v = d[i - a.rot8] * r * a.norm_w[i - a.rot8];
    store_act<T>(out + i, v);
  }
  T *qo = queries + (int64_t)blockIdx.x * a.heads * a.key_elems;
  for (int h = tid >> 6; h < a.heads; h += 4) {
    const float *q = row + (int64_t)h * (a.dim + a.rot_dim);
    for (int k = tid & 63; k < a.key_elems; k += 64) {
      float v = 0.f;
      if (k < a.dim)
        v = q[k] * a.scale;
      else if (k >= a.dim16 && k < a.dim16 + a.rot_dim)
        v = turned(q + a.dim, k - a.dim16) * a.scale;
      store_act<T>(qo + (int64_t)h * a.key_elems + k, v);
    }
  }
}

struct LatentAttnArgs {
  int heads, dim16, rot8, vdim, nv, row_elems, window, ring_mask;
  int ld, gate_at, rows, start, first, value_ld, out_ld;
  int kd; // elements of a query
};

// Grid (heads, query blocks).  A wavefront owns 16 queries, the workgroup's four
// share tiles of kKeys keys through LDS; the next tile is on its way in registers
// meanwhile.
// NK: 32-element steps of a key, NV: 16-channel groups of a value, at most; smaller
// heads are padded with zeros (keys) or with rows whose results are not stored
// (values), so that the loop has no branches.
template <typename T, int NK, int NV>
__global__ void __launch_bounds__(256, NV <= 8 ? 2 : 1)
latent_attention_kernel(const T *__restrict__ queries, const T *__restrict__ keys,
                        const T *__restrict__ values_t, const T *__restrict__ cache,
                        const float *__restrict__ proj, T *__restrict__ out, LatentAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned char raw[];
  constexpr int E = 16 / (int)sizeof(T), KEYS = KeyTile<T>::kKeys;
  constexpr int KL = NK, VL = (NV + 1) / 2; // 16-byte loads per thread and tile
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x;
  constexpr int kBlock = 64;
  const int q0 = (gridDim.y - 1 - blockIdx.y) * kBlock; // long blocks first
  constexpr int kKeyRow = Flash<T, NK, NV>::kKeyRow, kValueRow = Flash<T, NK, NV>::kValueRow;
  T *kt = reinterpret_cast<T *>(raw); // [KEYS][kKeyRow]
  T *vt = kt + KEYS * kKeyRow;        // [16 * NV][kValueRow]

  // this lane's query, also as a key index, and its fragments
  const int qi = q0 + wave * 16 + col, my_q = a.start + qi - a.first;
  Frag<T> qf[NK];
  const T *q = queries + ((int64_t)min(qi, a.rows - 1) * a.heads + h) * a.kd + quad * 8;
#pragma unroll
  for (int t = 0; t < NK; ++t) {
    if (t * 32 < a.kd)
      qf[t].load(q + t * 32);
    else
      qf[t] = Frag<T>{};
  }
  const int nkeys = a.start + a.rows - a.first;
  const int last_q = min(q0 + kBlock, a.rows) - 1;
  const int key_hi = a.start + last_q - a.first;                               // last visible
  const int key_lo = max(0, a.start + q0 - a.window + 1 - a.first) & ~(KEYS - 1); // tile of the first
  const int wave_q0 = a.start + q0 + wave * 16 - a.first, wave_q1 = wave_q0 + 15;

  // the 16-byte runs this thread moves.  A key's runs: its head's part, the shared
  // rotated part; the rest of the row in LDS stays zero.
  const int runs_head = a.dim16 / E, runs = runs_head + a.rot8 / E;
  const T *ksrc[KL];
  int kkey[KL], kdst[KL], kstep[KL];
  bool kring[KL];
#pragma unroll
  for (int i = 0; i < KL; ++i) {
    const int id = min(i * 256 + tid, KEYS * runs - 1); // past the end: the last one again
    const int r = id / runs, c = id - r * runs;
    kkey[i] = r;
    kdst[i] = r * kKeyRow + (c < runs_head ? c * E : a.dim16 + (c - runs_head) * E);
    kring[i] = c >= runs_head;
    kstep[i] = c < runs_head ? a.heads * a.dim16 : a.row_elems;
    ksrc[i] = c < runs_head ? keys + h * a.dim16 + c * E : cache + (c - runs_head) * E;
  }
  const T *vsrc[VL];
  int vdst[VL], vcol[VL];
  const int vruns = 16 * a.nv * 8;
#pragma unroll
  for (int i = 0; i < VL; ++i) {
    const int id = min(i * 256 + tid, vruns - 1), r = id >> 3, c = id & 7;
    vsrc[i] = values_t + (int64_t)(h * 16 * a.nv + r) * a.value_ld + c * E;
    vcol[i] = c * E;
    vdst[i] = Flash<T, NK, NV>::value_at(r, c);
  }
  u32x4 kr[KL], vr[VL];
  auto fetch = [&](int k0, u32x4 (&kr)[KL], u32x4 (&vr)[VL]) {
#pragma unroll
    for (int i = 0; i < KL; ++i) {
      const int k = min(k0 + kkey[i], nkeys - 1); // masked past the end
      const int row = kring[i] ? (a.first + k) & a.ring_mask : k;
      kr[i] = *reinterpret_cast<const u32x4 *>(ksrc[i] + (int64_t)row * kstep[i]);
    }
#pragma unroll
    for (int i = 0; i < VL; ++i)
      vr[i] = *reinterpret_cast<const u32x4 *>(vsrc[i] + k0);
  };
  fetch(key_lo, kr, vr);
  if (runs * E < NK * 32) { // the padding of the keys
    const int pad = NK * 32 - runs * E, at = a.dim16 + a.rot8;
    for (int i = tid; i < KEYS * pad; i += 256)
      kt[(i / pad) * kKeyRow + at + i % pad] = 0;
  }

  Flash<T, NK, NV> flash;
  for (int k0 = key_lo; k0 <= key_hi; k0 += KEYS) {
    __syncthreads(); // the previous tile has been read
#pragma unroll
    for (int i = 0; i < KL; ++i)
      *reinterpret_cast<u32x4 *>(kt + kdst[i]) = kr[i];
    if (k0 + KEYS > nkeys) { // value columns past the last key hold anything
#pragma unroll
      for (int i = 0; i < VL; ++i) {
        const int keep = nkeys - k0 - vcol[i];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          if constexpr (sizeof(T) == 4)
            vr[i][j] = j < keep ? vr[i][j] : 0u;
          else
            vr[i][j] = 2 * j + 1 < keep ? vr[i][j] : 2 * j < keep ? vr[i][j] & 0xffffu : 0u;
        }
      }
    }
#pragma unroll
    for (int i = 0; i < VL; ++i)
      Flash<T, NK, NV>::store_value(vt, vdst[i], vr[i]);
    __syncthreads();
    fetch(min(k0 + KEYS, (nkeys - 1) & ~(KEYS - 1)), kr, vr);
    if (k0 > wave_q1 || k0 + KEYS - 1 <= wave_q0 - a.window)
      continue; // nothing of this tile is visible to this wavefront
    const bool whole = k0 + KEYS - 1 <= wave_q0 && wave_q1 - k0 < a.window;
    flash.tile(kt, vt, qf, whole, my_q - k0, a.window);
  }
  const float sum = sum_rows(flash.l);
  if (qi >= a.rows)
    return;
  const float f = sigmoid_f(proj[(int64_t)qi * a.ld + a.gate_at + h]) / sum;
  T *dst = out + (int64_t)qi * a.out_ld + (int64_t)h * a.vdim;
#pragma unroll
  for (int v = 0; v < NV; ++v)
    if (v < a.nv) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = v * 16 + quad * 4 + r;
        if (c < a.vdim)
          store_act<T>(dst + c, flash.o[v][r] * f);
      }
    }
}

bool shape_ok(const LatentShape &s) {
  return s.heads > 0 && s.dim > 0 && s.rot_dim >= 0 && s.rot_dim % 2 == 0 && s.vdim > 0 &&
         s.rank > 0 && s.window > 0 && s.ring_mask > 0 && ((s.ring_mask + 1) & s.ring_mask) == 0;
}

constexpr int part_waves(int key_tiles) { return key_tiles <= 2 ? 8 : 4; } // per key tile
size_t part_lds(const LatentShape &s, int kt, int *stride) {
  // rows of the tile start 4 banks apart
  *stride = s.row_elems() + (s.f32 ? 4 : 8);
  return (size_t)(s.f32 ? 4 : 2) * 16 * kt * *stride + 4 * (size_t)kt * part_waves(kt) * 256;
}
constexpr size_t kLdsLimit = 156 * 1024;

} // namespace

LatentCut latent_step_cut(const LatentShape &s, int span) {
  span = std::min(span, s.window);
  int kt = span <= 2048 ? 1 : span <= 8192 ? 2 : 4, stride;
  while (kt > 1 && part_lds(s, kt, &stride) > kLdsLimit)
    kt /= 2;
  return {kt, (int)ceil_div(span, 16 * kt)};
}

int latent_max_chunks(const LatentShape &s) {
  int most = 1; // the cuts change at these spans
  for (int span : {2048, 8192, s.window})
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
    LatentQueryArgs q{s.heads, s.rot8(), s.rank, re, s.ring_mask, a.dkv_at, s.scale, s.eps, a.norm_w,
                      a.turns, a.cache, a.query};
    const int groups = s.rank16() / 16;
    const dim3 grid((unsigned)(s.heads + 1), (unsigned)ceil_div(groups, kStepWaves));
    const size_t lds = sizeof(float) * (size_t)a.uk_t.ktiles * kBfTileK;
    BH_REQUIRE(lds <= 60 * 1024, "latent_step: head of %d values", s.dim);
    if (s.f32)
      hipLaunchKernelGGL(latent_query_kernel<float>, grid, dim3(kStepThreads), lds, stream,
                         a.uk_t.tiles, a.proj, a.pos, groups, a.uk_t.ktiles, s.dim, s.rot_dim, q);
    else
      hipLaunchKernelGGL(latent_query_kernel<bf16_bits>, grid, dim3(kStepThreads), lds, stream,
                         a.uk_t.tiles, a.proj, a.pos, groups, a.uk_t.ktiles, s.dim, s.rot_dim, q);
    BH_CHECK_HIP(hipGetLastError());
  }
  const LatentCut cut = latent_step_cut(s, span);
  {
    LatentPartArgs p{s.heads16(), s.rank16(), s.rot8(), a.part_acc, a.part_ml};
    int stride = 0;
    const size_t lds = part_lds(s, cut.key_tiles, &stride);
    BH_REQUIRE(lds <= kLdsLimit, "latent_step: a cache row of %d values does not fit LDS", re);
    const dim3 grid((unsigned)cut.chunks, (unsigned)(s.heads16() / 16));
#define BH_PART(T, KT)                                                                           \
  do {                                                                                           \
    static DynLdsOnce once;                                                                      \
    constexpr int WK = part_waves(KT);                                                           \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)latent_part_kernel<T, KT, WK>,               \
                                (int)kLdsLimit));                                                \
    hipLaunchKernelGGL((latent_part_kernel<T, KT, WK>), grid, dim3(KT * WK * 64), lds, stream,   \
                       static_cast<const T *>(a.cache), a.query, a.pos, re, s.window,            \
                       s.ring_mask, stride, p);                                                  \
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
    LatentFoldArgs f{s.rank, s.vdim, a.proj + a.gate_at, a.out};
    const int groups = s.vdim16() / 16;
    const size_t lds = sizeof(float) * ((size_t)5 * a.uv.ktiles * kBfTileK + (size_t)round_up(cut.chunks, 4));
    BH_REQUIRE(lds <= kLdsLimit, "latent_step: %d partials do not fit LDS", cut.chunks);
    static DynLdsOnce once;
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)latent_value_kernel, (int)kLdsLimit));
    hipLaunchKernelGGL(latent_value_kernel, dim3((unsigned)s.heads, (unsigned)ceil_div(groups, 4)),
                       dim3(kStepThreads), lds, stream, a.uv.tiles, a.part_acc, a.part_ml, groups,
                       a.uv.ktiles, cut.chunks, s.heads16(), s.rank16(), f);
    BH_CHECK_HIP(hipGetLastError());
  }
  return BUDDY_HIP_OK;
}

int latent_first_visible(const LatentShape &s, int start) { return std::max(0, start - s.window + 1); }

int launch_latent_rows(const LatentRows &a, hipStream_t stream) {
  const LatentShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.norm_w && a.turns && a.cache && a.queries && a.rows > 0 &&
                 a.start >= 0 && a.rows + std::min(a.start, s.window - 1) <= s.ring_mask + 1,
             "latent_rows: bad argument (%d rows from %d)", a.rows, a.start);
  LatentRowsArgs r{s.heads, s.dim, s.dim16(), s.rot_dim, s.rot8(), s.rank, s.row_elems(),
                   s.key_elems(), s.ring_mask, a.dkv_at, a.ld, a.start, s.scale, s.eps, a.norm_w,
                   a.turns};
  const size_t lds = sizeof(float) * (size_t)std::max(2, s.rot_dim);
  if (s.f32)
    hipLaunchKernelGGL(latent_rows_kernel<float>, dim3(a.rows), dim3(256), lds, stream, a.proj,
                       static_cast<float *>(a.cache), static_cast<float *>(a.queries), r);
  else
    hipLaunchKernelGGL(latent_rows_kernel<bf16_bits>, dim3(a.rows), dim3(256), lds, stream, a.proj,
                       static_cast<bf16_bits *>(a.cache), static_cast<bf16_bits *>(a.queries), r);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

namespace {
template <typename T, int NK, int NV>
int launch_attention(const LatentRows &a, const LatentAttnArgs &p, hipStream_t stream) {
  constexpr int E = 16 / (int)sizeof(T), KEYS = KeyTile<T>::kKeys;
  constexpr size_t lds = sizeof(T) * ((size_t)KEYS * (NK * 32 + E) + (size_t)16 * NV * (KEYS + E));
  static_assert(lds <= kLdsLimit, "the tiles must fit LDS");
  static DynLdsOnce once;
  BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)latent_attention_kernel<T, NK, NV>, (int)kLdsLimit));
  hipLaunchKernelGGL((latent_attention_kernel<T, NK, NV>),
                     dim3((unsigned)a.s.heads, (unsigned)ceil_div(a.rows, 64)), dim3(256), lds,
                     stream, static_cast<const T *>(a.queries), static_cast<const T *>(a.keys),
                     static_cast<const T *>(a.values_t), static_cast<const T *>(a.cache), a.proj,
                     static_cast<T *>(a.out), p);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}
template <typename T>
int launch_attention_any(const LatentRows &a, const LatentAttnArgs &p, hipStream_t stream) {
  const int nk = p.kd / 32;
  BH_REQUIRE(nk <= 18 && p.nv <= 32, "latent_attention: heads of %d and %d values", p.kd, a.s.vdim);
  if (nk <= 2 && p.nv <= 2)
    return launch_attention<T, 2, 2>(a, p, stream);
  if (nk <= 4 && p.nv <= 4)
    return launch_attention<T, 4, 4>(a, p, stream);
  if (nk <= 6 && p.nv <= 8)
    return launch_attention<T, 6, 8>(a, p, stream);
  if (nk <= 10 && p.nv <= 16)
    return launch_attention<T, 10, 16>(a, p, stream);
  return launch_attention<T, 18, 32>(a, p, stream);
}
} // namespace

int launch_latent_attention(const LatentRows &a, hipStream_t stream) {
  const LatentShape &s = a.s;
  BH_REQUIRE(shape_ok(s) && a.proj && a.cache && a.queries && a.keys && a.values_t && a.out &&
                 a.rows > 0 && a.start >= 0 && a.first == latent_first_visible(s, a.start) &&
                 a.value_ld % kLatentKeyTile == 0 && a.value_ld >= a.start + a.rows - a.first,
             "latent_attention: bad argument");
  LatentAttnArgs p{s.heads, s.dim16(), s.rot8(), s.vdim, s.vdim16() / 16, s.row_elems(), s.window,
                   s.ring_mask, a.ld, a.gate_at, a.rows, a.start, a.first, a.value_ld, a.out_ld,
                   s.key_elems()};
  return s.f32 ? launch_attention_any<float>(a, p, stream)
               : launch_attention_any<bf16_bits>(a, p, stream);
}

} // namespace bh
