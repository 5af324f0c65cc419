// delta_rule.hip -- the gated delta rule: token by token, and a prompt in chunks.
//
// Chunks of 64 tokens, four blocks of 16.  With G_t the product of the decays from the
// chunk's first token to t (per key channel) and S0 the state ahead of the chunk, the
// writes u solve
//   u_t + beta_t sum_{s<t} a_ts u_s = beta_t (v_t - S0^T (G_t k_t)),
//   a_ts = sum_d k_t k_s G_t / G_s,
// so u = U - W S0 with W and U free of the state, and
//   o_t = S0^T (G_t q_t) + sum_{s<=t} b_ts u_s,   b_ts = sum_d q_t k_s G_t / G_s,
//   S = diag(G_last) S0 + sum_s (G_last / G_s k_s) u_s^T.
// Quotients of G are taken of logarithms that are summed within a block, and between
// blocks through the border of the later one, so that every factor is at most 1 however
// strong a decay is.  f32 throughout.
#include "delta_rule.h"
#include "bf16_dev.h"

#include <algorithm>

namespace bh {
namespace {

constexpr float kUnitEps = 1e-6f; // of the unit vectors

// log(1 + e^z); what rounding 1 + e loses of a small e is made up for by e / ((1 + e) - 1)
__device__ __forceinline__ float softplus_f(float z) {
  const float e = fast_exp(-fabsf(z)), u = 1.0f + e, d = u - 1.0f;
  const float l = __builtin_amdgcn_logf(u) * 0.693147180559945309f;
  return fmaxf(z, 0.f) + (d == 0.f ? e : l * (e / d));
}

__device__ __forceinline__ float dot_run8(uint4 v, const float *x, float acc) {
  acc = fmaf(bf_lo(v.x), x[0], acc);
  acc = fmaf(bf_hi(v.x), x[1], acc);
  acc = fmaf(bf_lo(v.y), x[2], acc);
  acc = fmaf(bf_hi(v.y), x[3], acc);
  acc = fmaf(bf_lo(v.z), x[4], acc);
  acc = fmaf(bf_hi(v.z), x[5], acc);
  acc = fmaf(bf_lo(v.w), x[6], acc);
  return fmaf(bf_hi(v.w), x[7], acc);
}
__device__ __forceinline__ float sum8(float v) { // over eight neighbouring lanes
  v = quad_sum(v);
  return v + __shfl_xor(v, 4, 64);
}
// Row `w` of a bfloat16 matrix times x (LDS), by eight neighbouring lanes; all of them
// get the sum.
__device__ __forceinline__ float row_dot8(const uint16_t *__restrict__ w, const float *x, int n) {
  const int l = threadIdx.x & 7;
  float acc = 0.f;
  if (n % 8 == 0) {
    for (int i = l * 8; i < n; i += 64)
      acc = dot_run8(*reinterpret_cast<const uint4 *>(w + i), x + i, acc);
  } else {
    for (int i = l; i < n; i += 8)
      acc = fmaf(bf_f(w[i]), x[i], acc);
  }
  return sum8(acc);
}

// The convolution of column c at position p; `row`: the projections of that position,
// `have`: how many rows ahead of it lie in the projections (earlier ones are in the ring).
__device__ __forceinline__ float short_conv(const DeltaShape &s, const float *row, int ld, int have,
                                            const float *__restrict__ ring, int p, int c) {
  float v = 0.f;
  for (int b0 = 0; b0 < s.taps; b0 += 4) {
    float e[4], w[4]; // asked for together
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int b = b0 + i;
      const bool some = b < s.taps && b <= p;
      const float *from = !some || b <= have ? row + c - (int64_t)(some ? b : 0) * ld
                                             : ring + (int64_t)((p - b) % s.taps) * s.channels + c;
      e[i] = *from;
      w[i] = s.conv_w[(int64_t)(some ? s.taps - 1 - b : 0) * s.channels + c];
      w[i] = some ? w[i] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      v = fmaf(w[i], e[i], v);
  }
  return silu_f(v);
}

constexpr int kScanThreads = 512, kScanCols = 32, kScanSlices = kScanThreads / kScanCols;

// Grid (heads, slices of 32 value channels).  A thread owns one value channel of N
// consecutive rows of the state, in registers from the first token to the last.  Both
// products with the state are taken of the decayed one: S^T q = (g S)^T q + u (k . q).
template <int N>
__global__ void __launch_bounds__(kScanThreads)
delta_scan_kernel(DeltaRows a) {
  __shared__ __attribute__((aligned(16))) float q[kScanSlices * N], k[kScanSlices * N], decay[kScanSlices * N];
  __shared__ float v[kScanCols], part[2][kScanSlices][kScanCols], dots[3];
  extern __shared__ __attribute__((aligned(16))) float lds[]; // inner decay, inner gate
  const DeltaShape &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, v0 = blockIdx.y * kScanCols;
  const int dim = s.dim, vdim = s.vdim, vcols = min(kScanCols, vdim - v0);
  float *inner_d = lds, *inner_g = lds + ((s.decay_rank + 3) & ~3);
  const int c = tid % kScanCols, slice = tid / kScanCols, d0 = slice * N;
  const bool owner = c < vcols;
  float *S = a.state + (int64_t)h * dim * vdim + v0 + min(c, vcols - 1);
  float st[N];
#pragma unroll
  for (int i = 0; i < N; ++i)
    st[i] = S[(int64_t)min(d0 + i, dim - 1) * vdim];
  // this thread's share of the low-rank projections' outer rows, if they are short: from
  // the same trip to memory
  constexpr int kPreRows = 3, kPreRuns = 2, kRowStep = kScanThreads / 8;
  const bool pre = dim + vcols <= kPreRows * kRowStep && s.decay_rank % 8 == 0 && s.gate_rank % 8 == 0 &&
                   max(s.decay_rank, s.gate_rank) <= kPreRuns * 64;
  auto low_row = [&](int i) { // row i: the decay of channel i, then the gates of the slice
    return i < dim ? s.decay_w + ((int64_t)h * dim + i) * s.decay_rank
                   : s.gate_w + ((int64_t)h * vdim + v0 + i - dim) * s.gate_rank;
  };
  uint4 low[kPreRows][kPreRuns];
  float bias[kPreRows];
  if (pre) {
#pragma unroll
    for (int m = 0; m < kPreRows; ++m) {
      const int i = min((tid >> 3) + m * kRowStep, dim + vcols - 1);
      const uint16_t *w = low_row(i);
      const int n = i < dim ? s.decay_rank : s.gate_rank;
#pragma unroll
      for (int j = 0; j < kPreRuns; ++j) // past the end: times zero
        low[m][j] = *reinterpret_cast<const uint4 *>(w + min((tid & 7) * 8 + j * 64, n - 8));
      bias[m] = s.decay_bias[(int64_t)h * dim + min(i, dim - 1)];
    }
  }
#pragma unroll
  for (int i = 0; i < N; ++i)
    st[i] = owner && d0 + i < dim ? st[i] : 0.f;
  for (int i = dim + tid; i < kScanSlices * N; i += kScanThreads)
    q[i] = k[i] = decay[i] = 0.f;
  const int group = s.heads / s.kv_heads, g = h / group;
  const int p0 = a.pos ? *a.pos : a.start;
  const float speed = s.decay_speed[h], root = sqrtf((float)dim);
  for (int r = 0; r < a.rows; ++r) {
    const float *row = a.proj + (int64_t)r * a.ld;
    const int p = p0 + r;
    for (int i = tid; i < 2 * dim + vcols; i += kScanThreads) {
      const int col = i < dim ? s.q_at + g * dim + i
                      : i < 2 * dim ? s.k_at + g * dim + i - dim
                                    : s.v_at + h * vdim + v0 + i - 2 * dim;
      const float x = short_conv(s, row, a.ld, r, a.ring, p, col);
      (i < dim ? q[i] : i < 2 * dim ? k[i - dim] : v[i - 2 * dim]) = x;
      // no workgroup reads this slot: it is the one of position p - taps
      if (a.rows == 1 && (i >= 2 * dim || (v0 == 0 && h == g * group)))
        a.ring[(int64_t)(p % s.taps) * s.channels + col] = row[col];
    }
    for (int i = tid; i < s.decay_rank; i += kScanThreads)
      inner_d[i] = row[s.decay_at + i];
    for (int i = tid; i < s.gate_rank; i += kScanThreads)
      inner_g[i] = row[s.gate_at + i];
    const float beta = sigmoid_f(row[s.beta_at + h]);
    __syncthreads();
    auto finish_low = [&](int i, float z, float bias_i) {
      if (tid & 7)
        return;
      if (i < dim)
        decay[i] = fast_exp(speed * softplus_f(z + bias_i));
      else
        a.gate[(int64_t)r * s.heads * vdim + (int64_t)h * vdim + v0 + i - dim] = z;
    };
    if (pre) {
#pragma unroll
      for (int m = 0; m < kPreRows; ++m) {
        const int i = (tid >> 3) + m * kRowStep;
        if (i >= dim + vcols)
          break;
        const int n = i < dim ? s.decay_rank : s.gate_rank;
        const float *x = i < dim ? inner_d : inner_g;
        float z = 0.f;
#pragma unroll
        for (int j = 0; j < kPreRuns; ++j) {
          const int k0 = (tid & 7) * 8 + j * 64;
          if (k0 < n)
            z = dot_run8(low[m][j], x + k0, z);
        }
        finish_low(i, sum8(z), bias[m]);
      }
    } else {
      for (int i = tid >> 3; i < dim + vcols; i += kRowStep)
        finish_low(i, row_dot8(low_row(i), i < dim ? inner_d : inner_g, i < dim ? s.decay_rank : s.gate_rank),
                   s.decay_bias[(int64_t)h * dim + min(i, dim - 1)]);
    }
    if (wave < 3) {
      const float *x = wave == 1 ? k : q, *y = wave == 0 ? q : k;
      float t = 0.f;
      for (int i = lane; i < dim; i += 64)
        t = fmaf(x[i], y[i], t);
      t = wave_sum(t);
      if (lane == 0)
        dots[wave] = t;
    }
    __syncthreads();
    const float rq = 1.0f / sqrtf(dots[0] + kUnitEps) / root, rk = 1.0f / sqrtf(dots[1] + kUnitEps);
    float sk = 0.f, sq = 0.f;
#pragma unroll
    for (int i = 0; i < N; i += 4) {
      const f32x4 dd = *reinterpret_cast<const f32x4 *>(decay + d0 + i);
      const f32x4 kk = *reinterpret_cast<const f32x4 *>(k + d0 + i);
      const f32x4 qq = *reinterpret_cast<const f32x4 *>(q + d0 + i);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        st[i + j] *= dd[j];
        sk = fmaf(st[i + j], kk[j], sk);
        sq = fmaf(st[i + j], qq[j], sq);
      }
    }
    part[0][slice][c] = sk;
    part[1][slice][c] = sq;
    __syncthreads();
    sk = sq = 0.f;
#pragma unroll
    for (int i = 0; i < kScanSlices; ++i) {
      sk += part[0][i][c];
      sq += part[1][i][c];
    }
    const float ku = owner ? rk * beta * (v[c] - sk * rk) : 0.f;
#pragma unroll
    for (int i = 0; i < N; i += 4) {
      const f32x4 kk = *reinterpret_cast<const f32x4 *>(k + d0 + i);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        st[i + j] = fmaf(kk[j], ku, st[i + j]);
    }
    if (slice == 0 && owner)
      a.o[(int64_t)r * s.heads * vdim + (int64_t)h * vdim + v0 + c] = rq * fmaf(ku, dots[2], sq);
    if (r + 1 < a.rows)
      __syncthreads(); // the next row takes the places of this one
  }
#pragma unroll
  for (int i = 0; i < N; ++i)
    if (owner && d0 + i < dim)
      S[(int64_t)(d0 + i) * vdim] = st[i];
}

// The last rows' projections into their slots.
__global__ void __launch_bounds__(64)
delta_keep_kernel(const float *__restrict__ proj, int ld, int rows, int start, int taps, int channels,
                  float *__restrict__ ring) {
  const int c = blockIdx.x * 64 + threadIdx.x;
  if (c >= channels)
    return;
  for (int b = 1; b < taps && b <= rows; ++b)
    ring[(int64_t)((start + rows - b) % taps) * channels + c] = proj[(int64_t)(rows - b) * ld + c];
}

int keep_rows(const DeltaRows &a, hipStream_t stream) {
  const DeltaShape &s = a.s;
  if (s.taps > 1)
    hipLaunchKernelGGL(delta_keep_kernel, dim3((unsigned)ceil_div(s.channels, 64)), dim3(64), 0, stream,
                       a.proj, a.ld, a.rows, a.start, s.taps, s.channels, a.ring);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

bool delta_ok(const DeltaRows &a) {
  const DeltaShape &s = a.s;
  return a.proj && a.ring && a.state && a.rows > 0 && (!a.pos || a.rows == 1) && s.heads > 0 &&
         s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.vdim > 0 && s.taps > 0 &&
         s.decay_rank > 0 && s.gate_rank > 0 && s.channels > 0 && s.conv_w && s.decay_w && s.gate_w &&
         s.decay_bias && s.decay_speed && s.norm_w;
}


// ---- chunks ------------------------------------------------------------------------

constexpr int kC = kDeltaChunk, kBlock = 16, kBlocks = kC / kBlock;
constexpr int kChunkThreads = 512;
constexpr float kLog2e = 1.44269504088896341f;
constexpr float kLeast = -200.f; // of a decay's log2: 2^-200 is no f32 number, the same as none left
__device__ __forceinline__ float exp2_f(float x) { return __builtin_amdgcn_exp2f(x); }

// Where the parts of a chunk and head lie in the workspace, in floats.
struct ChunkParts {
  int dp, v16;                     // dim32, vdim16
  int w, q, kt, b, ut, last, size; // W, G q: [64][dim32]; (G_last / G k)^T: [dim32][64]; b: [64][64];
                                   // U^T, later u^T: [vdim16][64]; G_last: [dim32]
};
ChunkParts chunk_parts(const DeltaShape &s) {
  const int d = kC * s.dim32();
  ChunkParts p;
  p.dp = s.dim32();
  p.v16 = s.vdim16();
  p.w = 0;
  p.q = d;
  p.kt = 2 * d;
  p.b = 3 * d;
  p.ut = p.b + kC * kC;
  p.last = p.ut + kC * s.vdim16();
  p.size = p.last + s.dim32();
  return p;
}

struct DeltaPrepArgs {
  DeltaShape s;
  const float *proj, *ring;
  int ld, rows, start;
  float *conv; // [rows][channels]
  float *dots; // [rows][kv_heads]: q . k
};

constexpr int kPrepRows = 8;

// A column of kPrepRows rows through a convolution of TAPS taps: all inputs are asked
// for at once, and each is loaded once.
template <int TAPS>
__device__ __forceinline__ void conv_rows(const DeltaPrepArgs &a, int r0, int c, float (&out)[kPrepRows]) {
  const DeltaShape &s = a.s;
  float x[kPrepRows + TAPS - 1], w[TAPS];
#pragma unroll
  for (int i = 0; i < kPrepRows + TAPS - 1; ++i)
    x[i] = a.proj[(int64_t)min(r0 + i - (TAPS - 1), a.rows - 1) * a.ld + c];
#pragma unroll
  for (int t = 0; t < TAPS; ++t)
    w[t] = s.conv_w[(int64_t)t * s.channels + c];
#pragma unroll
  for (int r = 0; r < kPrepRows; ++r) {
    float v = 0.f;
#pragma unroll
    for (int t = 0; t < TAPS; ++t)
      v = fmaf(w[t], x[r + t], v);
    out[r] = silu_f(v);
  }
}

// A wavefront per kPrepRows rows and head (not the first rows, whose convolution reaches
// into the ring), like delta_prep_kernel; heads of at most 128 values.
template <int TAPS> __global__ void __launch_bounds__(256) delta_prep_rows_kernel(DeltaPrepArgs a) {
  const DeltaShape &s = a.s;
  const int lane = threadIdx.x & 63;
  const int u = blockIdx.y * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int r0 = (blockIdx.x + 1) * kPrepRows;
  if (u >= s.kv_heads + s.heads)
    return;
  float *out = a.conv + (int64_t)r0 * s.channels;
  const int rows = min(kPrepRows, a.rows - r0);
  if (u >= s.kv_heads) {
    const int at = s.v_at + (u - s.kv_heads) * s.vdim;
    for (int i = lane; i < s.vdim; i += 64) {
      float v[kPrepRows];
      conv_rows<TAPS>(a, r0, at + i, v);
#pragma unroll
      for (int r = 0; r < kPrepRows; ++r)
        if (r < rows)
          out[(int64_t)r * s.channels + at + i] = v[r];
    }
    return;
  }
  const int qa = s.q_at + u * s.dim, ka = s.k_at + u * s.dim;
  float q[2][kPrepRows], k[2][kPrepRows];
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int i = lane + j * 64;
    if (i < s.dim) {
      conv_rows<TAPS>(a, r0, qa + i, q[j]);
      conv_rows<TAPS>(a, r0, ka + i, k[j]);
    } else {
#pragma unroll
      for (int r = 0; r < kPrepRows; ++r)
        q[j][r] = k[j][r] = 0.f;
    }
  }
  const float root = sqrtf((float)s.dim);
#pragma unroll
  for (int r = 0; r < kPrepRows; ++r) {
    const float qq = wave_sum(fmaf(q[0][r], q[0][r], q[1][r] * q[1][r]));
    const float kk = wave_sum(fmaf(k[0][r], k[0][r], k[1][r] * k[1][r]));
    const float qk = wave_sum(fmaf(q[0][r], k[0][r], q[1][r] * k[1][r]));
    const float rq = 1.0f / sqrtf(qq + kUnitEps) / root, rk = 1.0f / sqrtf(kk + kUnitEps);
    if (r >= rows)
      continue;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int i = lane + j * 64;
      if (i < s.dim) {
        out[(int64_t)r * s.channels + qa + i] = q[j][r] * rq;
        out[(int64_t)r * s.channels + ka + i] = k[j][r] * rk;
      }
    }
    if (lane == 0)
      a.dots[(int64_t)(r0 + r) * s.kv_heads + u] = qk * rq * rk;
  }
}

// A wavefront per row and head: convolution and silu of a query and key head, made unit
// vectors, or of a value head.
__global__ void __launch_bounds__(256) delta_prep_kernel(DeltaPrepArgs a, int rows) {
  const DeltaShape &s = a.s;
  const int lane = threadIdx.x & 63;
  const int64_t id = (int64_t)blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int units = s.kv_heads + s.heads;
  if (id >= (int64_t)rows * units)
    return;
  const int r = (int)(id / units), u = (int)(id - (int64_t)r * units), p = a.start + r;
  const float *row = a.proj + (int64_t)r * a.ld;
  float *out = a.conv + (int64_t)r * s.channels;
  if (u >= s.kv_heads) {
    const int at = s.v_at + (u - s.kv_heads) * s.vdim;
    for (int i = lane; i < s.vdim; i += 64)
      out[at + i] = short_conv(s, row, a.ld, r, a.ring, p, at + i);
    return;
  }
  const int qa = s.q_at + u * s.dim, ka = s.k_at + u * s.dim;
  float qq = 0.f, kk = 0.f, qk = 0.f;
  constexpr int kKeep = 4; // values a lane keeps in registers
  float qv[kKeep], kv[kKeep];
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = lane + j * 64;
    qv[j] = kv[j] = 0.f;
    if (i < s.dim) {
      qv[j] = short_conv(s, row, a.ld, r, a.ring, p, qa + i);
      kv[j] = short_conv(s, row, a.ld, r, a.ring, p, ka + i);
    }
    qq = fmaf(qv[j], qv[j], qq);
    kk = fmaf(kv[j], kv[j], kk);
    qk = fmaf(qv[j], kv[j], qk);
  }
  const float rq = 1.0f / sqrtf(wave_sum(qq) + kUnitEps) / sqrtf((float)s.dim);
  const float rk = 1.0f / sqrtf(wave_sum(kk) + kUnitEps);
  qk = wave_sum(qk);
#pragma unroll
  for (int j = 0; j < kKeep; ++j) {
    const int i = lane + j * 64;
    if (i < s.dim) {
      out[qa + i] = qv[j] * rq;
      out[ka + i] = kv[j] * rk;
    }
  }
  if (lane == 0)
    a.dots[(int64_t)r * s.kv_heads + u] = qk * rq * rk;
}

struct DeltaChunkArgs {
  DeltaShape s;
  const float *conv, *dots, *decay; // decay: [rows][ld_decay], before bias and softplus
  const float *proj;
  int ld, ld_decay, rows;
  bool quads; // rows can be read four floats at a time
  float *parts;
  ChunkParts at;
};

// Grid (chunks, heads): everything about a chunk that does not need the state.
__global__ void __launch_bounds__(kChunkThreads) delta_chunk_kernel(DeltaChunkArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const DeltaShape &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int c = blockIdx.x, h = blockIdx.y, g = h / (s.heads / s.kv_heads);
  const int dim = s.dim, dp = a.at.dp, row_at = dp + 4;
  constexpr int kARow = kC + 4, kIRow = kBlock + 4;
  float *ks = lds;                  // [64][row_at]
  float *qs = ks + kC * row_at;     // [64][row_at]
  float *gs = qs + kC * row_at;     // [64][row_at]: log2 decay, summed from the block's first token
  float *as = gs + kC * row_at;     // [64][kARow]: beta_t a_ts
  float *tot = as + kC * kARow;     // [kBlocks][dp]: a block's sum
  float *beta = tot + kBlocks * dp; // [64]
  float *inv = beta + kC;           // [64][kIRow]: inverses of the blocks' own triangles
  const int r0 = c * kC, rows = min(kC, a.rows - r0);
  float *out = a.parts + ((int64_t)c * s.heads + h) * a.at.size;
  {
    const float speed = s.decay_speed[h] * kLog2e;
    const float *conv = a.conv + (int64_t)r0 * s.channels;
    const float *bias = s.decay_bias + h * dim, *raw = a.decay + (int64_t)r0 * a.ld_decay + h * dim;
    if (a.quads) { // four channels a time, several rows in flight
      const int cols = dp / 4, per = kChunkThreads / cols, d = tid % cols * 4;
      const int dl = d < dim ? d : 0;
      const f32x4 bb = *reinterpret_cast<const f32x4 *>(bias + dl);
      constexpr int kFlight = 4;
      for (int t0 = tid / cols; t0 < kC && tid < per * cols; t0 += per * kFlight) {
        f32x4 k[kFlight], q[kFlight], z[kFlight];
#pragma unroll
        for (int i = 0; i < kFlight; ++i) {
          const int64_t r = min(t0 + i * per, rows - 1);
          k[i] = *reinterpret_cast<const f32x4 *>(conv + r * s.channels + s.k_at + g * dim + dl);
          q[i] = *reinterpret_cast<const f32x4 *>(conv + r * s.channels + s.q_at + g * dim + dl);
          z[i] = *reinterpret_cast<const f32x4 *>(raw + r * a.ld_decay + dl);
        }
#pragma unroll
        for (int i = 0; i < kFlight; ++i) {
          const int t = t0 + i * per;
          if (t >= kC)
            continue;
          const bool some = t < rows && d < dim; // a row past the last: no write, no decay
          f32x4 l;
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            l[j] = some ? fmaxf(speed * softplus_f(z[i][j] + bb[j]), kLeast) : 0.f;
            k[i][j] = some ? k[i][j] : 0.f;
            q[i][j] = some ? q[i][j] : 0.f;
          }
          *reinterpret_cast<f32x4 *>(ks + t * row_at + d) = k[i];
          *reinterpret_cast<f32x4 *>(qs + t * row_at + d) = q[i];
          *reinterpret_cast<f32x4 *>(gs + t * row_at + d) = l;
        }
      }
    }
    for (int i = tid; !a.quads && i < kC * dp; i += kChunkThreads) {
      const int r = i / dp, d = i - r * dp;
      float k = 0.f, q = 0.f, l = 0.f; // a row past the last: no write, no decay
      if (r < rows && d < dim) {
        k = conv[(int64_t)r * s.channels + s.k_at + g * dim + d];
        q = conv[(int64_t)r * s.channels + s.q_at + g * dim + d];
        l = fmaxf(speed * softplus_f(raw[(int64_t)r * a.ld_decay + d] + bias[d]), kLeast);
      }
      ks[r * row_at + d] = k;
      qs[r * row_at + d] = q;
      gs[r * row_at + d] = l;
    }
    if (tid < kC)
      beta[tid] = tid < rows ? sigmoid_f(a.proj[(int64_t)(r0 + tid) * a.ld + s.beta_at + h]) : 0.f;
  }
  for (int i = tid; i < kC * kARow; i += kChunkThreads)
    as[i] = 0.f;
  __syncthreads();
  for (int i = tid; i < kBlocks * dp; i += kChunkThreads) {
    const int b = i / dp, d = i - b * dp;
    float *p = gs + b * kBlock * row_at + d, v[kBlock];
#pragma unroll
    for (int t = 0; t < kBlock; ++t)
      v[t] = p[t * row_at];
#pragma unroll
    for (int t = 1; t < kBlock; ++t)
      v[t] += v[t - 1];
#pragma unroll
    for (int t = 0; t < kBlock; ++t)
      p[t * row_at] = v[t];
    tot[i] = v[kBlock - 1];
  }
  __syncthreads();
  // pairs of different blocks: a product of 16 x 16 over the key channels each
  if (wave < 6) {
    const int bi = wave < 1 ? 1 : wave < 3 ? 2 : 3, bj = wave < 1 ? 0 : wave < 3 ? wave - 1 : wave - 3;
    const float *kt = ks + (bi * kBlock + col) * row_at, *qt = qs + (bi * kBlock + col) * row_at;
    const float *gt = gs + (bi * kBlock + col) * row_at;
    const float *kr = ks + (bj * kBlock + col) * row_at, *gr = gs + (bj * kBlock + col) * row_at;
    f32x4 sa{0.f, 0.f, 0.f, 0.f}, sb = sa;
    for (int d0 = quad * 8; d0 < dp; d0 += 32)
#pragma unroll
      for (int j0 = 0; j0 < 8; j0 += 4) {
        const int d = d0 + j0;
        f32x4 left = *reinterpret_cast<const f32x4 *>(gt + d);
        f32x4 right = *reinterpret_cast<const f32x4 *>(tot + bj * dp + d) - *reinterpret_cast<const f32x4 *>(gr + d);
        for (int b = bj + 1; b < bi; ++b)
          right += *reinterpret_cast<const f32x4 *>(tot + b * dp + d);
        const f32x4 k = *reinterpret_cast<const f32x4 *>(kt + d), q = *reinterpret_cast<const f32x4 *>(qt + d);
        const f32x4 w = *reinterpret_cast<const f32x4 *>(kr + d);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float l = exp2_f(left[j]), x = w[j] * exp2_f(right[j]);
          sa = mfma_f32(k[j] * l, x, sa);
          sb = mfma_f32(q[j] * l, x, sb);
        }
      }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = bi * kBlock + quad * 4 + r, x = bj * kBlock + col;
      as[t * kARow + x] = sa[r] * beta[t];
      out[a.at.b + t * kC + x] = sb[r];
      out[a.at.b + x * kC + t] = 0.f;
    }
  }
  // pairs within a block: a lane each, 120 of them on two wavefronts
  {
    const int b = wave >> 1, id = (wave & 1) * 60 + lane;
    if (lane < 60) {
      int t = (int)((1.0f + sqrtf((float)(8 * id + 1))) * 0.5f);
      t -= t * (t - 1) / 2 > id;
      t += (t + 1) * t / 2 <= id;
      const int x = id - t * (t - 1) / 2; // x < t
      const int tr = (b * kBlock + t) * row_at, xr = (b * kBlock + x) * row_at;
      float sa = 0.f, sb = 0.f;
      for (int d = 0; d < dp; d += 4) {
        const f32x4 gap = *reinterpret_cast<const f32x4 *>(gs + tr + d) - *reinterpret_cast<const f32x4 *>(gs + xr + d);
        const f32x4 k = *reinterpret_cast<const f32x4 *>(ks + tr + d), q = *reinterpret_cast<const f32x4 *>(qs + tr + d);
        const f32x4 w = *reinterpret_cast<const f32x4 *>(ks + xr + d);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float e = w[j] * exp2_f(gap[j]);
          sa = fmaf(k[j], e, sa);
          sb = fmaf(q[j], e, sb);
        }
      }
      const int ta = b * kBlock + t, xa = b * kBlock + x;
      as[ta * kARow + xa] = sa * beta[ta];
      out[a.at.b + ta * kC + xa] = sb;
      out[a.at.b + xa * kC + ta] = 0.f;
    } else {
      // the block's own tokens, four per wavefront at a time
      for (int t = (wave & 1) * 8 + lane - 60; t < (wave & 1) * 8 + 8; t += 4) {
        const int r = b * kBlock + t;
        out[a.at.b + r * kC + r] = r < rows ? a.dots[(int64_t)(r0 + r) * s.kv_heads + g] : 0.f;
      }
    }
  }
  __syncthreads();
  // the inverse of a block's own triangle, a lane per column, on one wavefront; the
  // others write what the carry takes as it is
  if (wave == 0) {
    const int b = lane >> 4;
    const float *m = as + b * kBlock * (kARow + 1); // the block's triangle
    float x[kBlock];
#pragma unroll
    for (int t = 0; t < kBlock; ++t) {
      float sum[4] = {t == col ? 1.f : 0.f, 0.f, 0.f, 0.f}; // none waits for the one before
#pragma unroll
      for (int y = 0; y < t; y += 4) {
        const f32x4 v = *reinterpret_cast<const f32x4 *>(m + t * kARow + y);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (y + j < t)
            sum[j] = fmaf(-v[j], x[y + j], sum[j]);
      }
      x[t] = (sum[0] + sum[1]) + (sum[2] + sum[3]);
      inv[(b * kBlock + t) * kIRow + col] = x[t];
    }
  } else {
    const int id = tid - 64, n = kChunkThreads - 64, cols = dp / 4;
    for (int i = id; i < kC * cols; i += n) {
      const int t = i / cols, d = (i - t * cols) * 4;
      f32x4 l = *reinterpret_cast<const f32x4 *>(gs + t * row_at + d);
      for (int b = 0; b < t / kBlock; ++b)
        l += *reinterpret_cast<const f32x4 *>(tot + b * dp + d);
      f32x4 q = *reinterpret_cast<const f32x4 *>(qs + t * row_at + d);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        q[j] *= exp2_f(l[j]);
      *reinterpret_cast<f32x4 *>(out + a.at.q + t * dp + d) = q;
    }
    for (int i = id; i < kC * cols; i += n) {
      const int t = i % kC, d = i / kC * 4, b = t / kBlock;
      f32x4 l = *reinterpret_cast<const f32x4 *>(tot + b * dp + d) - *reinterpret_cast<const f32x4 *>(gs + t * row_at + d);
      for (int j = b + 1; j < kBlocks; ++j)
        l += *reinterpret_cast<const f32x4 *>(tot + j * dp + d);
      const f32x4 k = *reinterpret_cast<const f32x4 *>(ks + t * row_at + d);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        out[a.at.kt + (d + j) * kC + t] = k[j] * exp2_f(l[j]);
    }
    for (int d = id; d < dp; d += n)
      out[a.at.last + d] = exp2_f((tot[d] + tot[dp + d]) + (tot[2 * dp + d] + tot[3 * dp + d]));
  }
  __syncthreads();
  // The triangular system, 16 right-hand sides at a time: block by block, what earlier
  // blocks wrote is taken off and the block's inverse applied.  A lane's four rows of a
  // result are its share of the next product's operand as they lie.
  for (int ct = wave; ct < (dp + a.at.v16) / 16; ct += kChunkThreads / 64) {
    f32x4 x[kBlocks];
    const int i = ct * 16 + col, v = i - dp;
    if (i < dp) {
      float ahead = 0.f;
#pragma unroll
      for (int b = 0; b < kBlocks; ++b) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = b * kBlock + quad * 4 + r;
          x[b][r] = beta[t] * ks[t * row_at + i] * exp2_f(ahead + gs[t * row_at + i]);
        }
        ahead += tot[b * dp + i];
      }
    } else {
      const float *src = a.conv + (int64_t)r0 * s.channels + s.v_at + h * s.vdim + min(v, s.vdim - 1);
#pragma unroll
      for (int b = 0; b < kBlocks; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          x[b][r] = src[(int64_t)min(b * kBlock + quad * 4 + r, rows - 1) * s.channels];
#pragma unroll
      for (int b = 0; b < kBlocks; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          x[b][r] = v < s.vdim ? x[b][r] * beta[b * kBlock + quad * 4 + r] : 0.f;
    }
#pragma unroll
    for (int b = 0; b < kBlocks; ++b) {
      f32x4 rhs = x[b];
#pragma unroll
      for (int e = 0; e < b; ++e) {
        const f32x4 m = *reinterpret_cast<const f32x4 *>(as + (b * kBlock + col) * kARow + e * kBlock + quad * 4);
#pragma unroll
        for (int j = 0; j < 4; ++j)
          rhs = mfma_f32(-m[j], x[e][j], rhs);
      }
      const f32x4 m = *reinterpret_cast<const f32x4 *>(inv + (b * kBlock + col) * kIRow + quad * 4);
      f32x4 y{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j)
        y = mfma_f32(m[j], rhs[j], y);
      x[b] = y;
    }
#pragma unroll
    for (int b = 0; b < kBlocks; ++b) {
      const int t = b * kBlock + quad * 4;
      if (i < dp) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          out[a.at.w + (t + r) * dp + i] = x[b][r];
      } else {
        *reinterpret_cast<f32x4 *>(out + a.at.ut + v * kC + t) = x[b];
      }
    }
  }
}

struct DeltaCarryArgs {
  int heads, dim, vdim, rows, chunks;
  const float *parts;
  ChunkParts at;
  float *state, *out; // out: [rows][heads * vdim]
};

// Grid (heads, value slices of 16): the state from chunk to chunk, and the outputs.  A
// wavefront takes 16 tokens of a chunk (products with the state) and every fourth tile
// of 16 key channels (the state itself, in registers).  ND: 32-channel steps, at most.
// What the chunk after this one needs is on its way meanwhile.
template <int ND>
__global__ void __launch_bounds__(256, 1) delta_carry_kernel(DeltaCarryArgs a) {
  constexpr int dp_max = ND * 32, kTiles = (2 * ND + 3) / 4; // state tiles per wavefront
  constexpr int kSRow = dp_max + 4, kURow = kC + 4;
  __shared__ __attribute__((aligned(16))) float st[16 * kSRow], ut[16 * kURow];
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, v0 = blockIdx.y * 16, v = v0 + col;
  const int dp = (a.dim + 31) & ~31, nd = dp / 32;
  float *S = a.state + (int64_t)h * a.dim * a.vdim;
  f32x4 own[kTiles];
#pragma unroll
  for (int i = 0; i < kTiles; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (wave + i * 4) * 16 + quad * 4 + r;
      own[i][r] = d < a.dim && v < a.vdim ? S[(int64_t)d * a.vdim + v] : 0.f;
    }
  struct Chunk {
    Frag<float> w[ND], q[ND], b[2], k[kTiles][2];
    f32x4 u, last[kTiles];
  };
  auto fetch = [&](int c, Chunk &x) {
    const float *p = a.parts + ((int64_t)min(c, a.chunks - 1) * a.heads + h) * a.at.size;
    const float *row = p + (int64_t)(wave * 16 + col) * dp + quad * 8;
#pragma unroll
    for (int t = 0; t < ND; ++t) {
      const int d = min(t, nd - 1) * 32;
      x.w[t].load(row + a.at.w + d);
      x.q[t].load(row + a.at.q + d);
    }
    x.u = *reinterpret_cast<const f32x4 *>(p + a.at.ut + (int64_t)(v0 + col) * kC + wave * 16 + quad * 4);
#pragma unroll
    for (int t = 0; t < 2; ++t)
      x.b[t].load(p + a.at.b + (wave * 16 + col) * kC + t * 32 + quad * 8);
#pragma unroll
    for (int i = 0; i < kTiles; ++i) {
      const int d0 = min((wave + i * 4) * 16, dp - 16);
#pragma unroll
      for (int t = 0; t < 2; ++t)
        x.k[i][t].load(p + a.at.kt + (int64_t)(d0 + col) * kC + t * 32 + quad * 8);
      x.last[i] = *reinterpret_cast<const f32x4 *>(p + a.at.last + d0 + quad * 4);
    }
  };
  Chunk cur;
  fetch(0, cur);
  for (int c = 0; c < a.chunks; ++c) {
    Chunk next;
    fetch(c + 1, next);
#pragma unroll
    for (int i = 0; i < kTiles; ++i)
      if ((wave + i * 4) * 16 < dp)
        *reinterpret_cast<f32x4 *>(st + col * kSRow + (wave + i * 4) * 16 + quad * 4) = own[i];
    __syncthreads();
    f32x4 ws{0.f, 0.f, 0.f, 0.f}, o = ws;
#pragma unroll
    for (int t = 0; t < ND; ++t)
      if (t < nd) {
        Frag<float> sf;
        sf.load(st + col * kSRow + t * 32 + quad * 8);
        ws = mfma32(cur.w[t], sf, ws);
        o = mfma32(cur.q[t], sf, o);
      }
    const f32x4 u = cur.u - ws;
    *reinterpret_cast<f32x4 *>(ut + col * kURow + wave * 16 + quad * 4) = u;
    __syncthreads();
    Frag<float> uf[2];
#pragma unroll
    for (int t = 0; t < 2; ++t)
      uf[t].load(ut + col * kURow + t * 32 + quad * 8);
#pragma unroll
    for (int i = 0; i < kTiles; ++i) {
      f32x4 n = own[i] * cur.last[i];
#pragma unroll
      for (int t = 0; t < 2; ++t)
        n = mfma32(cur.k[i][t], uf[t], n);
      own[i] = n;
    }
#pragma unroll
    for (int t = 0; t < 2; ++t)
      if (t * 32 <= wave * 16 + 15)
        o = mfma32(cur.b[t], uf[t], o);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = c * kC + wave * 16 + quad * 4 + r;
      if (row < a.rows && v < a.vdim)
        a.out[((int64_t)row * a.heads + h) * a.vdim + v] = o[r];
    }
    cur = next;
  }
#pragma unroll
  for (int i = 0; i < kTiles; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = (wave + i * 4) * 16 + quad * 4 + r;
      if (d < a.dim && v < a.vdim)
        S[(int64_t)d * a.vdim + v] = own[i][r];
    }
}

struct DeltaGateArgs {
  int heads, vdim, rows, ld_gate, out_ld;
  float eps;
};

// A wavefront per row and head: the output's norm and gate.
template <typename T>
__global__ void __launch_bounds__(256)
delta_gate_kernel(const float *__restrict__ o, const float *__restrict__ gate, const float *__restrict__ norm_w,
                  T *__restrict__ out, DeltaGateArgs a) {
  const int lane = threadIdx.x & 63;
  const int64_t id = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (id >= (int64_t)a.rows * a.heads)
    return;
  const int64_t row = id / a.heads;
  const int at = (int)(id - row * a.heads) * a.vdim;
  const float *x = o + id * a.vdim;
  float ss = 0.f;
  for (int i = lane; i < a.vdim; i += 64)
    ss = fmaf(x[i], x[i], ss);
  const float f = 1.0f / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
  for (int i = lane; i < a.vdim; i += 64)
    store_act<T>(out + row * a.out_ld + at + i,
                 x[i] * f * norm_w[i] * sigmoid_f(gate[row * a.ld_gate + at + i]));
}

constexpr size_t kChunkLdsLimit = 156 * 1024;
size_t chunk_lds(const DeltaShape &s) {
  return sizeof(float) * ((size_t)3 * kC * (s.dim32() + 4) + (size_t)kC * (kC + 4) + kBlocks * s.dim32() + kC + kC * (kBlock + 4));
}
struct Workspace {
  size_t conv, dots, decay, gate, out, parts, size; // offsets in floats
};
Workspace workspace(const DeltaShape &s, int rows) {
  Workspace w;
  size_t at = 0;
  auto take = [&](size_t n) {
    const size_t here = at;
    at += (size_t)round_up((int64_t)n, 64);
    return here;
  };
  const size_t n = (size_t)rows;
  w.conv = take(n * s.channels);
  w.dots = take(n * s.kv_heads);
  w.decay = take(n * s.decay.N);
  w.gate = take(n * s.gate.N);
  w.out = take(n * s.heads * s.vdim);
  w.parts = take((size_t)ceil_div(rows, kC) * s.heads * chunk_parts(s).size);
  w.size = at;
  return w;
}

} // namespace

int launch_delta_scan(const DeltaRows &a, hipStream_t stream) {
  const DeltaShape &s = a.s;
  BH_REQUIRE(delta_ok(a) && a.o && a.gate, "delta_scan: bad argument");
  const int per = (int)ceil_div(s.dim, kScanSlices);
  const size_t lds = sizeof(float) * (size_t)(round_up(s.decay_rank, 4) + round_up(s.gate_rank, 4));
  BH_REQUIRE(per <= 64 && lds <= 40 * 1024, "delta_scan: key heads of %d, ranks of %d and %d", s.dim, s.decay_rank,
             s.gate_rank);
  const dim3 grid((unsigned)s.heads, (unsigned)ceil_div(s.vdim, kScanCols));
#define BH_SCAN(N) hipLaunchKernelGGL(delta_scan_kernel<N>, grid, dim3(kScanThreads), lds, stream, a)
  if (per <= 4)
    BH_SCAN(4);
  else if (per <= 8)
    BH_SCAN(8);
  else if (per <= 16)
    BH_SCAN(16);
  else if (per <= 32)
    BH_SCAN(32);
  else
    BH_SCAN(64);
#undef BH_SCAN
  BH_CHECK_HIP(hipGetLastError());
  return a.rows > 1 ? keep_rows(a, stream) : BUDDY_HIP_OK;
}

int launch_delta_gate(const DeltaShape &s, const float *o, const float *gate, int ld_gate, int rows, void *out,
                      int out_ld, bool act_f32, hipStream_t stream) {
  BH_REQUIRE(o && gate && out && rows > 0 && s.heads > 0 && s.vdim > 0 && s.norm_w, "delta_gate: bad argument");
  DeltaGateArgs e{s.heads, s.vdim, rows, ld_gate, out_ld, s.eps};
  const dim3 grid((unsigned)ceil_div((int64_t)rows * s.heads, 4));
  if (act_f32)
    hipLaunchKernelGGL(delta_gate_kernel<float>, grid, dim3(256), 0, stream, o, gate, s.norm_w,
                       static_cast<float *>(out), e);
  else
    hipLaunchKernelGGL(delta_gate_kernel<bf16_bits>, grid, dim3(256), 0, stream, o, gate, s.norm_w,
                       static_cast<bf16_bits *>(out), e);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

size_t delta_workspace(const DeltaShape &s, int rows) {
  if (s.dim > 256 || chunk_lds(s) > kChunkLdsLimit)
    return 0;
  return workspace(s, rows).size;
}

int launch_delta_chunks(const DeltaRows &a, float *ws, hipStream_t stream) {
  const DeltaShape &s = a.s;
  BH_REQUIRE(delta_ok(a) && a.out && !a.pos && ws && ((uintptr_t)ws & 15) == 0 && delta_workspace(s, a.rows) > 0 &&
                 s.decay.tiles && s.gate.tiles && s.decay.K == s.decay_rank && s.gate.K == s.gate_rank &&
                 s.decay.N >= s.heads * s.dim && s.gate.N >= s.heads * s.vdim,
             "delta_chunks: bad argument");
  const Workspace w = workspace(s, a.rows);
  int rc;
  // the outer halves of the low-rank projections, on f32 activations
  for (const bool gate : {false, true}) {
    RowsGemm g;
    g.W = gate ? s.gate : s.decay;
    g.A = a.proj + (gate ? s.gate_at : s.decay_at);
    g.lda = a.ld;
    g.f32 = true;
    g.rows = a.rows;
    g.C = ws + (gate ? w.gate : w.decay);
    g.ldc = g.W.N;
    if ((rc = launch_rows_gemm(g, stream)))
      return rc;
  }
  DeltaPrepArgs p{s, a.proj, a.ring, a.ld, a.rows, a.start, ws + w.conv, ws + w.dots};
  const int units = s.kv_heads + s.heads;
  const bool blocks = s.dim <= 128 && s.taps >= 2 && s.taps <= 4 && a.rows > kPrepRows;
  const int singly = blocks ? kPrepRows : a.rows; // the first rows, or all of them
  hipLaunchKernelGGL(delta_prep_kernel, dim3((unsigned)ceil_div((int64_t)singly * units, 4)), dim3(256), 0, stream, p,
                     singly);
  if (blocks) {
    const dim3 grid((unsigned)ceil_div(a.rows - kPrepRows, kPrepRows), (unsigned)ceil_div(units, 4));
    if (s.taps == 2)
      hipLaunchKernelGGL(delta_prep_rows_kernel<2>, grid, dim3(256), 0, stream, p);
    else if (s.taps == 3)
      hipLaunchKernelGGL(delta_prep_rows_kernel<3>, grid, dim3(256), 0, stream, p);
    else
      hipLaunchKernelGGL(delta_prep_rows_kernel<4>, grid, dim3(256), 0, stream, p);
  }
  BH_CHECK_HIP(hipGetLastError());
  if ((rc = keep_rows(a, stream)))
    return rc;
  const int chunks = (int)ceil_div(a.rows, kC);
  DeltaChunkArgs c{s, ws + w.conv, ws + w.dots, ws + w.decay, a.proj, a.ld, s.decay.N, a.rows, false,
                   ws + w.parts, chunk_parts(s)};
  c.quads = s.dim % 4 == 0 && s.q_at % 4 == 0 && s.k_at % 4 == 0 && s.channels % 4 == 0 &&
            ((uintptr_t)s.decay_bias & 15) == 0;
  static DynLdsOnce once;
  BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)delta_chunk_kernel, (int)kChunkLdsLimit));
  hipLaunchKernelGGL(delta_chunk_kernel, dim3((unsigned)chunks, (unsigned)s.heads), dim3(kChunkThreads),
                     chunk_lds(s), stream, c);
  BH_CHECK_HIP(hipGetLastError());
  DeltaCarryArgs k{s.heads, s.dim, s.vdim, a.rows, chunks, ws + w.parts, chunk_parts(s), a.state, ws + w.out};
  const dim3 grid((unsigned)s.heads, (unsigned)(s.vdim16() / 16));
  const int nd = s.dim32() / 32;
  if (nd <= 1)
    hipLaunchKernelGGL(delta_carry_kernel<1>, grid, dim3(256), 0, stream, k);
  else if (nd <= 2)
    hipLaunchKernelGGL(delta_carry_kernel<2>, grid, dim3(256), 0, stream, k);
  else if (nd <= 4)
    hipLaunchKernelGGL(delta_carry_kernel<4>, grid, dim3(256), 0, stream, k);
  else
    hipLaunchKernelGGL(delta_carry_kernel<8>, grid, dim3(256), 0, stream, k);
  BH_CHECK_HIP(hipGetLastError());
  return launch_delta_gate(s, ws + w.out, ws + w.gate, s.gate.N, a.rows, a.out, a.out_ld, a.act_f32, stream);
}

} // namespace bh
