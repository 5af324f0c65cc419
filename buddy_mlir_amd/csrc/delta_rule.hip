// delta_rule.hip -- the gated delta rule, token by token.
#include "delta_rule.h"
#include "bf16_dev.h"

#include <algorithm>

namespace bh {
namespace {

constexpr int kScanThreads = 1024, kScanWaves = kScanThreads / 64;
constexpr float kUnitEps = 1e-6f; // of the unit vectors

__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// Row `w` of a bfloat16 matrix times x (LDS), by eight neighbouring lanes; all of them
// get the sum.
__device__ __forceinline__ float row_dot8(const uint16_t *__restrict__ w, const float *x, int n) {
  const int l = threadIdx.x & 7;
  float acc = 0.f;
  if (n % 8 == 0) {
    for (int i = l * 8; i < n; i += 64) {
      const uint4 v = *reinterpret_cast<const uint4 *>(w + i);
      acc = fmaf(bf_lo(v.x), x[i], acc);
      acc = fmaf(bf_hi(v.x), x[i + 1], acc);
      acc = fmaf(bf_lo(v.y), x[i + 2], acc);
      acc = fmaf(bf_hi(v.y), x[i + 3], acc);
      acc = fmaf(bf_lo(v.z), x[i + 4], acc);
      acc = fmaf(bf_hi(v.z), x[i + 5], acc);
      acc = fmaf(bf_lo(v.w), x[i + 6], acc);
      acc = fmaf(bf_hi(v.w), x[i + 7], acc);
    }
  } else {
    for (int i = l; i < n; i += 8)
      acc = fmaf(bf_f(w[i]), x[i], acc);
  }
  acc = quad_sum(acc);
  return acc + __shfl_xor(acc, 4, 64);
}

// The convolution of column c at position p; `row`: the projections of that position,
// `have`: how many rows ahead of it lie in the projections (earlier ones are in the ring).
__device__ __forceinline__ float short_conv(const DeltaShape &s, const float *row, int ld, int have,
                                            const float *__restrict__ ring, int p, int c) {
  float v = 0.f;
  for (int b = s.taps - 1; b >= 0; --b) {
    if (p - b < 0)
      continue;
    const float e = b <= have ? row[c - (int64_t)b * ld] : ring[(int64_t)((p - b) % s.taps) * s.channels + c];
    v = fmaf(s.conv_w[(int64_t)(s.taps - 1 - b) * s.channels + c], e, v);
  }
  return silu_f(v);
}

// A workgroup per head.  A thread owns one value channel of N consecutive rows of the
// state, in registers from the first token to the last.  Both products with the
// state are taken of the decayed one: S^T q = (g S)^T q + u (k . q).
template <typename T, int N>
__global__ void __launch_bounds__(kScanThreads)
delta_scan_kernel(DeltaRows a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float red[kScanWaves], dots[3];
  const DeltaShape &s = a.s;
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int h = blockIdx.x, group = s.heads / s.kv_heads, g = h / group;
  const int dim = s.dim, vdim = s.vdim;
  const int vcols = (vdim + 63) & ~63, slices = kScanThreads / vcols;
  const int padded = slices * N; // rows of the state with those past the last, which stay zero
  float *q = lds, *k = q + padded, *decay = k + padded, *v = decay + padded, *gate = v + vdim;
  float *inner_d = gate + vdim, *inner_g = inner_d + ((s.decay_rank + 3) & ~3);
  float *part = inner_g + ((s.gate_rank + 3) & ~3); // [2][slices][vcols]
  const int c = tid % vcols, slice = tid / vcols;
  const bool owner = slice < slices && c < vdim;
  float *S = a.state + (int64_t)h * dim * vdim + min(c, vdim - 1);
  const int d0 = min(slice, slices - 1) * N;
  float st[N];
#pragma unroll
  for (int i = 0; i < N; ++i)
    st[i] = owner && d0 + i < dim ? S[(int64_t)(d0 + i) * vdim] : 0.f;
  for (int i = dim + tid; i < padded; i += kScanThreads)
    q[i] = k[i] = decay[i] = 0.f;
  const int p0 = a.pos ? *a.pos : a.start;
  const float speed = s.decay_speed[h];
  for (int r = 0; r < a.rows; ++r) {
    const float *row = a.proj + (int64_t)r * a.ld;
    const int p = p0 + r;
    for (int i = tid; i < 2 * dim + vdim; i += kScanThreads) {
      const int col = i < dim ? s.q_at + g * dim + i
                      : i < 2 * dim ? s.k_at + g * dim + i - dim
                                    : s.v_at + h * vdim + i - 2 * dim;
      const float x = short_conv(s, row, a.ld, r, a.ring, p, col);
      (i < dim ? q[i] : i < 2 * dim ? k[i - dim] : v[i - 2 * dim]) = x;
      // no workgroup reads this slot: it is the one of position p - taps
      if (a.rows == 1 && (i >= 2 * dim || h == g * group))
        a.ring[(int64_t)(p % s.taps) * s.channels + col] = row[col];
    }
    for (int i = tid; i < s.decay_rank; i += kScanThreads)
      inner_d[i] = row[s.decay_at + i];
    for (int i = tid; i < s.gate_rank; i += kScanThreads)
      inner_g[i] = row[s.gate_at + i];
    __syncthreads();
    for (int i = tid >> 3; i < dim + vdim; i += kScanThreads / 8) {
      if (i < dim) {
        const int64_t at = (int64_t)h * dim + i;
        const float z = row_dot8(s.decay_w + at * s.decay_rank, inner_d, s.decay_rank);
        if ((tid & 7) == 0)
          decay[i] = expf(speed * softplus_f(z + s.decay_bias[at]));
      } else {
        const float z = row_dot8(s.gate_w + ((int64_t)h * vdim + i - dim) * s.gate_rank, inner_g, s.gate_rank);
        if ((tid & 7) == 0)
          gate[i - dim] = sigmoid_f(z);
      }
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
    const float rq = 1.0f / sqrtf(dots[0] + kUnitEps) / sqrtf((float)dim), rk = 1.0f / sqrtf(dots[1] + kUnitEps);
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
    if (slice < slices) {
      part[slice * vcols + c] = sk;
      part[(slices + slice) * vcols + c] = sq;
    }
    __syncthreads();
    sk = sq = 0.f;
    for (int i = 0; i < slices; ++i) {
      sk += part[i * vcols + c];
      sq += part[(slices + i) * vcols + c];
    }
    const float beta = sigmoid_f(row[s.beta_at + h]);
    const float u = owner ? beta * (v[c] - sk * rk) : 0.f;
    const float ku = rk * u;
#pragma unroll
    for (int i = 0; i < N; i += 4) {
      const f32x4 kk = *reinterpret_cast<const f32x4 *>(k + d0 + i);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        st[i + j] = fmaf(kk[j], ku, st[i + j]);
    }
    const float o = rq * fmaf(ku, dots[2], sq);
    const float ss = wave_sum(slice == 0 && owner ? o * o : 0.f);
    if (lane == 0)
      red[wave] = ss;
    __syncthreads();
    if (slice == 0 && owner) {
      float t = 0.f;
      for (int w = 0; w < vcols / 64; ++w)
        t += red[w];
      const float f = 1.0f / sqrtf(t / (float)vdim + s.eps);
      store_act<T>(static_cast<T *>(a.out) + (int64_t)r * a.out_ld + (int64_t)h * vdim + c,
                   o * f * s.norm_w[c] * gate[c]);
    }
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

bool delta_ok(const DeltaRows &a) {
  const DeltaShape &s = a.s;
  return a.proj && a.ring && a.state && a.out && a.rows > 0 && (!a.pos || a.rows == 1) && s.heads > 0 &&
         s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.vdim > 0 && s.taps > 0 &&
         s.decay_rank > 0 && s.gate_rank > 0 && s.channels > 0 && s.conv_w && s.decay_w && s.gate_w &&
         s.decay_bias && s.decay_speed && s.norm_w;
}

} // namespace

int launch_delta_scan(const DeltaRows &a, hipStream_t stream) {
  const DeltaShape &s = a.s;
  BH_REQUIRE(delta_ok(a), "delta_scan: bad argument");
  const int vcols = (int)round_up(s.vdim, 64);
  BH_REQUIRE(vcols <= kScanThreads, "delta_scan: value heads of %d", s.vdim);
  const int slices = kScanThreads / vcols, per = (int)ceil_div(s.dim, slices);
  const int rows_per = per <= 8 ? 8 : per <= 16 ? 16 : per <= 32 ? 32 : 64;
  const size_t lds = sizeof(float) * (3 * (size_t)slices * rows_per + 2 * (size_t)s.vdim + round_up(s.decay_rank, 4) +
                                      round_up(s.gate_rank, 4) + 2 * (size_t)slices * vcols);
  constexpr size_t kLimit = 64 * 1024;
  BH_REQUIRE(per <= 64 && lds <= kLimit, "delta_scan: a state of %d x %d", s.dim, s.vdim);
#define BH_SCAN(T, N)                                                                              \
  hipLaunchKernelGGL((delta_scan_kernel<T, N>), dim3((unsigned)s.heads), dim3(kScanThreads), lds,  \
                     stream, a)
#define BH_SCANS(T)                                                                                \
  do {                                                                                             \
    if (rows_per == 8)                                                                             \
      BH_SCAN(T, 8);                                                                               \
    else if (rows_per == 16)                                                                       \
      BH_SCAN(T, 16);                                                                              \
    else if (rows_per == 32)                                                                       \
      BH_SCAN(T, 32);                                                                              \
    else                                                                                           \
      BH_SCAN(T, 64);                                                                              \
  } while (0)
  if (a.act_f32)
    BH_SCANS(float);
  else
    BH_SCANS(bf16_bits);
#undef BH_SCANS
#undef BH_SCAN
  BH_CHECK_HIP(hipGetLastError());
  if (a.rows > 1 && s.taps > 1)
    hipLaunchKernelGGL(delta_keep_kernel, dim3((unsigned)ceil_div(s.channels, 64)), dim3(64), 0, stream,
                       a.proj, a.ld, a.rows, a.start, s.taps, s.channels, a.ring);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

} // namespace bh
