// linear_attn.hip -- the decaying linear-attention recurrence: one token, and a
// prompt in chunks of 64 tokens: every chunk's own contribution to the state, a
// scan over the chunks, then every chunk's outputs from the state it starts with
// and its own tokens.  f32 matrix cores throughout.
#include "linear_attn.h"
#include "bf16_dev.h"

#include <algorithm>

namespace bh {
namespace {

// Grid (heads, ceil(vdim / 16)): 16 value channels x 16 slices of the key
// dimensions, which meet in LDS in slice order.
__global__ void __launch_bounds__(256)
linear_step_kernel(const float *__restrict__ q, const float *__restrict__ k,
                   const float *__restrict__ v, int dim, int vdim,
                   const float *__restrict__ powers, float *__restrict__ state,
                   float *__restrict__ out) {
  __shared__ float part[16][17];
  const int h = blockIdx.x, c = threadIdx.x & 15, slice = threadIdx.x >> 4;
  const int vi = blockIdx.y * 16 + c;
  const bool ok = vi < vdim;
  const int vc = min(vi, vdim - 1);
  const float decay = powers[h * (kLinearChunk + 1) + 1];
  const float vv = v[(int64_t)h * vdim + vc];
  float *S = state + (int64_t)h * dim * vdim + vc;
  float acc = 0.f;
  for (int d0 = slice; d0 < dim; d0 += 16 * 8) {
    float s[8], kk[8], qq[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int d = min(d0 + u * 16, dim - 1);
      s[u] = S[(int64_t)d * vdim];
      kk[u] = k[(int64_t)h * dim + d];
      qq[u] = q[(int64_t)h * dim + d];
    }
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (d0 + u * 16 < dim) {
        const float n = fmaf(decay, s[u], kk[u] * vv);
        acc = fmaf(n, qq[u], acc);
        if (ok)
          S[(int64_t)(d0 + u * 16) * vdim] = n;
      }
  }
  part[slice][c] = acc;
  __syncthreads();
  if (slice == 0 && ok) {
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i)
      t += part[i][c];
    out[(int64_t)h * vdim + vi] = t;
  }
}

struct LinearArgs {
  int heads, dim, vdim, ld, q_at, k_at, v_at, rows;
  int dp;     // LDS row of q / k: dim padded to 32, plus 4
  bool quads; // rows can be moved four floats at a time
  const float *powers;
};

// Rows 0..kLinearChunk - 1 of src into LDS as [.][stride]; rows past `rows` and columns
// past `width` (of `padded`, a multiple of 4) as zeros.  With `quads` (width, ld and
// the address are multiples of four floats) 16 bytes a load, eight in flight.
template <int THREADS>
__device__ __forceinline__ void stage_rows(float *dst, int stride, const float *src, int64_t ld,
                                           int rows, int total_rows, int width, int padded, bool quads) {
  const int cols = padded / 4, c = threadIdx.x % cols * 4, per = THREADS / cols;
  int r = threadIdx.x / cols;
  if (r >= per)
    return;
  if (quads) {
#pragma unroll 8
    for (; r < total_rows; r += per) {
      f32x4 v{0.f, 0.f, 0.f, 0.f};
      if (r < rows && c < width)
        v = *reinterpret_cast<const f32x4 *>(src + r * ld + c);
      *reinterpret_cast<f32x4 *>(dst + r * stride + c) = v;
    }
  } else {
    for (; r < total_rows; r += per) {
      f32x4 v;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        v[j] = r < rows && c + j < width ? src[r * ld + c + j] : 0.f;
      *reinterpret_cast<f32x4 *>(dst + r * stride + c) = v;
    }
  }
}

// Grid (chunks, heads, value slices of SV channels): sum over the chunk's tokens of
// decay^(last - i) k_i v_i^T.
template <int SV>
__global__ void __launch_bounds__(SV * 4)
linear_chunk_kernel(const float *__restrict__ proj, float *__restrict__ chunk_states, LinearArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float pw[kLinearChunk];
  constexpr int kThreads = SV * 4, kWaves = kThreads / 64;
  const int kw = (a.dim + 31) / 32 * 32, kKRow = kw + 8;
  constexpr int kVRow = SV + 8; // the four rows of an operand start 8 banks apart
  const int lane = threadIdx.x & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * SV;
  const int rows = min(kLinearChunk, a.rows - c * kLinearChunk);
  const int vw = min(SV, a.vdim - v0);
  float *k = lds, *v = lds + kLinearChunk * kKRow;
  const float *src = proj + (int64_t)c * kLinearChunk * a.ld;
  stage_rows<kThreads>(k, kKRow, src + a.k_at + h * a.dim, a.ld, rows, kLinearChunk, a.dim, kw, a.quads);
  stage_rows<kThreads>(v, kVRow, src + a.v_at + h * a.vdim + v0, a.ld, rows, kLinearChunk, vw, SV, a.quads);
  if (threadIdx.x < kLinearChunk) // of a token: what is left of it at the chunk's end
    pw[threadIdx.x] = threadIdx.x < rows ? a.powers[h * (kLinearChunk + 1) + rows - 1 - threadIdx.x] : 0.f;
  __syncthreads();
  float *dst = chunk_states + ((int64_t)c * a.heads + h) * a.dim * a.vdim;
  for (int dt = wave; dt * 16 < a.dim; dt += kWaves) {
    f32x4 acc[SV / 16];
#pragma unroll
    for (int t = 0; t < SV / 16; ++t)
      acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    // operands of the next two steps are read while these two are multiplied
    constexpr int kSteps = kLinearChunk / 4, kPair = 2;
    float ka[2][kPair], vb[2][kPair][SV / 16];
    auto read = [&](int s0, float (&ks)[kPair], float (&vs)[kPair][SV / 16]) {
#pragma unroll
      for (int j = 0; j < kPair; ++j) {
        const int r = (s0 + j) * 4 + quad;
        ks[j] = k[r * kKRow + dt * 16 + col] * pw[r];
#pragma unroll
        for (int t = 0; t < SV / 16; ++t)
          vs[j][t] = v[r * kVRow + t * 16 + col];
      }
    };
    read(0, ka[0], vb[0]);
#pragma unroll
    for (int s = 0; s < kSteps; s += kPair) {
      const int cur = (s / kPair) & 1;
      if (s + kPair < kSteps)
        read(s + kPair, ka[cur ^ 1], vb[cur ^ 1]);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int j = 0; j < kPair; ++j)
#pragma unroll
        for (int t = 0; t < SV / 16; ++t)
          acc[t] = mfma_f32(ka[cur][j], vb[cur][j][t], acc[t]);
      __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int t = 0; t < SV / 16; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = dt * 16 + quad * 4 + r, x = t * 16 + col;
        if (d < a.dim && x < vw)
          dst[(int64_t)d * a.vdim + v0 + x] = acc[t][r];
      }
  }
}

// One thread per state element: turns the chunks' contributions into the state each
// chunk starts with, and leaves the last one in the sequence's state.
__global__ void __launch_bounds__(256)
linear_scan_kernel(float *__restrict__ chunk_states, float *__restrict__ state, int per_head,
                   int64_t total, int rows, const float *__restrict__ powers) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total)
    return;
  const float *pw = powers + (i / per_head) * (kLinearChunk + 1);
  float s = state[i];
  const int chunks = (rows + kLinearChunk - 1) / kLinearChunk;
  for (int c0 = 0; c0 < chunks; c0 += 8) {
    float d[8];
#pragma unroll
    for (int u = 0; u < 8; ++u)
      d[u] = chunk_states[(int64_t)min(c0 + u, chunks - 1) * total + i];
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (c0 + u < chunks) {
        const int c = c0 + u, n = min(kLinearChunk, rows - c * kLinearChunk);
        chunk_states[(int64_t)c * total + i] = s;
        s = fmaf(s, pw[n], d[u]);
      }
  }
  state[i] = s;
}

// Grid (chunks, heads, value slices of SV channels): o_i = decay^(i+1) S^T q_i + sum
// over j <= i of decay^(i-j) (q_i . k_j) v_j.  A wavefront owns 16 queries, which it
// keeps in registers (NF steps of 32 key dimensions; 0: any number, loaded where they
// are used), and 64 value channels.  The state takes the place of the chunk's keys
// and values in LDS once those have been used; its loads are in flight meanwhile.
template <int SV, int NF>
__global__ void __launch_bounds__(SV * 4)
linear_out_kernel(const float *__restrict__ proj, const float *__restrict__ chunk_states,
                  float *__restrict__ out, LinearArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float pw[kLinearChunk + 1];
  constexpr int kThreads = SV * 4, NV = 4, kStateLoads = 8;
  constexpr int kVRow = SV + 4; // rows that are read four apart start 16 banks apart
  constexpr int kSRow = SV + 8; // rows that are read together start 8 banks apart
  const int tid = threadIdx.x, lane = tid & 63, col = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  // query tile (late ones have more keys: a SIMD gets one of either end), value channels
  const int qt = wave < 4 ? wave : 7 - wave, vt0 = wave >> 2 << 6;
  const int c = blockIdx.x, h = blockIdx.y, v0 = blockIdx.z * SV;
  const int rows = min(kLinearChunk, a.rows - c * kLinearChunk);
  const int vw = min(SV, a.vdim - v0);
  const int nf = (a.dp - 4) / 32;
  float *k = lds, *v = k + kLinearChunk * a.dp, *st = lds;
  const float *src = proj + (int64_t)c * kLinearChunk * a.ld;
  const float *S = chunk_states + ((int64_t)c * a.heads + h) * a.dim * a.vdim + v0;
  const int qi = qt * 16 + col; // this lane's query within the chunk
  const float *qrow = src + (int64_t)min(qi, rows - 1) * a.ld + a.q_at + h * a.dim;
  auto query = [&](int t) { // dimensions t * 32 + quad * 8 + 0..7
    Frag<float> f;
    const int d = t * 32 + quad * 8;
    if (a.quads) {
      const f32x4 z{0.f, 0.f, 0.f, 0.f};
      f.lo = d < a.dim ? *reinterpret_cast<const f32x4 *>(qrow + d) : z;
      f.hi = d + 4 < a.dim ? *reinterpret_cast<const f32x4 *>(qrow + d + 4) : z;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        f.lo[j] = d + j < a.dim ? qrow[d + j] : 0.f;
        f.hi[j] = d + 4 + j < a.dim ? qrow[d + 4 + j] : 0.f;
      }
    }
    return f;
  };
  Frag<float> qf[NF > 0 ? NF : 1];
  if constexpr (NF > 0) {
#pragma unroll
    for (int t = 0; t < NF; ++t)
      qf[t] = query(t); // zeros past the last dimension
  }
  stage_rows<kThreads>(k, a.dp, src + a.k_at + h * a.dim, a.ld, rows, kLinearChunk, a.dim, a.dp - 4, a.quads);
  stage_rows<kThreads>(v, kVRow, src + a.v_at + h * a.vdim + v0, a.ld, rows, kLinearChunk, vw, SV, a.quads);
  if (tid <= kLinearChunk)
    pw[tid] = a.powers[h * (kLinearChunk + 1) + tid];
  // the first rows of the state: SV / 4 threads a row, 16 rows a pass
  const int sc = tid % (SV / 4) * 4, sr = tid / (SV / 4);
  f32x4 ahead[kStateLoads];
  if (a.quads) {
#pragma unroll
    for (int i = 0; i < kStateLoads; ++i)
      ahead[i] = *reinterpret_cast<const f32x4 *>(S + (int64_t)min(sr + i * 16, a.dim - 1) * a.vdim +
                                                  (sc < vw ? sc : 0));
  }
  __syncthreads();
  f32x4 o[NV];
#pragma unroll
  for (int t = 0; t < NV; ++t)
    o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bool busy = qt * 16 < rows;
  // tokens of the chunk up to the query
  for (int kt = 0; busy && kt <= qt; ++kt) {
    f32x4 s{0.f, 0.f, 0.f, 0.f}, s2 = s; // two sums: the products of one do not wait for each other
    const float *kr = k + (kt * 16 + col) * a.dp + quad * 8;
    auto score = [&](const Frag<float> &kf, const Frag<float> &q) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s = mfma_f32(kf.lo[j], q.lo[j], s);
        s2 = mfma_f32(kf.hi[j], q.hi[j], s2);
      }
    };
    if constexpr (NF > 0) {
      Frag<float> kf[NF];
#pragma unroll
      for (int t = 0; t < NF; ++t)
        kf[t].load(kr + (t < nf ? t : 0) * 32); // past the last dimension: times zero
#pragma unroll
      for (int t = 0; t < NF; ++t)
        score(kf[t], qf[t]);
    } else {
      for (int t = 0; t < nf; ++t) {
        Frag<float> kf;
        kf.load(kr + t * 32);
        score(kf, query(t));
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int gap = qi - (kt * 16 + quad * 4 + r);
      s[r] = gap >= 0 ? (s[r] + s2[r]) * pw[max(gap, 0)] : 0.f;
    }
    float va[4][NV];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int t = 0; t < NV; ++t)
        va[r][t] = v[(kt * 16 + quad * 4 + r) * kVRow + vt0 + t * 16 + col];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int t = 0; t < NV; ++t)
        o[t] = mfma_f32(va[r][t], s[r], o[t]);
  }
  __syncthreads();
  // The state, its rows in the order in which the matrix instructions take them:
  // dimension t * 32 + q * 8 + j in row t * 32 + j * 4 + q.
  auto place = [](int d) { return (d & ~31) + (d & 7) * 4 + (d >> 3 & 3); };
  const int padded = nf * 32;
  if (a.quads) {
#pragma unroll
    for (int i = 0; i < kStateLoads; ++i)
      if (sr + i * 16 < a.dim)
        *reinterpret_cast<f32x4 *>(st + place(sr + i * 16) * kSRow + sc) = ahead[i];
    for (int r = sr + kStateLoads * 16; r < a.dim; r += 16)
      *reinterpret_cast<f32x4 *>(st + place(r) * kSRow + sc) =
          *reinterpret_cast<const f32x4 *>(S + (int64_t)r * a.vdim + (sc < vw ? sc : 0));
  } else {
    for (int r = sr; r < a.dim; r += 16)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        st[place(r) * kSRow + sc + j] = sc + j < vw ? S[(int64_t)r * a.vdim + sc + j] : 0.f;
  }
  for (int r = a.dim + sr; r < padded; r += 16) // times zero, but it must be a number
    *reinterpret_cast<f32x4 *>(st + place(r) * kSRow + sc) = f32x4{0.f, 0.f, 0.f, 0.f};
  __syncthreads();
  if (!busy)
    return;
  // state part: A = S^T (value channels x key dimensions), B = the scaled queries
  const float lead = pw[qi + 1];
  auto readout = [&](int t, const Frag<float> &q) {
    float sa[8][NV];
#pragma unroll
    for (int j = 0; j < 8; ++j)
#pragma unroll
      for (int x = 0; x < NV; ++x)
        sa[j][x] = st[(t * 32 + j * 4 + quad) * kSRow + vt0 + x * 16 + col];
#pragma unroll
    for (int j = 0; j < 8; ++j)
#pragma unroll
      for (int x = 0; x < NV; ++x)
        o[x] = mfma_f32(sa[j][x], (j < 4 ? q.lo[j & 3] : q.hi[j & 3]) * lead, o[x]);
  };
  if constexpr (NF > 0) {
#pragma unroll
    for (int t = 0; t < NF; ++t)
      if (t < nf)
        readout(t, qf[t]);
  } else {
    for (int t = 0; t < nf; ++t)
      readout(t, query(t));
  }
  if (qi >= rows)
    return;
  float *dst = out + ((int64_t)c * kLinearChunk + qi) * a.heads * a.vdim + (int64_t)h * a.vdim + v0;
#pragma unroll
  for (int t = 0; t < NV; ++t) {
    const int x = vt0 + t * 16 + quad * 4;
    if (a.quads && x < vw) {
      *reinterpret_cast<f32x4 *>(dst + x) = o[t];
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (x + r < vw)
          dst[x + r] = o[t][r];
    }
  }
}

template <int SV>
size_t out_lds_bytes(const LinearArgs &p) { // keys and values, or the state
  const size_t own = (size_t)kLinearChunk * (p.dp + SV + 4), state = (size_t)(p.dp - 4) * (SV + 8);
  return sizeof(float) * std::max(own, state);
}
constexpr size_t kLinearLds = 156 * 1024;

template <int SV> int launch_rows(const LinearRows &a, const LinearArgs &p, hipStream_t stream) {
  const LinearShape &s = a.s;
  const size_t chunk_lds = sizeof(float) * kLinearChunk * ((size_t)p.dp + 4 + SV + 8);
  static DynLdsOnce once_chunk;
  BH_CHECK_HIP(ensure_dyn_lds(once_chunk, (const void *)linear_chunk_kernel<SV>, (int)kLinearLds));
  const dim3 grid((unsigned)linear_chunks(a.rows), (unsigned)s.heads, (unsigned)ceil_div(s.vdim, SV));
  hipLaunchKernelGGL(linear_chunk_kernel<SV>, grid, dim3(SV * 4), chunk_lds, stream, a.proj,
                     a.chunk_states, p);
  const int64_t total = (int64_t)s.heads * s.dim * s.vdim;
  hipLaunchKernelGGL(linear_scan_kernel, dim3((unsigned)ceil_div(total, 256)), dim3(256), 0, stream,
                     a.chunk_states, a.state, s.dim * s.vdim, total, a.rows, a.powers);
#define BH_OUT(NF)                                                                                  \
  do {                                                                                              \
    static DynLdsOnce once;                                                                         \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)linear_out_kernel<SV, NF>, (int)kLinearLds));   \
    hipLaunchKernelGGL((linear_out_kernel<SV, NF>), grid, dim3(SV * 4), out_lds_bytes<SV>(p),       \
                       stream, a.proj, a.chunk_states, a.out, p);                                   \
  } while (0)
  if (s.dim <= 64)
    BH_OUT(2);
  else if (s.dim <= 128)
    BH_OUT(4);
  else
    BH_OUT(0);
#undef BH_OUT
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

} // namespace

int launch_linear_step(const LinearStep &a, hipStream_t stream) {
  BH_REQUIRE(a.q && a.k && a.v && a.powers && a.state && a.out && a.s.heads > 0 && a.s.dim > 0 &&
                 a.s.vdim > 0,
             "linear_step: bad argument");
  hipLaunchKernelGGL(linear_step_kernel, dim3(a.s.heads, (unsigned)ceil_div(a.s.vdim, 16)),
                     dim3(256), 0, stream, a.q, a.k, a.v, a.s.dim, a.s.vdim, a.powers, a.state,
                     a.out);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_linear_rows(const LinearRows &a, hipStream_t stream) {
  const LinearShape &s = a.s;
  BH_REQUIRE(a.proj && a.powers && a.state && a.chunk_states && a.out && a.rows > 0 && s.heads > 0 &&
                 s.dim > 0 && s.vdim > 0,
             "linear_rows: bad argument");
  LinearArgs p{s.heads, s.dim, s.vdim, a.ld, a.q_at, a.k_at, a.v_at, a.rows, 0, false, a.powers};
  p.dp = (int)round_up(s.dim, 32) + 4;
  p.quads = s.dim % 4 == 0 && s.vdim % 4 == 0 && a.ld % 4 == 0 && a.q_at % 4 == 0 &&
            a.k_at % 4 == 0 && a.v_at % 4 == 0 && ((uintptr_t)a.proj & 15) == 0 &&
            ((uintptr_t)a.chunk_states & 15) == 0 && ((uintptr_t)a.out & 15) == 0;
  if (s.vdim > 64 && out_lds_bytes<128>(p) <= kLinearLds)
    return launch_rows<128>(a, p, stream);
  BH_REQUIRE(out_lds_bytes<64>(p) <= kLinearLds, "linear_rows: key heads of %d values do not fit LDS",
             s.dim);
  return launch_rows<64>(a, p, stream);
}

} // namespace bh
