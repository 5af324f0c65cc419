// row_ops.hip -- residual, norm, convolution and routing of many rows.
#include "row_ops.h"
#include "bf16_dev.h"
#include "bf16_linear.h"

#include <algorithm>

namespace bh {
namespace {

__device__ __forceinline__ float block_sum4(float v, float *red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0)
    red[threadIdx.x >> 6] = v;
  __syncthreads();
  return (red[0] + red[1]) + (red[2] + red[3]);
}

__global__ void __launch_bounds__(256)
embed_rows_kernel(const uint16_t *__restrict__ table, const int *__restrict__ tokens, int width,
                  int vocab, float scale, const float *__restrict__ norm_w, float eps,
                  float *__restrict__ x) {
  __shared__ float red[4];
  int t = tokens[blockIdx.x];
  if (t < 0 || t >= vocab)
    t = 0;
  const uint16_t *row = table + (int64_t)t * width;
  float *dst = x + (int64_t)blockIdx.x * width;
  if (norm_w) {
    float ss = 0.f;
    for (int i = threadIdx.x; i < width; i += 256) {
      const float v = bf_f(row[i]) * scale;
      ss = fmaf(v, v, ss);
    }
    const float g = scale / sqrtf(block_sum4(ss, red) / (float)width + eps);
    for (int i = threadIdx.x; i < width; i += 256)
      dst[i] = bf_f(row[i]) * g * norm_w[i];
    return;
  }
  for (int i = threadIdx.x; i < width; i += 256)
    dst[i] = bf_f(row[i]) * scale;
}

// V consecutive values of a row at a time: 4 where every row is 16-byte aligned, else 1
template <int V> struct Run {
  float v[V];
};
template <int V> __device__ __forceinline__ Run<V> load_run(const float *p) {
  Run<V> r;
  if constexpr (V == 4) {
    const f32x4 x = *reinterpret_cast<const f32x4 *>(p);
#pragma unroll
    for (int j = 0; j < V; ++j)
      r.v[j] = x[j];
  } else {
    r.v[0] = *p;
  }
  return r;
}
template <int V> __device__ __forceinline__ void store_run(float *p, const Run<V> &r) {
  if constexpr (V == 4)
    *reinterpret_cast<f32x4 *>(p) = f32x4{r.v[0], r.v[1], r.v[2], r.v[3]};
  else
    *p = r.v[0];
}
template <int V> __device__ __forceinline__ void store_run(bf16_bits *p, const Run<V> &r) {
  if constexpr (V == 4)
    *reinterpret_cast<uint2 *>(p) = uint2{pack_bf(r.v[0], r.v[1]), pack_bf(r.v[2], r.v[3])};
  else
    *p = f_bf(r.v[0]);
}

template <typename T, int V>
__global__ void __launch_bounds__(256) norm_rows_kernel(NormRows a) {
  extern __shared__ __attribute__((aligned(16))) float lds[]; // x' of the row, then y
  __shared__ float red[2][4];
  const int tid = threadIdx.x * V, W = a.width;
  const int64_t r = a.pick ? a.pick[blockIdx.x] : blockIdx.x;
  float *x = a.x + r * W;
  float *xb = lds, *yb = lds + W;
  const bool pending = a.y || a.expert_out || a.add;
  float ss = 0.f;
  for (int i = tid; i < W; i += 256 * V) {
    store_run<V>(xb + i, load_run<V>(x + i));
    if (pending) {
      Run<V> y{};
      if (a.y)
        y = load_run<V>(a.y + r * a.ldy + i);
      for (int j = 0; j < a.top; ++j) {
        const float w = a.expert_w[r * a.top + j];
        const Run<V> e = load_run<V>(a.expert_out + (r * a.top + j) * a.lde + i);
#pragma unroll
        for (int k = 0; k < V; ++k)
          y.v[k] = fmaf(w, e.v[k], y.v[k]);
      }
      if (a.add) { // (only with plain_y)
        const Run<V> e = load_run<V>(a.add + i);
#pragma unroll
        for (int k = 0; k < V; ++k)
          y.v[k] += e.v[k];
      }
      store_run<V>(yb + i, y);
#pragma unroll
      for (int k = 0; k < V; ++k)
        ss = fmaf(y.v[k], y.v[k], ss);
    }
  }
  float sx = 0.f;
  if (pending) {
    const float ry = a.plain_y ? 1.0f : a.out_gain / sqrtf(block_sum4(ss, red[0]) / (float)W + a.eps);
    for (int i = tid; i < W; i += 256 * V) {
      Run<V> v = load_run<V>(xb + i);
      const Run<V> y = load_run<V>(yb + i);
#pragma unroll
      for (int k = 0; k < V; ++k)
        v.v[k] = fmaf(y.v[k], ry, v.v[k]);
      store_run<V>(xb + i, v);
      if (a.write_x)
        store_run<V>(x + i, v);
    }
  }
  if (!a.out_f32 && !a.out_act)
    return;
  for (int i = tid; i < W; i += 256 * V) {
    const Run<V> v = load_run<V>(xb + i);
#pragma unroll
    for (int k = 0; k < V; ++k)
      sx = fmaf(v.v[k], v.v[k], sx);
  }
  const float g = a.gain / sqrtf(block_sum4(sx, red[1]) / (float)W + a.eps);
  for (int i = tid; i < W; i += 256 * V) {
    Run<V> v = load_run<V>(xb + i);
#pragma unroll
    for (int k = 0; k < V; ++k)
      v.v[k] *= g;
    if (a.norm_w) {
      const Run<V> w = load_run<V>(a.norm_w + i);
#pragma unroll
      for (int k = 0; k < V; ++k)
        v.v[k] *= w.v[k];
    }
    if (a.out_f32)
      store_run<V>(a.out_f32 + (int64_t)blockIdx.x * W + i, v);
    if (a.out_act)
      store_run<V>(static_cast<T *>(a.out_act) + (int64_t)blockIdx.x * a.ld_act + i, v);
  }
}

template <typename T, int V> __global__ void __launch_bounds__(256) conv_rows_kernel(ConvRows a) {
  const int64_t r = blockIdx.x;
  const int p = a.start + (int)r;
  for (int i = (blockIdx.y * 256 + threadIdx.x) * V; i < a.width; i += gridDim.y * 256 * V) {
    const Run<V> h = load_run<V>(a.h + r * a.width + i);
    Run<V> c{};
    for (int b = a.taps - 1; b >= 1; --b) {
      if (p - b < 0)
        continue;
      const Run<V> e = load_run<V>(r >= b ? a.h + (r - b) * a.width + i
                                          : a.ring + (int64_t)((p - b) % a.taps) * a.width + i);
      const Run<V> w = load_run<V>(a.w + (int64_t)(a.taps - 1 - b) * a.width + i);
#pragma unroll
      for (int k = 0; k < V; ++k)
        c.v[k] = fmaf(w.v[k], e.v[k], c.v[k]);
    }
    const Run<V> w = load_run<V>(a.w + (int64_t)(a.taps - 1) * a.width + i);
#pragma unroll
    for (int k = 0; k < V; ++k)
      c.v[k] = h.v[k] + fmaf(w.v[k], h.v[k], c.v[k]);
    store_run<V>(static_cast<T *>(a.out) + r * a.ld + i, c);
  }
}

// one thread per channel: the last rows into their slots, and what the ring adds next
__global__ void __launch_bounds__(64)
conv_save_kernel(const float *__restrict__ h, const float *__restrict__ w, float *__restrict__ ring,
                 float *__restrict__ next, int taps, int width, int rows, int start) {
  const int i = blockIdx.x * 64 + threadIdx.x;
  if (i >= width)
    return;
  const int end = start + rows;
  float c = 0.f;
  for (int b = taps - 1; b >= 1; --b) {
    if (end - b < 0)
      continue;
    const float e = rows >= b ? h[(int64_t)(rows - b) * width + i]
                              : ring[(int64_t)((end - b) % taps) * width + i];
    c = fmaf(w[(int64_t)(taps - 1 - b) * width + i], e, c);
    if (rows >= b)
      ring[(int64_t)((end - b) % taps) * width + i] = e;
  }
  next[(int64_t)(end & 1) * width + i] = c;
}

template <typename T> __global__ void __launch_bounds__(256) gated_norm_rows_kernel(GatedNormRows a) {
  extern __shared__ float lds[];
  __shared__ float red[4];
  const int64_t r = blockIdx.x;
  float ss = 0.f;
  for (int i = threadIdx.x; i < a.width; i += 256) {
    const float v = a.x[r * a.width + i];
    lds[i] = v;
    ss = fmaf(v, v, ss);
  }
  const float g = 1.0f / sqrtf(block_sum4(ss, red) / (float)a.width + a.eps);
  for (int i = threadIdx.x; i < a.width; i += 256)
    store_act<T>(static_cast<T *>(a.out) + r * a.ld + i,
                 lds[i] * g * a.w[i] * sigmoid_f(a.gate[r * a.ld_gate + i]));
}

__device__ __forceinline__ unsigned rank_key(float f) {
  const unsigned u = __float_as_uint(f);
  return max(u & 0x80000000u ? ~u : u | 0x80000000u, 1u);
}

// A wavefront per row, four rows per workgroup.
template <int R>
__global__ void __launch_bounds__(256) route_pick_kernel(RouteRows a) {
  const int lane = threadIdx.x & 63;
  const int64_t row = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (row >= a.rows)
    return;
  float val[R];
  unsigned key[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int i = r * 64 + lane;
    val[r] = a.logits[row * a.ld + min(i, a.experts - 1)];
    key[r] = i < a.experts ? rank_key(val[r]) : 0u;
  }
  float mine = -INFINITY;
  int mine_idx = 0;
  for (int it = 0; it < a.top; ++it) {
    unsigned best = key[0];
#pragma unroll
    for (int r = 1; r < R; ++r)
      best = max(best, key[r]);
    const unsigned m = wave_max_u32(best);
    bool found = false;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      const unsigned long long b = __ballot(key[r] == m);
      if (!found && b) {
        found = true;
        const int l = __builtin_ctzll(b);
        const float z = lane_f(val[r], l);
        if (lane == l)
          key[r] = 0;
        if (lane == it) {
          mine = z;
          mine_idx = r * 64 + l;
        }
      }
    }
  }
  const float most = wave_max(mine); // with all lanes, not under the condition below
  const float e = lane < a.top ? expf(mine - most) : 0.f;
  const float w = e / wave_sum(e);
  if (lane < a.top) {
    a.chosen[row * a.top + lane] = mine_idx;
    a.weights[row * a.top + lane] = w;
  }
}

// A workgroup per expert walks all assignments in order.
__global__ void __launch_bounds__(1024)
route_list_kernel(const int *__restrict__ chosen, int total, int *__restrict__ counts,
                  int *__restrict__ lists, int list_cap) {
  __shared__ int wave_count[16];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int *list = lists + (int64_t)e * list_cap;
  int have = 0;
  for (int base = 0; base < total; base += 1024) {
    const int i = base + tid;
    const bool hit = i < total && chosen[i] == e;
    const unsigned long long b = __ballot(hit);
    if (lane == 0)
      wave_count[wave] = __popcll(b);
    __syncthreads();
    int before = have;
    for (int w = 0; w < 16; ++w) {
      if (w < wave)
        before += wave_count[w];
      have += wave_count[w];
    }
    if (hit)
      list[before + __popcll(b & ((1ull << lane) - 1))] = i;
    __syncthreads();
  }
  if (tid == 0)
    counts[e] = have;
}

} // namespace

int launch_embed_rows(const uint16_t *table, const int *tokens, int rows, int width, int vocab,
                      float scale, const float *norm_w, float eps, float *x, hipStream_t stream) {
  BH_REQUIRE(table && tokens && x && rows > 0 && width > 0 && vocab > 0, "embed_rows: bad argument");
  hipLaunchKernelGGL(embed_rows_kernel, dim3(rows), dim3(256), 0, stream, table, tokens, width,
                     vocab, scale, norm_w, eps, x);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_norm_rows(const NormRows &a, hipStream_t stream) {
  BH_REQUIRE(a.x && a.rows > 0 && a.width > 0 && (!a.pick || !a.write_x) &&
                 (!a.expert_out || (a.expert_w && a.top > 0)) && (a.expert_out || a.top == 0) &&
                 (!a.add || a.plain_y),
             "norm_rows: bad argument");
  const size_t lds = 2 * sizeof(float) * (size_t)a.width;
  constexpr size_t kLimit = 150 * 1024;
  BH_REQUIRE(lds <= kLimit, "norm_rows: a row of %d values does not fit LDS", a.width);
  bool quads = a.width % 4 == 0 && a.ldy % 4 == 0 && a.lde % 4 == 0 && a.ld_act % 4 == 0;
  for (const void *p : {(const void *)a.x, (const void *)a.y, (const void *)a.expert_out,
                        (const void *)a.add, (const void *)a.norm_w, (const void *)a.out_f32, (const void *)a.out_act})
    quads = quads && ((uintptr_t)p & 15) == 0;
#define BH_NORM(T, V)                                                                          \
  do {                                                                                         \
    static DynLdsOnce once;                                                                    \
    BH_CHECK_HIP(ensure_dyn_lds(once, (const void *)norm_rows_kernel<T, V>, (int)kLimit));     \
    hipLaunchKernelGGL((norm_rows_kernel<T, V>), dim3(a.rows), dim3(256), lds, stream, a);     \
  } while (0)
  if (a.act_f32) {
    if (quads)
      BH_NORM(float, 4);
    else
      BH_NORM(float, 1);
  } else {
    if (quads)
      BH_NORM(bf16_bits, 4);
    else
      BH_NORM(bf16_bits, 1);
  }
#undef BH_NORM
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_conv_rows(const ConvRows &a, hipStream_t stream) {
  BH_REQUIRE(a.h && a.w && a.ring && a.next && a.out && a.taps > 0 && a.width > 0 && a.rows > 0 && a.start >= 0,
             "conv_rows: bad argument");
  const bool quads = a.width % 4 == 0 && a.ld % 4 == 0 &&
                     (((uintptr_t)a.h | (uintptr_t)a.w | (uintptr_t)a.ring | (uintptr_t)a.out) & 15) == 0;
  const dim3 grid((unsigned)a.rows, (unsigned)std::min<int64_t>(4, ceil_div(a.width, quads ? 1024 : 256)));
  if (a.act_f32 && quads)
    hipLaunchKernelGGL((conv_rows_kernel<float, 4>), grid, dim3(256), 0, stream, a);
  else if (a.act_f32)
    hipLaunchKernelGGL((conv_rows_kernel<float, 1>), grid, dim3(256), 0, stream, a);
  else if (quads)
    hipLaunchKernelGGL((conv_rows_kernel<bf16_bits, 4>), grid, dim3(256), 0, stream, a);
  else
    hipLaunchKernelGGL((conv_rows_kernel<bf16_bits, 1>), grid, dim3(256), 0, stream, a);
  hipLaunchKernelGGL(conv_save_kernel, dim3((unsigned)ceil_div(a.width, 64)), dim3(64), 0, stream,
                     a.h, a.w, a.ring, a.next, a.taps, a.width, a.rows, a.start);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_gated_norm_rows(const GatedNormRows &a, hipStream_t stream) {
  BH_REQUIRE(a.x && a.w && a.gate && a.out && a.rows > 0 && a.width > 0 && a.width <= 16384,
             "gated_norm_rows: bad argument");
  const size_t lds = sizeof(float) * (size_t)a.width;
  if (a.act_f32)
    hipLaunchKernelGGL(gated_norm_rows_kernel<float>, dim3(a.rows), dim3(256), lds, stream, a);
  else
    hipLaunchKernelGGL(gated_norm_rows_kernel<bf16_bits>, dim3(a.rows), dim3(256), lds, stream, a);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

int launch_route_rows(const RouteRows &a, hipStream_t stream) {
  BH_REQUIRE(a.logits && a.chosen && a.weights && a.counts && a.lists && a.rows > 0 &&
                 a.experts > 0 && a.experts <= kMaxExperts && a.top > 0 && a.top <= 64 &&
                 a.top <= a.experts && a.list_cap >= a.rows,
             "route_rows: bad argument");
  const dim3 grid((unsigned)ceil_div(a.rows, 4));
  if (a.experts <= 64)
    hipLaunchKernelGGL(route_pick_kernel<1>, grid, dim3(256), 0, stream, a);
  else
    hipLaunchKernelGGL(route_pick_kernel<kMaxExperts / 64>, grid, dim3(256), 0, stream, a);
  hipLaunchKernelGGL(route_list_kernel, dim3(a.experts), dim3(1024), 0, stream, a.chosen,
                     a.rows * a.top, a.counts, a.lists, a.list_cap);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

} // namespace bh
