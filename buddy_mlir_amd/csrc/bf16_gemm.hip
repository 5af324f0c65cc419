// bf16_gemm.hip -- many activation rows times resident bfloat16 matrices on the
// matrix cores: the matrix products of a prompt, plain and per expert.
//
// A workgroup of four wavefronts computes 16*RT rows x 64*GT channels.  Weights go
// from memory to registers as they lie (a tile is the A operand: 16 channels x 32
// k), each wavefront its own channels; the activation rows are the B operand and
// are shared through LDS, 128 bytes of every row per step.  Both are requested
// kStages - 1 steps ahead.  With f32 activations the same tiles are widened and
// multiplied by v_mfma_f32_16x16x4_f32, so nothing is rounded below 32 bits.
#include "bf16_linear.h"
#include "bf16_dev.h"

#include <algorithm>

namespace bh {
namespace {

constexpr int kGemmThreads = 256;
constexpr int kStages = 4;
constexpr int kRowBytes = 128;           // of one row per step
constexpr int kLdsRow = kRowBytes + 16;  // padded: rows start 4 banks apart

struct GemmDev {
  const void *A;
  void *C;
  int lda, ldc;
  int rows, K, groups; // groups of one matrix
  int ring_base, ring_mask;
  int silu_channels;
  GatedAct act;
  float limit;
  const int *counts, *lists;
  int experts, list_cap, list_div;
  int64_t expert_tiles;
};

template <typename T> struct ActTraits;
template <> struct ActTraits<bf16_bits> {
  static constexpr int kElems = 64, kTiles = 2; // per step: elements of a row, weight tiles
};
template <> struct ActTraits<float> {
  static constexpr int kElems = 32, kTiles = 1;
};

// the first `keep` elements of a 16-byte run, the others as zeros
template <typename T> __device__ __forceinline__ uint4 keep_run(uint4 v, int keep) {
  unsigned d[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    if constexpr (sizeof(T) == 4)
      d[j] = j < keep ? d[j] : 0u;
    else
      d[j] = 2 * j + 1 < keep ? d[j] : 2 * j < keep ? d[j] & 0xffffu : 0u;
  }
  return uint4{d[0], d[1], d[2], d[3]};
}

template <typename T>
__device__ __forceinline__ void store4(T *p, f32x4 v);
template <> __device__ __forceinline__ void store4<float>(float *p, f32x4 v) {
  *reinterpret_cast<f32x4 *>(p) = v;
}
template <> __device__ __forceinline__ void store4<bf16_bits>(bf16_bits *p, f32x4 v) {
  *reinterpret_cast<uint2 *>(p) = uint2{pack_bf(v[0], v[1]), pack_bf(v[2], v[3])};
}

// Workgroups go to the eight dies in turn, each with an L2 of its own.  A die takes a run
// of tiles, in panels of kPanel column blocks by all row blocks: the workgroups that it
// runs at the same time share rows and channels.
constexpr int kDies = 8, kPanel = 4;
__device__ __forceinline__ void place_tile(int &bx, int &by) {
  const int gx = gridDim.x, gy = gridDim.y, total = gx * gy, id = blockIdx.y * gx + blockIdx.x;
  const int die = id % kDies, q = total / kDies, r = total % kDies;
  const int t = die * q + min(die, r) + id / kDies;
  const int panel = t / (kPanel * gy), rest = t - panel * kPanel * gy;
  const int width = min(kPanel, gx - panel * kPanel);
  by = rest / width;
  bx = panel * kPanel + rest - by * width;
}

template <typename T, int RT, int GT, int OUT, bool GROUPED>
__global__ void __launch_bounds__(kGemmThreads)
rows_gemm_kernel(const uint4 *__restrict__ W, int ktiles, int steps, GemmDev a) {
  using Tr = ActTraits<T>;
  constexpr bool kPair = OUT == kOutExpertAct;
  constexpr int kGroups = kPair ? GT / 2 : GT; // channel groups of the result per wavefront
  constexpr int kRows = 16 * RT;
  constexpr int kRuns = kRows * 8;                               // 16-byte runs per step
  constexpr int kLoads = (kRuns + kGemmThreads - 1) / kGemmThreads;
  __shared__ __attribute__((aligned(16))) unsigned char lds[2][kRows * kLdsRow];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);

  int bx = blockIdx.x, by = blockIdx.y;
  if constexpr (!GROUPED)
    place_tile(bx, by);
  int row0 = by * kRows, rows = a.rows;
  const int *list = nullptr;
  if constexpr (GROUPED) {
    // blockIdx.y counts the row blocks of all experts: find this one's expert
    int block = blockIdx.y, e = -1;
    for (int base = 0; base < a.experts; base += 64) {
      const int i = base + lane;
      const int nb = i < a.experts ? (a.counts[i] + kRows - 1) / kRows : 0;
      int incl = nb;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int v = __shfl_up(incl, o, 64);
        if (lane >= o)
          incl += v;
      }
      const unsigned long long past = __ballot(incl > block);
      if (past) {
        const int l = __builtin_ctzll(past);
        block -= __builtin_amdgcn_readlane(incl - nb, l);
        e = base + l;
        break;
      }
      block -= __builtin_amdgcn_readlane(incl, 63);
    }
    if (e < 0)
      return; // more workgroups than row blocks
    e = __builtin_amdgcn_readfirstlane(e);
    row0 = block * kRows;
    rows = a.counts[e];
    list = a.lists + (int64_t)e * a.list_cap;
    W += (int64_t)e * a.expert_tiles * 64;
  }

  // the runs this thread moves: fixed rows, k advancing by the step
  const T *src[kLoads];
  int run_k[kLoads];
  int lds_at[kLoads];
#pragma unroll
  for (int i = 0; i < kLoads; ++i) {
    const int c = i * kGemmThreads + tid;
    const int r = c >> 3, q = c & 7;
    run_k[i] = q * (16 / (int)sizeof(T));
    lds_at[i] = r * kLdsRow + q * 16;
    // a row past the end repeats the last one: its column of the result is not stored
    const int lr = min(row0 + r, rows - 1);
    int pr;
    if constexpr (GROUPED)
      pr = list[lr] / a.list_div;
    else
      pr = (a.ring_base + lr) & a.ring_mask;
    src[i] = static_cast<const T *>(a.A) + (int64_t)pr * a.lda;
  }

  const int ch0 = (bx * 4 + wave) * kGroups; // first channel group of this wavefront
  const uint4 *wp[GT];
#pragma unroll
  for (int g = 0; g < GT; ++g) {
    const int mat = kPair ? g / kGroups : 0, gg = min(ch0 + (kPair ? g % kGroups : g), a.groups - 1);
    wp[g] = W + ((int64_t)(mat * a.groups + gg) * ktiles) * 64 + lane;
  }

  uint4 wr[kStages][GT * Tr::kTiles], ar[kStages][kLoads];
  constexpr int kRunElems = 16 / (int)sizeof(T);
  const int last_run = (a.K - 1) / kRunElems * kRunElems;
  const bool ragged = a.K % Tr::kElems != 0; // the last step reaches past K
  auto fetch = [&](int s, uint4 (&w)[GT * Tr::kTiles], uint4 (&x)[kLoads]) {
    const int t = min(s, steps - 1) * Tr::kTiles;
#pragma unroll
    for (int i = 0; i < kLoads; ++i)
      x[i] = *reinterpret_cast<const uint4 *>(src[i] + min(t * kBfTileK + run_k[i], last_run));
#pragma unroll
    for (int g = 0; g < GT; ++g)
#pragma unroll
      for (int u = 0; u < Tr::kTiles; ++u)
        w[g * Tr::kTiles + u] = wp[g][(int64_t)(t + u) * 64];
  };
#pragma unroll
  for (int s = 0; s < kStages - 1; ++s)
    fetch(s, wr[s], ar[s]);

  f32x4 acc[GT][RT];
#pragma unroll
  for (int g = 0; g < GT; ++g)
#pragma unroll
    for (int r = 0; r < RT; ++r)
      acc[g][r] = f32x4{0.f, 0.f, 0.f, 0.f};

  const int frag_at = (lane & 15) * kLdsRow + (lane >> 4) * 8 * (int)sizeof(T);
  auto step = [&](int s, uint4 (&w)[GT * Tr::kTiles], uint4 (&x)[kLoads], uint4 (&w_next)[GT * Tr::kTiles],
                  uint4 (&x_next)[kLoads], unsigned char *buf) {
    if (ragged && s == steps - 1) {
#pragma unroll
      for (int i = 0; i < kLoads; ++i)
        x[i] = keep_run<T>(x[i], a.K - s * Tr::kElems - run_k[i]);
    }
#pragma unroll
    for (int i = 0; i < kLoads; ++i)
      if (kRuns % kGemmThreads == 0 || i * kGemmThreads + tid < kRuns)
        *reinterpret_cast<uint4 *>(buf + lds_at[i]) = x[i];
    fetch(s + kStages - 1, w_next, x_next);
    __syncthreads(); // the other buffer was last read before the previous barrier
#pragma unroll
    for (int t = 0; t < Tr::kTiles; ++t) {
      Frag<T> b[RT];
#pragma unroll
      for (int r = 0; r < RT; ++r)
        b[r].load(reinterpret_cast<const T *>(buf + frag_at + r * 16 * kLdsRow +
                                              t * kBfTileK * (int)sizeof(T)));
#pragma unroll
      for (int g = 0; g < GT; ++g) {
        Frag<T> wf;
        if constexpr (sizeof(T) == 2)
          wf.v = w[g * Tr::kTiles + t];
        else
          wf = widen(w[g * Tr::kTiles + t]);
#pragma unroll
        for (int r = 0; r < RT; ++r)
          acc[g][r] = mfma32(wf, b[r], acc[g][r]);
      }
    }
  };
  static_assert(kStages == 4, "the stages below are written out");
  int s = 0;
  for (; s + kStages <= steps; s += kStages) {
    step(s, wr[0], ar[0], wr[3], ar[3], lds[0]);
    step(s + 1, wr[1], ar[1], wr[0], ar[0], lds[1]);
    step(s + 2, wr[2], ar[2], wr[1], ar[1], lds[0]);
    step(s + 3, wr[3], ar[3], wr[2], ar[2], lds[1]);
  }
  if (s < steps)
    step(s, wr[0], ar[0], wr[3], ar[3], lds[0]);
  if (s + 1 < steps)
    step(s + 1, wr[1], ar[1], wr[0], ar[0], lds[1]);
  if (s + 2 < steps)
    step(s + 2, wr[2], ar[2], wr[1], ar[1], lds[0]);

  // a lane holds channels (lane / 16) * 4 + 0..3 of row lane % 16 of every tile
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    const int lr = row0 + r * 16 + (lane & 15);
    if (lr >= rows)
      continue;
    int orow = lr;
    if constexpr (GROUPED)
      orow = list[lr];
#pragma unroll
    for (int g = 0; g < kGroups; ++g) {
      if (ch0 + g >= a.groups)
        continue;
      const int ch = (ch0 + g) * 16 + (lane >> 4) * 4;
      f32x4 v = acc[g][r];
      if constexpr (OUT == kOutExpertAct) {
        const f32x4 up = acc[g + kGroups][r];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          v[j] = gated_act(a.act, v[j], up[j], a.limit);
        store4<T>(static_cast<T *>(a.C) + (int64_t)orow * a.ldc + ch, v);
      } else if constexpr (OUT == kOutF32) {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (ch + j < a.silu_channels)
            v[j] = silu_f(v[j]);
        store4<float>(static_cast<float *>(a.C) + (int64_t)orow * a.ldc + ch, v);
      } else if constexpr (OUT == kOutAct) {
        store4<T>(static_cast<T *>(a.C) + (int64_t)orow * a.ldc + ch, v);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          store_act<T>(static_cast<T *>(a.C) + (int64_t)(ch + j) * a.ldc + orow, v[j]);
      }
    }
  }
}

template <typename T, int RT, int GT, int OUT, bool GROUPED>
int launch_variant(const RowsGemm &a, hipStream_t stream) {
  GemmDev d{};
  d.A = a.A;
  d.C = a.C;
  d.lda = a.lda;
  d.ldc = a.ldc;
  d.rows = a.rows;
  d.K = a.W.K;
  d.groups = a.W.groups();
  d.ring_base = a.ring_base;
  d.ring_mask = a.ring_mask;
  d.silu_channels = a.silu_channels;
  d.act = a.act;
  d.limit = a.limit;
  d.counts = a.counts;
  d.lists = a.lists;
  d.experts = a.experts;
  d.list_cap = a.list_cap;
  d.list_div = a.list_div;
  d.expert_tiles = a.expert_tiles;
  constexpr int per = 4 * (OUT == kOutExpertAct ? GT / 2 : GT);
  const int64_t blocks = GROUPED ? std::min<int64_t>(ceil_div(a.list_total, 16 * RT) + a.experts,
                                                     a.list_total)
                                 : ceil_div(a.rows, 16 * RT);
  BH_REQUIRE(blocks <= 65535, "rows_gemm: %lld row blocks", (long long)blocks);
  hipLaunchKernelGGL((rows_gemm_kernel<T, RT, GT, OUT, GROUPED>),
                     dim3((unsigned)ceil_div(d.groups, per), (unsigned)blocks), dim3(kGemmThreads),
                     0, stream, a.W.tiles, a.W.ktiles, (int)ceil_div(a.W.K, ActTraits<T>::kElems), d);
  BH_CHECK_HIP(hipGetLastError());
  return BUDDY_HIP_OK;
}

// rows and channels of a workgroup: tall tiles when there are rows for them, wide
// ones when the launch still fills the 256 compute units
template <typename T, int OUT, bool GROUPED>
int launch_shape(const RowsGemm &a, hipStream_t stream) {
  const int64_t rows = GROUPED ? ceil_div(a.list_total, a.experts) : a.rows;
  const int64_t all_blocks = GROUPED ? std::min<int64_t>(a.experts, a.list_total) : 1;
  constexpr int P = OUT == kOutExpertAct ? 2 : 1; // groups come in pairs
  auto workgroups = [&](int rt, int gt) {
    return ceil_div(a.W.groups(), 4 * gt / P) * ceil_div(rows, 16 * rt) * all_blocks;
  };
  if (rows <= 16)
    return workgroups(1, 2 * P) >= 256 ? launch_variant<T, 1, 2 * P, OUT, GROUPED>(a, stream)
                                       : launch_variant<T, 1, P, OUT, GROUPED>(a, stream);
  if (rows <= 32)
    return workgroups(2, 2 * P) >= 256 ? launch_variant<T, 2, 2 * P, OUT, GROUPED>(a, stream)
                                       : launch_variant<T, 2, P, OUT, GROUPED>(a, stream);
  // what a workgroup fetches per product shrinks with both sides of its tile
  if constexpr (sizeof(T) == 2) {
    // -- but one such workgroup fills a compute unit: whole rounds of 256 pay
    const int64_t w = workgroups(8, 4);
    if (rows > 64 && w >= 240 && w * 5 >= round_up(w, 256) * 4)
      return launch_variant<T, 8, 4, OUT, GROUPED>(a, stream);
  }
  return workgroups(4, 2 * P) >= 256 ? launch_variant<T, 4, 2 * P, OUT, GROUPED>(a, stream)
                                     : launch_variant<T, 4, P, OUT, GROUPED>(a, stream);
}

template <typename T> int launch_typed(const RowsGemm &a, hipStream_t stream) {
  const bool grouped = a.counts != nullptr;
  switch (a.out) {
  case kOutF32:
    return grouped ? launch_shape<T, kOutF32, true>(a, stream)
                   : launch_shape<T, kOutF32, false>(a, stream);
  case kOutAct:
    BH_REQUIRE(!grouped, "rows_gemm: form not compiled for expert lists");
    return launch_shape<T, kOutAct, false>(a, stream);
  case kOutActTrans:
    BH_REQUIRE(!grouped, "rows_gemm: form not compiled for expert lists");
    return launch_shape<T, kOutActTrans, false>(a, stream);
  case kOutExpertAct:
    return grouped ? launch_shape<T, kOutExpertAct, true>(a, stream)
                   : launch_shape<T, kOutExpertAct, false>(a, stream);
  }
  return fail(BUDDY_HIP_ERR_ARG, "rows_gemm: output form %d", (int)a.out);
}

} // namespace

int launch_rows_gemm(const RowsGemm &a, hipStream_t stream) {
  const Bf16Matrix &W = a.W;
  BH_REQUIRE(W.tiles && W.K > 0 && W.N > 0 && W.N % 16 == 0 && W.ktiles == bf16_ktiles(W.K) &&
                 a.A && a.C && a.rows >= 0,
             "rows_gemm: bad argument");
  // rows are read 16 bytes at a time up to the run that holds element K - 1
  BH_REQUIRE(a.lda % 8 == 0 && a.lda >= round_up(W.K, 8) && ((uintptr_t)a.A & 15) == 0,
             "rows_gemm: activation rows must be 16-byte aligned (lda %d, K %d)", a.lda, W.K);
  BH_REQUIRE(((uintptr_t)a.C & 15) == 0 &&
                 (a.out == kOutActTrans ? a.ldc >= a.rows : (a.ldc % 4 == 0 && a.ldc >= W.N)),
             "rows_gemm: result rows (ldc %d, N %d)", a.ldc, W.N);
  BH_REQUIRE(!a.counts || (a.lists && a.experts > 0 && a.list_cap > 0 && a.list_div > 0),
             "rows_gemm: expert lists");
  if (a.counts ? a.list_total == 0 : a.rows == 0)
    return BUDDY_HIP_OK;
  return a.f32 ? launch_typed<float>(a, stream) : launch_typed<bf16_bits>(a, stream);
}

} // namespace bh

extern "C" {

int buddy_hip_gemm_bf16(const void *A, int64_t lda, int dtype, const void *tiles, float *C,
                        int64_t ldc, int64_t M, int64_t K, int64_t N, buddy_hip_stream stream) try {
  BH_REQUIRE(A && tiles && C && M > 0 && K > 0 && N > 0 && M < (1 << 30) && K < (1 << 30) &&
                 N < (1 << 30) && lda < (1 << 30) && ldc < (1 << 30) &&
                 (dtype == BUDDY_HIP_MODEL_BF16 || dtype == BUDDY_HIP_MODEL_F32),
             "gemm_bf16: bad argument");
  bh::RowsGemm g;
  g.W.tiles = static_cast<const uint4 *>(tiles);
  g.W.K = (int)K;
  g.W.N = (int)bh::round_up(N, 16);
  g.W.ktiles = bh::bf16_ktiles(K);
  g.A = A;
  g.lda = (int)lda;
  g.f32 = dtype == BUDDY_HIP_MODEL_F32;
  g.rows = (int)M;
  g.C = C;
  g.ldc = (int)ldc;
  return bh::launch_rows_gemm(g, bh::as_stream(stream));
} BH_CATCH_INT("buddy_hip_gemm_bf16")
}
