// bf16_dev.h -- device helpers shared by the kernels on bfloat16 weights.
#pragma once

#include "common.h"

namespace bh {

// How a gate and an up value become one.
enum GatedAct {
  kActClamped = 0, // g = min(g, limit), u = clamp(u, +-limit): g * sigmoid(1.702 g) * (u + 1)
  kActGeluTanh = 1 // gelu(g) * u, the tanh form of gelu
};

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef unsigned u32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef unsigned short bf16_bits;

#if defined(__HIPCC__)
__device__ __forceinline__ float bf_lo(unsigned u) { return __uint_as_float(u << 16); }
__device__ __forceinline__ float bf_hi(unsigned u) { return __uint_as_float(u & 0xffff0000u); }
__device__ __forceinline__ float bf_f(bf16_bits b) { return __uint_as_float((unsigned)b << 16); }
// round to nearest even; a NaN stays a NaN
__device__ __forceinline__ bf16_bits f_bf(float f) {
  const __bf16 b = (__bf16)f;
  return __builtin_bit_cast(bf16_bits, b);
}
__device__ __forceinline__ unsigned pack_bf(float a, float b) {
  return (unsigned)f_bf(a) | ((unsigned)f_bf(b) << 16);
}
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z * sigmoid_f(z); }
// z * (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))) / 2, by (1 + tanh(y)) / 2 = sigmoid(2 y)
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return z * sigmoid_f(1.59576912160573071f * fmaf(0.044715f * z * z, z, z));
}
__device__ __forceinline__ float expert_act(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(1.702f * g) * (u + 1.0f);
}
__device__ __forceinline__ float gated_act(GatedAct act, float g, float u, float limit) {
  return act == kActGeluTanh ? gelu_tanh_f(g) * u : expert_act(g, u, limit);
}

// an element of an activation buffer
template <typename T> __device__ __forceinline__ float load_act(const T *p);
template <> __device__ __forceinline__ float load_act<float>(const float *p) { return *p; }
template <> __device__ __forceinline__ float load_act<bf16_bits>(const bf16_bits *p) { return bf_f(*p); }
template <typename T> __device__ __forceinline__ void store_act(T *p, float v);
template <> __device__ __forceinline__ void store_act<float>(float *p, float v) { *p = v; }
template <> __device__ __forceinline__ void store_act<bf16_bits>(bf16_bits *p, float v) { *p = f_bf(v); }

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mfma_bf16(uint4 a, uint4 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
// Eight consecutive k of one row as a matrix operand.  In the f32 form a product
// of 32 k is eight instructions whose k are (lane / 16) * 8 + j: both operands
// name them in the same order, so lying consecutively is enough.
template <typename T> struct Frag;
template <> struct Frag<bf16_bits> {
  uint4 v;
  __device__ __forceinline__ void load(const bf16_bits *p) { v = *reinterpret_cast<const uint4 *>(p); }
};
template <> struct Frag<float> {
  f32x4 lo, hi;
  __device__ __forceinline__ void load(const float *p) {
    lo = *reinterpret_cast<const f32x4 *>(p);
    hi = *reinterpret_cast<const f32x4 *>(p + 4);
  }
};
__device__ __forceinline__ Frag<float> widen(uint4 w) {
  Frag<float> f;
  f.lo = f32x4{bf_lo(w.x), bf_hi(w.x), bf_lo(w.y), bf_hi(w.y)};
  f.hi = f32x4{bf_lo(w.z), bf_hi(w.z), bf_lo(w.w), bf_hi(w.w)};
  return f;
}
__device__ __forceinline__ f32x4 mfma32(const Frag<bf16_bits> &a, const Frag<bf16_bits> &b, f32x4 c) {
  return mfma_bf16(a.v, b.v, c);
}
__device__ __forceinline__ f32x4 mfma32(const Frag<float> &a, const Frag<float> &b, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 4; ++j)
    c = mfma_f32(a.lo[j], b.lo[j], c);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    c = mfma_f32(a.hi[j], b.hi[j], c);
  return c;
}
#endif

} // namespace bh
