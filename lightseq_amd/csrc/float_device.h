// Device helpers of the floating-point decoder kernels (bfloat16 serving, true float32): element
// traits, 16-byte fragments and the matrix-core products over them.
//
// A fragment is 16 bytes of a K-contiguous row: 8 bfloat16 or 4 float values.  mma32 / mma16 take
// one fragment per lane of either operand.  For bfloat16 that is one instruction; for float32
// four, each contracting one element per lane -- the elements pair up between the operands, so the
// sum runs over the same products, in full float32 (there is no reduced-precision float mode on
// this chip).  Both types therefore share every tile layout of this library, counted in bytes.
#pragma once
#include "ls_device.h"

namespace lsh {

typedef __bf16 bf16_t;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16v __attribute__((ext_vector_type(16)));
typedef uint32_t frag_t __attribute__((ext_vector_type(4)));  // 16 bytes

template <typename T>
struct FT;
template <>
struct FT<float> {
  static constexpr int kVec = 4;  // elements per fragment
};
template <>
struct FT<bf16_t> {
  static constexpr int kVec = 8;
};

__device__ __forceinline__ float to_f(float x) { return x; }
__device__ __forceinline__ float to_f(bf16_t x) { return (float)x; }
template <typename T>
__device__ __forceinline__ T from_f(float x) {
  return (T)x;
}

__device__ __forceinline__ f32x16v mma32(bf16_t, frag_t a, frag_t b, f32x16v c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
__device__ __forceinline__ f32x16v mma32(float, frag_t a, frag_t b, f32x16v c) {
  const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
  for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_32x32x2f32(x[j], y[j], c, 0, 0, 0);
  return c;
}
__device__ __forceinline__ f32x4 mma16(bf16_t, frag_t a, frag_t b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a),
                                                 __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma16(float, frag_t a, frag_t b, f32x4 c) {
  const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
#pragma unroll
  for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], y[j], c, 0, 0, 0);
  return c;
}

// V consecutive elements as floats (V * sizeof(T) <= 16, aligned to that)
template <int V, typename T>
__device__ __forceinline__ void ldv(const T* p, float (&o)[V]) {
  typedef T tv __attribute__((ext_vector_type(V)));
  const tv t = *reinterpret_cast<const tv*>(p);
#pragma unroll
  for (int k = 0; k < V; ++k) o[k] = to_f((T)t[k]);
}
template <int V, typename T>
__device__ __forceinline__ void stv(T* p, const float (&o)[V]) {
  typedef T tv __attribute__((ext_vector_type(V)));
  tv t;
#pragma unroll
  for (int k = 0; k < V; ++k) t[k] = from_f<T>(o[k]);
  *reinterpret_cast<tv*>(p) = t;
}
template <>
__device__ __forceinline__ void ldv<1, float>(const float* p, float (&o)[1]) { o[0] = *p; }
template <>
__device__ __forceinline__ void ldv<1, bf16_t>(const bf16_t* p, float (&o)[1]) { o[0] = (float)*p; }
template <>
__device__ __forceinline__ void stv<1, float>(float* p, const float (&o)[1]) { *p = o[0]; }
template <>
__device__ __forceinline__ void stv<1, bf16_t>(bf16_t* p, const float (&o)[1]) { *p = (bf16_t)o[0]; }

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
// log(1 + exp(z)) without overflow
__device__ __forceinline__ float softplus_f(float z) {
  return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
}

}  // namespace lsh
