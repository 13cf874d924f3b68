// Element access for kernels that exist in bf16 and in fp32 (activations `uint16_t` = bf16 bits, or `float`), and the
// scalar functions of recurrences in full fp32 accuracy.
#pragma once

#include "common.hpp"

namespace sgl_amd {

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));

__device__ __forceinline__ float ld1(const uint16_t* p) { return bf2f(*p); }
__device__ __forceinline__ float ld1(const float* p) { return *p; }
__device__ __forceinline__ void st1(uint16_t* p, float v) { *p = f2bf(v); }
__device__ __forceinline__ void st1(float* p, float v) { *p = v; }

__device__ __forceinline__ void ld4(const uint16_t* p, float (&f)[4]) {
  const uint2 w = *reinterpret_cast<const uint2*>(p);
  f[0] = bf_lo(w.x); f[1] = bf_hi(w.x); f[2] = bf_lo(w.y); f[3] = bf_hi(w.y);
}
__device__ __forceinline__ void ld4(const float* p, float (&f)[4]) {
  const f32x4_t v = *reinterpret_cast<const f32x4_t*>(p);
  f[0] = v[0]; f[1] = v[1]; f[2] = v[2]; f[3] = v[3];
}
__device__ __forceinline__ void st4(uint16_t* p, const float (&f)[4]) {
  uint2 w;
  w.x = pack_bf2(f[0], f[1]); w.y = pack_bf2(f[2], f[3]);
  *reinterpret_cast<uint2*>(p) = w;
}
__device__ __forceinline__ void st4(float* p, const float (&f)[4]) {
  *reinterpret_cast<f32x4_t*>(p) = f32x4_t{f[0], f[1], f[2], f[3]};
}

__device__ __forceinline__ void ld8(const uint16_t* p, float (&f)[8]) {
  const U4 w = ld16(p);
  f[0] = bf_lo(w.x); f[1] = bf_hi(w.x); f[2] = bf_lo(w.y); f[3] = bf_hi(w.y);
  f[4] = bf_lo(w.z); f[5] = bf_hi(w.z); f[6] = bf_lo(w.w); f[7] = bf_hi(w.w);
}
__device__ __forceinline__ void ld8(const float* p, float (&f)[8]) {
  const f32x4_t a = *reinterpret_cast<const f32x4_t*>(p), b = *reinterpret_cast<const f32x4_t*>(p + 4);
  f[0] = a[0]; f[1] = a[1]; f[2] = a[2]; f[3] = a[3]; f[4] = b[0]; f[5] = b[1]; f[6] = b[2]; f[7] = b[3];
}
__device__ __forceinline__ void st8(uint16_t* p, const float (&f)[8]) {
  U4 w;
  w.x = pack_bf2(f[0], f[1]); w.y = pack_bf2(f[2], f[3]); w.z = pack_bf2(f[4], f[5]); w.w = pack_bf2(f[6], f[7]);
  st16(p, w);
}
__device__ __forceinline__ void st8(float* p, const float (&f)[8]) {
  *reinterpret_cast<f32x4_t*>(p) = f32x4_t{f[0], f[1], f[2], f[3]};
  *reinterpret_cast<f32x4_t*>(p + 4) = f32x4_t{f[4], f[5], f[6], f[7]};
}

// VEC consecutive elements, VEC in {1, 4, 8}
template <int VEC, typename T>
__device__ __forceinline__ void ldv(const T* p, float (&f)[VEC]) {
  if constexpr (VEC == 8) ld8(p, f);
  else if constexpr (VEC == 4) ld4(p, f);
  else f[0] = ld1(p);
}
template <int VEC, typename T>
__device__ __forceinline__ void stv(T* p, const float (&f)[VEC]) {
  if constexpr (VEC == 8) st8(p, f);
  else if constexpr (VEC == 4) st4(p, f);
  else st1(p, f[0]);
}

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
// log(1 + e^z) without overflow and without losing small values
__device__ __forceinline__ float softplus_f(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

inline bool aligned_to(const void* p, size_t n) { return (reinterpret_cast<uintptr_t>(p) & (n - 1)) == 0; }

}  // namespace sgl_amd
