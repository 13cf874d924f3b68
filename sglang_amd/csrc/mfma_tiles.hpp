// Fragments of the 16x16x32 bf16 matrix instruction, and a transposed operand straight from a row-major LDS tile.
#pragma once

#include "elem_io.hpp"

namespace sgl_amd {

constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ bf16x8_t as_frag(const U4& v) { return __builtin_bit_cast(bf16x8_t, v); }
// v, or zeros
__device__ __forceinline__ U4 keep_if(U4 v, bool k) {
  const uint32_t m = k ? 0xffffffffu : 0u;
  v.x &= m; v.y &= m; v.z &= m; v.w &= m;
  return v;
}

__device__ __forceinline__ f32x4_t mfma_bf16(bf16x8_t a, bf16x8_t b, f32x4_t c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

typedef short v4s16_t __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) v4s16_t* lds_v4_t;

// columns c .. c + 15 (one per lane of a 16-lane group) of rows r0 + 4 g + {0..3} and r0 + 16 + 4 g + {0..3} of a row-major tile
__device__ __forceinline__ bf16x8_t read_transposed(const uint16_t* tile, int row_elems, int r0, int c, int i16, int g) {
  const uint16_t* a = tile + (r0 + 4 * g + (i16 >> 2)) * row_elems + c + (i16 & 3) * 4;
  const v4s16_t lo = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4_t)(a));
  const v4s16_t hi = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_v4_t)(a + 16 * row_elems));
  U4 o;
  o.x = __builtin_bit_cast(uint2, lo).x; o.y = __builtin_bit_cast(uint2, lo).y;
  o.z = __builtin_bit_cast(uint2, hi).x; o.w = __builtin_bit_cast(uint2, hi).y;
  return as_frag(o);
}

}  // namespace sgl_amd
