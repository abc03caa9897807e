// bf16 MFMA helpers of the chunked matrix-state kernels: fp32 operands go
// through the matrix cores as two bf16 halves, x = hi + lo.
#pragma once

#include "elem_types.h"

typedef __bf16 mc_bf16x8 __attribute__((ext_vector_type(8)));
typedef uint16_t u16x4 __attribute__((ext_vector_type(4)));

#define MC_T 64   // tokens per chunk
#define MC_TP 72  // padded LDS row of one

LIG_DEVICE f32x4 mc_mfma(u16x8 a, u16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(mc_bf16x8, a),
                                                 __builtin_bit_cast(mc_bf16x8, b), c, 0, 0, 0);
}

LIG_DEVICE void mc_split(float x, uint16_t& hi, uint16_t& lo) {
  hi = f32_to_bf16(x);
  lo = f32_to_bf16(x - bf16_to_f32(hi));
}

typedef float f32x2 __attribute__((ext_vector_type(2)));
typedef __bf16 mc_bf16x2 __attribute__((ext_vector_type(2)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));

// The same for two neighbours at once, packed as an operand holds them.
LIG_DEVICE void mc_split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2{a, b}, mc_bf16x2));
  const float ra = a - __builtin_bit_cast(float, hi << 16);
  const float rb = b - __builtin_bit_cast(float, hi & 0xffff0000u);
  lo = __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2{ra, rb}, mc_bf16x2));
}
// Four accumulator entries into half `half` (0 or 1) of an operand pair.
LIG_DEVICE void mc_split4(f32x4 x, int half, u32x4& hi, u32x4& lo) {
  uint32_t h0, h1, l0, l1;
  mc_split2(x[0], x[1], h0, l0);
  mc_split2(x[2], x[3], h1, l1);
  hi[2 * half] = h0;
  hi[2 * half + 1] = h1;
  lo[2 * half] = l0;
  lo[2 * half + 1] = l1;
}
LIG_DEVICE f32x4 mc_mfma(u32x4 a, u16x8 b, f32x4 c) { return mc_mfma(__builtin_bit_cast(u16x8, a), b, c); }
LIG_DEVICE f32x4 mc_mfma(u16x8 a, u32x4 b, f32x4 c) { return mc_mfma(a, __builtin_bit_cast(u16x8, b), c); }

LIG_DEVICE u16x8 mc_ld16(const uint16_t* p) { return *reinterpret_cast<const u16x8*>(p); }
LIG_DEVICE u16x8 mc_ld8x2(const uint16_t* p, const uint16_t* q) {
  const u16x4 a = *reinterpret_cast<const u16x4*>(p), b = *reinterpret_cast<const u16x4*>(q);
  return u16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}
// 16 bytes to an 8-byte aligned place.
LIG_DEVICE void mc_st8x2(uint16_t* p, u16x8 v) {
  *reinterpret_cast<u16x4*>(p) = u16x4{v[0], v[1], v[2], v[3]};
  *reinterpret_cast<u16x4*>(p + 4) = u16x4{v[4], v[5], v[6], v[7]};
}
