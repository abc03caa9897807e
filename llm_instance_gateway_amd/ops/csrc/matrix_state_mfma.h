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

LIG_DEVICE u16x8 mc_ld16(const uint16_t* p) { return *reinterpret_cast<const u16x8*>(p); }
LIG_DEVICE u16x8 mc_ld8x2(const uint16_t* p, const uint16_t* q) {
  const u16x4 a = *reinterpret_cast<const u16x4*>(p), b = *reinterpret_cast<const u16x4*>(q);
  return u16x8{a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
}
