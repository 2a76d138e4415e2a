// fp32 operands of bf16 MFMA as pairs (a value's rounding, and the rounding of what that leaves), for the chunked
// recurrences (retention_chunk.hip, mlstm_chunk.hip): hi hi + hi lo + lo hi, an error of about 2^-16 per operand.
#pragma once
#include "common.h"

// where row r of 64 lies when an accumulator of one product is the operand of the next
LSA_DEVICE int vidx(int r) { return (r & 32) | ((r & 12) << 1) | ((r & 16) >> 2) | (r & 3); }  // accumulator order

// two values rounded, f below g
LSA_DEVICE unsigned pack2(float f, float g) {
  typedef float f2_t __attribute__((ext_vector_type(2)));
  typedef __bf16 b2_t __attribute__((ext_vector_type(2)));
  return __builtin_bit_cast(unsigned, __builtin_convertvector((f2_t{f, g}), b2_t));
}
// two values -> their rounding and the rounding of what that leaves
LSA_DEVICE void split2(float f, float g, unsigned& h, unsigned& l) {
  h = pack2(f, g);
  l = pack2(f - __uint_as_float(h << 16), g - __uint_as_float(h & 0xffff0000u));
}
LSA_DEVICE void split8(const float* f, u32x4_t& h, u32x4_t& l) {
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    unsigned x, y;
    split2(f[2 * j], f[2 * j + 1], x, y);
    h[j] = x;
    l[j] = y;
  }
}
