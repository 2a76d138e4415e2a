// fp32 operands of bf16 MFMA as pairs (a value's rounding, and the rounding of what that leaves), for the chunked
// recurrences (retention_chunk.hip, mlstm_chunk.hip): hi hi + hi lo + lo hi, an error of about 2^-16 per operand.
#pragma once
#include "common.h"

// where row r of 64 lies when an accumulator of one product is the operand of the next
LSA_DEVICE int vidx(int r) { return (r & 32) | ((r & 12) << 1) | ((r & 16) >> 2) | (r & 3); }  // accumulator order

// 8 values -> their rounding and the rounding of what that leaves
LSA_DEVICE void split8(const float* f, u32x4_t& h, u32x4_t& l) {
  float r[8], t[8];
  h = pack8(f);
  unpack8(h, r);
#pragma unroll
  for (int j = 0; j < 8; ++j) t[j] = f[j] - r[j];
  l = pack8(t);
}
// two values, one above the other
LSA_DEVICE void split2(float f, float g, unsigned& h, unsigned& l) {
  h = (unsigned)f2bf(f) | ((unsigned)f2bf(g) << 16);
  l = (unsigned)f2bf(f - __uint_as_float(h << 16)) | ((unsigned)f2bf(g - __uint_as_float(h & 0xffff0000u)) << 16);
}
