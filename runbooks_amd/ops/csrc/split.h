// MFMA products of fp32 factors that enter as two bf16 parts each, big and
// small: big big + big small + small big keeps all but 2^-16 of a factor.
//
// Operands of 16x16x32 products are 64 lanes x 16 bytes. Their summed index
// runs, in lane l, 4 (l / 16) + {0..3} and 16 + that, so that two stacked
// result tiles (register r of a lane: row 4 (l / 16) + r) are, packed, an
// operand.
#pragma once

#include "common.h"

namespace split {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(4))) float f32x4v;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4v;

union Frag { u32x4v u; bf16x8v v; };

RB_DEV unsigned pack2(float lo, float hi) {
  union { __bf16 b[2]; unsigned u; } c;
  c.b[0] = (__bf16)lo;
  c.b[1] = (__bf16)hi;
  return c.u;
}
// two floats as packed bf16 and the packed rest
RB_DEV void split2(float x, float y, unsigned &big, unsigned &small) {
  big = pack2(x, y);
  small = pack2(x - __uint_as_float(big << 16),
                y - __uint_as_float(big & 0xffff0000u));
}
RB_DEV void split8(const float *f, u32x4v &big, u32x4v &small) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    unsigned b, s;
    split2(f[2 * i], f[2 * i + 1], b, s);
    big[i] = b;
    small[i] = s;
  }
}

RB_DEV f32x4v mfma(const Frag &a, const Frag &b, f32x4v c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
// one of the three products that make an fp32 product of split factors
RB_DEV f32x4v part(int i, const Frag *a, const Frag &bh, const Frag &bl,
                   f32x4v c) {
  return mfma(a[i == 2], i == 1 ? bl : bh, c);
}

}  // namespace split
