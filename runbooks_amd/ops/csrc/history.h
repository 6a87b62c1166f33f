// Causal convolutions over the tokens of a ragged batch: where a tap reads.
//
// Tap j of `taps` at token t of a portion reads the input taps - 1 - j tokens
// earlier: a row of this batch, a row of the sequence's slot (its last taps - 1
// inputs, the oldest first), or, before the sequence's start, zero.
#pragma once

#include "common.h"

namespace rb {

struct Ragged {
  const int *positions, *cu_q, *slots, *seq_of;
  int taps;
};

struct Source {
  int first, pos0, slot;               // portion: row, position, slot
  // row of the batch (>= 0), ~(row of the slot) or INT_MIN for zero
  RB_DEV int at(int t, int j, int taps) const {
    const int s = t - (taps - 1 - j);
    if (s >= first) return s;
    const int back = first - s;                // 1 .. taps - 1
    return pos0 >= back ? ~(taps - 1 - back) : (int)0x80000000;
  }
};

RB_DEV Source source_of(const Ragged &b, int t) {
  const int seq = b.seq_of[t], first = b.cu_q[seq];
  return {first, b.positions[first], b.slots[seq]};
}

// V neighbouring values (V = 8 or 1) of E, as fp32
template <int V, typename E> RB_DEV void load_v(const E *p, float *f) {
  if constexpr (V == 8) {
    VIO<E>::load(p, f);
    if constexpr (VIO<E>::W == 4) VIO<E>::load(p + 4, f + 4);
  } else {
    f[0] = bf16_to_f32_or_id(*p);
  }
}
template <int V, typename E> RB_DEV void store_v(E *p, const float *f) {
  if constexpr (V == 8) {
    VIO<E>::store(p, f);
    if constexpr (VIO<E>::W == 4) VIO<E>::store(p + 4, f + 4);
  } else {
    store_scalar(p, f[0]);
  }
}

// decode-GEMM operand slot of column k
RB_DEV int64_t operand_slot(int k, int row) {
  return (int64_t)(k >> 4) * 512 + ((k >> 3) & 1) * 256 + row * 8 + (k & 7);
}

}  // namespace rb
