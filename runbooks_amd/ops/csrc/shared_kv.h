// Attention over paged rows that hold a token's key and value at once: what
// the kernels share.
//
// A row has `ec` columns. The key is its first `hc`, the value `vc` from
// column `voff` on. Where a token's unrotated key doubles as its value, the
// two overlap,
//
//   [ rotated | not rotated | rotated dimensions before rotation ]   (ec)
//     \------- key (hc) -----/
//               \------------------ value (vc = hc) ------------/
//
// so the value's columns come in another order than the key's; the output
// projection's weight has its columns in the value's order. Otherwise the
// value follows the key. The cache is [blocks, kv heads, PAGE, ec]: a page of
// one head is contiguous.
//
// With two maps a row is [ key 1 | key 2 | value ], and a head has a query for
// each key; its result is rms_norm(o1 - lam o2) times out_scale.
#pragma once

#include "common.h"

namespace skv {

constexpr int PAGE = 16;               // tokens per cache block

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8v;
typedef __attribute__((ext_vector_type(4))) float f32x4v;
typedef __attribute__((ext_vector_type(16))) float f32x16v;
typedef __attribute__((ext_vector_type(4))) unsigned int u32x4v;

// Query rows are (token, head of the group) pairs, heads fastest.
struct Args {
  const void *y;                       // [T, ny]; q heads first
  int64_t ny;
  const void *cache;
  const int *tables, *cu_q, *seq_lens;
  int table_width, heads, kv, group, hc, vc, voff, ec, nsplit, total_rows;
  int window;                          // keys a query sees (0: all)
  int chunk;                           // or: keys of its own chunk (0: all)
  const int *positions;                // [T], absolute; with chunks
  const float *sink;                   // [heads], a further score, or null
  float scale;                         // MFMA kernels: times log2(e)
  float out_scale;                     // factor on the result
  void *z;                             // [T, nz]; heads first
  int64_t nz;
  uint16_t *swz;                       // decode operand of z, or null
  float *part_o;                       // [nsplit, T*H, vc], or null
  float *part_ml;                      // [nsplit, T*H, 2]
  const float *lam;                    // two maps
  int count;                           // columns that their norm counts
  float eps;
  bool f32;                            // z's type
};

// First key that a query at retained position `pos` sees, possibly below 0;
// `dropped`: the absolute position of retained position 0.
RB_DEV int first_key(const Args &a, int pos, int dropped) {
  if (a.chunk > 0) {
    const int p = pos + dropped;
    return p - p % a.chunk - dropped;
  }
  return a.window > 0 ? pos - a.window + 1 : 0;
}
RB_DEV int dropped_of(const Args &a, int q0, int v0) {
  return a.chunk > 0 ? a.positions[q0] - v0 : 0;
}

// LDS bytes between two cached rows: an odd number of 16-byte chunks
RB_DEV __host__ constexpr int row_stride(int ec) {
  return ec * 2 + (ec / 8 % 2 ? 0 : 16);
}

// A page of one kv head from memory to LDS through registers: lane l moves
// the 16-byte chunks l, l + 64, ... (the last one is repeated).
template <int NI> struct PageCopy {
  int src[NI], dst[NI];
  RB_DEV PageCopy(int lane, int ec) {
    const int per_row = ec / 8;
    const unsigned inv = ((1u << 20) + per_row - 1) / per_row;
#pragma unroll
    for (int i = 0; i < NI; ++i) {
      const int c = min(lane + i * 64, PAGE * per_row - 1);
      const int key = (int)((c * inv) >> 20);
      src[i] = c * 8;
      dst[i] = key * row_stride(ec) + (c - key * per_row) * 16;
    }
  }
  RB_DEV void load(u32x4v *reg, const uint16_t *page) const {
#pragma unroll
    for (int i = 0; i < NI; ++i)
      reg[i] = *reinterpret_cast<const u32x4v *>(page + src[i]);
  }
  RB_DEV void store(char *lds, const u32x4v *reg) const {
#pragma unroll
    for (int i = 0; i < NI; ++i)
      *reinterpret_cast<u32x4v *>(lds + dst[i]) = reg[i];
  }
};

// decode-GEMM operand slot of 8 columns from k (k % 8 == 0)
RB_DEV int64_t operand_at(int k, int row) {
  return (int64_t)(k >> 4) * 512 + ((k >> 3) & 1) * 256 + row * 8;
}

// four values of row `t` from column `col` (col % 4 == 0) of z
RB_DEV void store4(const Args &a, int64_t t, int col, const float *v) {
  uint2 w;
  w.x = rb::pack_bf16x2(v[0], v[1]);
  w.y = rb::pack_bf16x2(v[2], v[3]);
  *reinterpret_cast<uint2 *>((uint16_t *)a.z + t * a.nz + col) = w;
  if (a.swz != nullptr)
    *reinterpret_cast<uint2 *>(a.swz + operand_at(col & ~7, (int)t) +
                               (col & 7)) = w;
}

// Sizes that a kernel is made for: HCK columns of a key, HCP of a value (and a
// key), NI chunks that a lane copies per page.
template <int K, int P, int N, int M> struct Sizes {
  static constexpr int HCK = K, HCP = P, NI = N, MAPS = M;
};

template <typename F> void pick_head(int hc, F go) {
  if (hc <= 32) go(std::integral_constant<int, 32>{});
  else if (hc <= 64) go(std::integral_constant<int, 64>{});
  else if (hc <= 96) go(std::integral_constant<int, 96>{});
  else if (hc <= 128) go(std::integral_constant<int, 128>{});
  else if (hc <= 192) go(std::integral_constant<int, 192>{});
  else go(std::integral_constant<int, 256>{});
}

// Calls f with the sizes for keys of hc columns, values (or keys) of up to
// `hc`, rows of ec.
template <typename F> void pick_sizes(int hc, int ec, F f) {
  const int ni = (ec + 31) / 32;
  auto go = [&](auto hcp) {
    constexpr int H = decltype(hcp)::value;
    constexpr int few = H / 32 + (H < 128 ? 1 : H / 128);
    constexpr int most = H / 16;
    if (ni <= few) f(Sizes<H, H, few, 1>{});
    else f(Sizes<H, H, most, 1>{});
  };
  pick_head(hc, go);
}
// the same for two maps with keys of hc columns, values of vc
template <typename F> void pick_sizes2(int hc, int vc, F f) {
  const int ni = (2 * hc + vc + 31) / 32;
  auto go = [&](auto hcp) {
    constexpr int H = decltype(hcp)::value;
    auto width = [&](auto k) {
      constexpr int K = decltype(k)::value;
      if constexpr (K < H) f(Sizes<K, H, (2 * K + H + 31) / 32, 2>{});
      else if (ni <= H / 16) f(Sizes<K, H, H / 16, 2>{});
      else f(Sizes<K, H, 3 * H / 32, 2>{});
    };
    if (hc <= H / 2) width(std::integral_constant<int, H / 2>{});
    else width(hcp);
  };
  pick_head(hc > vc ? hc : vc, go);
}

}  // namespace skv
