// What the attention kernels on the matrix units share: operand types, sums and maxima over the
// lanes that hold one row, division by the page size.
#pragma once

#include "common.h"

namespace shk {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

union AFrag {
  uint4 u;
  bf16x8 v;
  uint16_t h[8];
};

// Maximum and sum over the four lanes j, j + 16, j + 32, j + 48 (one query's scores in
// the transposed products), in every one of them.  Two swaps of the vector unit (gfx950's
// v_permlane16_swap / v_permlane32_swap) instead of two trips through the LDS crossbar,
// which the chunk's chain of dependent steps would wait for: with rows of 16 lanes r0 r1
// r2 r3, the first swap of v with itself gives (r0 r0 r2 r2) and (r1 r1 r3 r3), the
// second, of what they combine to, (a a a a) and (b b b b).  Everything here is written
// so that the compiler sees it: an instruction in asm would hide from it what the
// swaps' operands have to wait for.
__device__ __forceinline__ float bits_as_float(unsigned v) { return __builtin_bit_cast(float, v); }
__device__ __forceinline__ float lanes4_max(float v) {
  const unsigned b = __builtin_bit_cast(unsigned, v);
  const auto rows = __builtin_amdgcn_permlane16_swap(b, b, false, false);
  const unsigned h = __builtin_bit_cast(unsigned, fmaxf(bits_as_float(rows[0]), bits_as_float(rows[1])));
  const auto halves = __builtin_amdgcn_permlane32_swap(h, h, false, false);
  return fmaxf(bits_as_float(halves[0]), bits_as_float(halves[1]));
}
__device__ __forceinline__ float lanes4_sum(float v) {
  const unsigned b = __builtin_bit_cast(unsigned, v);
  const auto rows = __builtin_amdgcn_permlane16_swap(b, b, false, false);
  const unsigned h = __builtin_bit_cast(unsigned, bits_as_float(rows[0]) + bits_as_float(rows[1]));
  const auto halves = __builtin_amdgcn_permlane32_swap(h, h, false, false);
  return bits_as_float(halves[0]) + bits_as_float(halves[1]);
}

// max(a, b, c) in one instruction.  Written out because fmaxf() first quiets each
// operand that might be a signalling NaN (one more instruction per operand), which
// scores, being products or -inf, never are.  The operands must come from vector
// instructions, never straight from a matrix instruction: the compiler does not
// count the wait states that a matrix result needs for an instruction it cannot
// see into (scores scaled inside the exponent, and so fed unscaled from the
// matrix unit into this, came out wrong).
__device__ __forceinline__ float max3(float a, float b, float c) {
  float r;
  asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(a), "v"(b), "v"(c));
  return r;
}

template <bool V>
struct EdgeTag {
  static constexpr bool value = V;
};

// x / page_size and x % page_size without a division: magic = ceil(2^32 / page_size)
// makes the high half of x * magic the quotient for 0 <= x < 2^32 / page_size.
struct PageDiv {
  int ps;
  uint32_t magic;
  __device__ __forceinline__ int div(int x) const {
    return static_cast<int>(__umulhi(static_cast<uint32_t>(x), magic));
  }
  __device__ __forceinline__ int mod(int x) const { return x - div(x) * ps; }
};

}  // namespace shk
