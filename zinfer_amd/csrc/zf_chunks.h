// What the recurrences that run a prompt in chunks of 128 tokens share: the chunk's MFMA on
// bfloat16 operands with 32-bit sums, 32-bit numbers as the sum of two bfloat16 numbers, and where
// the elements of a chunk's tiles lie in LDS.
#pragma once
#include "zf_common.h"

#define FC_C 128                 // tokens of a chunk

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 fc_bf16x8_t;
typedef __attribute__((__vector_size__(16 * sizeof(float)))) float fc_f32x16_t;
typedef __attribute__((__vector_size__(4 * sizeof(uint32_t)))) uint32_t fc_u32x4_t;

__device__ __forceinline__ float fc_pow(float log2g, int n) {
  return __builtin_amdgcn_exp2f(log2g * (float)n);
}
// two floats as bfloat16 numbers in one register (`a` in the low half), and what that leaves
__device__ __forceinline__ uint32_t fc_pack(float a, float b, uint32_t& lo) {
  const uint32_t hi = pack_bf16x2(a, b);
  lo = pack_bf16x2(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
  return hi;
}
__device__ __forceinline__ fc_f32x16_t fc_mfma(const fc_u32x4_t& a, const fc_u32x4_t& b,
                                               const fc_f32x16_t& c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(*(const fc_bf16x8_t*)&a, *(const fc_bf16x8_t*)&b,
                                                 c, 0, 0, 0);
}

// Where the pair of tokens (2 tp, 2 tp + 1) of row c lies in a [rows][FC_C tokens] tile, in
// registers: groups of 8 tokens stay together, and are permuted by the row so that neither rows
// side by side (an MFMA operand's reads) nor every 8th row (the transposing stores) meet in a bank.
__device__ __forceinline__ int fc_tr(int c, int tp) {
  return c * (FC_C / 2) + (((tp >> 2) ^ (((c >> 3) ^ c) & 15)) << 2) + (tp & 3);
}
// Where the group of 8 elements number g of row r lies in a [rows][KD] tile, in bfloat16 numbers.
template <int KD> __device__ __forceinline__ int fc_row(int r, int g) {
  constexpr int NG = KD / 8;
  constexpr int SH = KD == 32 ? 2 : (KD == 64 ? 1 : 0);
  return (r * NG + (g ^ ((r >> SH) & (NG - 1)))) * 8;
}
