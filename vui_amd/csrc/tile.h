// The tiled operand layout and the matrix-core fragments that read it, for bf16 and fp32 elements.
//
// A matrix of R rows x K columns (K a multiple of BK, rows padded to 16) is cut into blocks of 16 rows x BK columns,
// block (r / 16, k / BK) at element offset ((r / 16) * (K / BK) + k / BK) * 16 * BK.  Inside a block lane
// (r % 16) + 16 * ((k % BK) / (BK / 4)) owns BK / 4 consecutive columns of one row, stored as pieces of 16 bytes:
// piece p of all 64 lanes is 1 KiB contiguous (lane l at byte 16 l).  A wave then fetches an operand fragment of a
// block with contiguous loads, where the row-major form makes the 16 lanes of a quarter-wave read 16 different lines -
// which the address unit serves at about a quarter of the rate (measured on this machine from an L2-sized buffer:
// 9.6 TB/s over the chip for 16 rows x 64 bytes per instruction, 31 TB/s for 1 KiB contiguous).  Which column a lane's
// element stands for is free as long as both operands of a product share the assignment.
#pragma once
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 tl_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float tl_f32x4;
// 16 bytes in flight: an array of HIP's uint4 structs that is filled and stored under conditions stays in scratch memory
typedef __attribute__((__vector_size__(4 * sizeof(uint32_t)))) uint32_t tl_u32x4;

template <typename T> struct Tl;
template <> struct Tl<bf16_t> {
  static constexpr int EP = 8;  // elements of a 16-byte piece
  static __device__ __forceinline__ tl_bf16x8 frag(const uint4& x) { return __builtin_bit_cast(tl_bf16x8, x); }
  // acc += A (16 x 32) B (32 x 16) for one piece of either operand
  static __device__ __forceinline__ tl_f32x4 mma(const uint4& a, const uint4& b, tl_f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(a), frag(b), acc, 0, 0, 0);
  }
  static __device__ __forceinline__ void st4(bf16_t* p, const float* v) {
    *reinterpret_cast<uint2*>(p) = make_uint2(f2bf2(v[0], v[1]), f2bf2(v[2], v[3]));
  }
  static __device__ __forceinline__ void st2(bf16_t* p, float a, float b) { *reinterpret_cast<uint32_t*>(p) = f2bf2(a, b); }
};
template <> struct Tl<float> {
  static constexpr int EP = 4;
  static __device__ __forceinline__ tl_f32x4 mma(const uint4& a, const uint4& b, tl_f32x4 acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.x), __uint_as_float(b.x), acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.y), __uint_as_float(b.y), acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.z), __uint_as_float(b.z), acc, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.w), __uint_as_float(b.w), acc, 0, 0, 0);
  }
  static __device__ __forceinline__ void st4(float* p, const float* v) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
  static __device__ __forceinline__ void st2(float* p, float a, float b) { *reinterpret_cast<float2*>(p) = make_float2(a, b); }
};

// element offset of (row r, column k) of a tiled matrix with K columns
template <typename T, int BK = 64>
__host__ __device__ __forceinline__ size_t tl_off(int r, int k, int K) {
  constexpr int EP = 16 / (int)sizeof(T), LC = BK / 4;  // columns per lane
  const int kb = k % BK, c = kb % LC;
  return ((size_t)(r >> 4) * (K / BK) + k / BK) * (16 * BK) + (size_t)((c / EP) * (64 * EP) + ((r & 15) + 16 * (kb / LC)) * EP + c % EP);
}
