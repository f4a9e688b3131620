// Device helpers of the dense (bf16-weight) kernels: element conversions, activations, lane reductions.
#pragma once
#include "dh_common.h"

namespace dh {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(8))) _Float16 f16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;
typedef __attribute__((ext_vector_type(16))) float f32x16_t;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4_t;

// A 32-bit word holds elements 2 i (low half) and 2 i + 1 (high half) of a bf16 row.
__device__ __forceinline__ float bf16_low(uint32_t w) { return __uint_as_float(w << 16); }
__device__ __forceinline__ float bf16_high(uint32_t w) { return __uint_as_float(w & 0xffff0000u); }
__device__ __forceinline__ float bf16_bits_to_f32(uint16_t b) { return __uint_as_float((uint32_t)b << 16); }
__device__ __forceinline__ uint16_t f32_to_bf16_bits(float v) {      // round to nearest even
  return __builtin_bit_cast(uint16_t, (__bf16)v);
}

// DH_ACT_* of one value (a plain activation, not a gated pair); DH_ACT_NONE passes it through.
__device__ __forceinline__ float activate(float z, int act) {
  if (act == DH_ACT_RELU2) {
    const float r = fmaxf(z, 0.f);
    return r * r;
  }
  if (act == DH_ACT_SILU) return z / (1.0f + __expf(-z));
  if (act == DH_ACT_GELU) return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  if (act == DH_ACT_GELU_ERF) return 0.5f * z * (1.0f + erff(0.7071067811865476f * z));
  return z;
}

// A lane's value combined over aligned groups of SPAN lanes (2, 4, .. 64); every lane of the group ends with the
// result.  Steps inside a 16-lane row are DPP modifiers (quad permutations, then mirrors, which cross the halves
// of a group whose halves are already uniform), the last two the gfx950 lane-swap instructions: no LDS traffic.
template <int CTRL>
__device__ __forceinline__ float dpp_lane(float v) {
  return __int_as_float(__builtin_amdgcn_update_dpp(__float_as_int(v), __float_as_int(v), CTRL, 0xF, 0xF, false));
}
struct AddOp {
  __device__ __forceinline__ float operator()(float a, float b) const { return a + b; }
};
struct MaxOp {
  __device__ __forceinline__ float operator()(float a, float b) const { return fmaxf(a, b); }
};
// FROM < 64, TO <= 64: the group of TO lanes from groups of FROM lanes that are uniform already.
template <int FROM, int TO, typename Op>
__device__ __forceinline__ float group_combine(float v, Op op) {
  if (FROM < 2 && TO >= 2) v = op(v, dpp_lane<0xB1>(v));        // quad_perm 1,0,3,2
  if (FROM < 4 && TO >= 4) v = op(v, dpp_lane<0x4E>(v));        // quad_perm 2,3,0,1
  if (FROM < 8 && TO >= 8) v = op(v, dpp_lane<0x141>(v));       // row_half_mirror
  if (FROM < 16 && TO >= 16) v = op(v, dpp_lane<0x140>(v));     // row_mirror
  if (FROM < 32 && TO >= 32) {
    auto s = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = op(__uint_as_float(s[0]), __uint_as_float(s[1]));
  }
  if (FROM < 64 && TO >= 64) {
    auto s = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = op(__uint_as_float(s[0]), __uint_as_float(s[1]));
  }
  return v;
}

// Workgroup index -> tile index such that each of the eight XCDs (which the hardware deals workgroups to in turn)
// gets a contiguous run of tiles and its L2 sees their shared operands.
__device__ __forceinline__ int xcd_contiguous(int id, int total) {
  const int xcd = id & 7, within = id >> 3, q = total >> 3, r = total & 7;
  return xcd * q + (xcd < r ? xcd : r) + within;
}

}  // namespace dh
