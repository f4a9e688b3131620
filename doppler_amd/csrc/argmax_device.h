// Argmax candidates and streaming weight loads shared by the output heads (lmhead.hip, dense_gemv.hip).
#pragma once
#include "dh_common.h"

namespace dh {

constexpr int kMaxParts = 2048;    // per-workgroup candidates a head leaves for the final reduction

// Folds `parts` candidates (one workgroup) and writes the token; ties go to the lowest index (lmhead.hip).
int launch_argmax_final(const char* op, const float* part_val, const uint32_t* part_idx, int parts, uint32_t* token_out,
                        int out_index);

struct Cand {
  float v;
  uint32_t i;
};

__device__ __forceinline__ bool beats(float cv, uint32_t ci, float bv, uint32_t bi) {
  if (cv > bv) return true;
  if (cv < bv) return false;
  return ci < bi;
}

__device__ __forceinline__ Cand wave_best(Cand c) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ov = __shfl_xor(c.v, off, 64);
    const uint32_t oi = __shfl_xor(c.i, off, 64);
    if (beats(ov, oi, c.v, c.i)) { c.v = ov; c.i = oi; }
  }
  return c;
}

// Workgroup-wide best of 256 threads; valid in thread 0.
__device__ __forceinline__ Cand block_best_256(Cand c, float* sv, uint32_t* si) {
  c = wave_best(c);
  const int wave = threadIdx.x >> 6;
  if ((threadIdx.x & 63) == 0) { sv[wave] = c.v; si[wave] = c.i; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < 4; w++)
      if (beats(sv[w], si[w], c.v, c.i)) { c.v = sv[w]; c.i = si[w]; }
  }
  return c;
}

// 16 bytes of a weight row, marked non-temporal.  Every row is read once per call, by one wave, as whole
// cache lines (a wave's load covers 1 KB of consecutive bytes): with the streaming hint the [151936 x 4096]
// f16 head is read at 6.6 TB/s against 5.9 TB/s with ordinary loads.  (The same hint on loads whose cache
// lines are shared between waves, the Q4_K units' 144-byte row pieces and the decode attention's K/V rows,
// made those kernels slower.)
__device__ __forceinline__ uint4 stream_load_16(const uint4* p) {
  typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
  const u32x4 t = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p));
  return make_uint4(t[0], t[1], t[2], t[3]);
}

}  // namespace dh
