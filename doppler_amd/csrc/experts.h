// Shared by the two files that serve mixtures of experts (experts.hip, dense_gemm.hip).
#pragma once
#include "dense_device.h"

namespace dh {

// Rows of an expert product.  GROUPED forms: rows sorted by expert, tiles of tile_rows rows.
struct ExpertRows {
  const int* tiles;        // [max_tiles][2]: expert (-1: no tile), first row inside its group; null: one group, rows as they are
  const int* group_off;    // [experts + 1] first row of every group
  const int* row_index;    // activation row of every sorted row, or null
  int64_t w_stride;        // elements between the experts' matrices
  int max_tiles, tile_rows;
  const float* row_in;     // factor of a row's input (gate and up before the clamps), or null
  const float* row_out;    // factor of a row's output, or null
  float limit;
};

// min(g, limit) sigmoid(1.702 min(g, limit)) (clamp(u, +-limit) + 1)
__device__ __forceinline__ float clamped_glu(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
}

// Row tiles of the grouped products for this many rows in all.
int expert_tile_rows(int a_dtype, int rows, int groups);
// act[row] = clamped_glu of a row's gate and up products with interleaved [N = 2 ff][K] weights (32 gate, 32 up rows, ..).
int experts_glu(const char* op, const ExpertRows& rows, const void* A, int a_dtype, int64_t lda, const uint16_t* W, int64_t ldw, int M,
                int N, int K, void* out, int out_dtype, int64_t ld_out);
// out[row] = W_expert act[row] for every sorted row, f32.
int experts_down(const char* op, const ExpertRows& rows, const void* A, int a_dtype, int64_t lda, const uint16_t* W, int64_t ldw, int N,
                 int K, float* out, int64_t ld_out);

}  // namespace dh
