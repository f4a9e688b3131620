// Matrix products with dense bf16 weights for several activation rows (prefill).
//
//   bf16 activations   v_mfma_f32_32x32x16_bf16, f32 accumulation
//   f16 activations    the same with f16 weights, v_mfma_f32_32x32x16_f16 (products of rows an f16 cache holds)
//   f32 activations    v_mfma_f32_32x32x2_f32 on the weights widened (exactly) to f32: a true 32-bit product
//
// Weights [N][ldw] and activations [M][lda] are both read along k, 64 elements (bf16) or 32 (f32) at a time; K is
// a multiple of 64, which the owner of the buffers reaches with zero padding.  A tile of each goes through
// registers into one of two LDS buffers (loads for the next tile are in flight while the current one is
// multiplied; one barrier per tile).  LDS rows hold their 16-byte pieces at slot (piece ^ row) & 7, so that both
// the row-wise stores and the column-wise fragment reads touch every bank once.
//
// The epilogue serves two outputs, because the projections that read one normalised row are stored as one
// stacked matrix: columns below n_first are (alpha * acc + bias) * column scale (+ residual) in f32, columns from n_first
// on are act(alpha * acc), written in the operand type of the product that reads them.
//
// Experts (dh_experts_*): the GROUPED forms take rows that are sorted by expert.  A table of row tiles names every tile's
// expert and first row; a tile gathers its activation rows by index, multiplies them by its own expert's weights and
// leaves when the table has ended.  The GLU forms read matrices whose gate and up rows alternate in blocks of 32, so
// that a wave's two neighbouring accumulator tiles hold the gate and the up value of the same column in the same lane;
// the epilogue clamps, gates and multiplies them and writes one column per pair.
//
// A grid of too few tiles for the device cuts k into slices instead (grid.y): every slice leaves its raw sums in the
// library's split-K workspace and a second launch adds them in slice order and runs the epilogue.
#include <algorithm>

#include "dense_device.h"
#include "experts.h"

namespace {

using dh::bf16x8_t;
using dh::f16x8_t;
using dh::f32x16_t;
using dh::f32x4_t;
using dh::u32x4_t;

struct GemmArgs {
  const void* A;          // [M][lda], bf16 or f32
  const uint16_t* W;      // [N][ldw] bf16
  int64_t lda, ldw;
  int M, N, K;
  float alpha;
  const float* bias;      // [n_first] or null
  const float* residual;  // [M][ldc] or null (may be C)
  const float* col_scale; // [n_first] or null
  float* C;
  int64_t ldc;
  int n_first;
  void* C2;               // [M][ldc2]
  int64_t ldc2;
  int c2_dtype, act;
  int tiles_m, tiles_n;
  float* parts;           // [slices][M][N] raw sums instead of the outputs, or null
  int k_slice;            // k extent of a slice (a multiple of 64); K when there is one
  dh::ExpertRows rows;    // GROUPED and GLU forms
};

// Second outputs a kernel is compiled for: none, one activation, or whatever the arguments say.
constexpr int kNoSecond = -2, kAnyAct = -3;

__device__ __forceinline__ void put_c2(const GemmArgs& a, int64_t at, float v) {
  if (a.c2_dtype == DH_BF16) static_cast<uint16_t*>(a.C2)[at] = dh::f32_to_bf16_bits(v);
  else if (a.c2_dtype == DH_F16) static_cast<_Float16*>(a.C2)[at] = (_Float16)v;
  else static_cast<float*>(a.C2)[at] = v;
}

// The two outputs of one element.
__device__ __forceinline__ void put(const GemmArgs& a, int m, int n, float acc) {
  if (n < a.n_first) {
    const int64_t at = (int64_t)m * a.ldc + n;
    float v = fmaf(acc, a.alpha, a.bias ? a.bias[n] : 0.f);
    if (a.col_scale) v *= a.col_scale[n];
    if (a.residual) v += a.residual[at];
    a.C[at] = v;
  } else {
    put_c2(a, (int64_t)m * a.ldc2 + (n - a.n_first), dh::activate(acc * a.alpha, a.act));
  }
}

// Where a workgroup's tile lies: its rows (base + 0 .. rows - 1 of the outputs), its first row among them, its weights.
struct TilePlace {
  int base, rows, m0;
  const uint16_t* W;
};
template <bool GROUPED>
__device__ __forceinline__ bool place_tile(const GemmArgs& a, int m_tile, int bm, TilePlace* p) {
  p->base = 0; p->rows = a.M; p->m0 = m_tile * bm; p->W = a.W;
  if (GROUPED) {
    const int g = a.rows.tiles[2 * m_tile];
    if (g < 0) return false;
    p->m0 = a.rows.tiles[2 * m_tile + 1];
    p->base = a.rows.group_off[g];
    p->rows = a.rows.group_off[g + 1] - p->base;
    p->W += (int64_t)g * a.rows.w_stride;
  }
  return true;
}
// The activation row behind a tile's row (rows past the group repeat its last one: their products are never stored).
template <bool GROUPED>
__device__ __forceinline__ int64_t source_row(const GemmArgs& a, const TilePlace& p, int row) {
  const int r = p.base + min(p.m0 + row, p.rows - 1);
  return GROUPED && a.rows.row_index ? a.rows.row_index[r] : r;
}

// One 32 x 32 accumulator tile: lane l holds column l & 31 and rows 8 (i / 4) + 4 (l >> 5) + i % 4.
template <int ACT>
__device__ __forceinline__ void store_tile(const GemmArgs& a, const TilePlace& p, const f32x16_t& acc, int m0, int n0, int lane) {
  const int n = n0 + (lane & 31);
  if (n >= a.N) return;
  const int mb = m0 + 4 * (lane >> 5);
  if (a.parts) {
    float* q = a.parts + (int64_t)blockIdx.y * a.M * a.N;
#pragma unroll
    for (int i = 0; i < 16; i++) {
      const int m = mb + 8 * (i >> 2) + (i & 3);
      if (m < a.M) q[(int64_t)m * a.N + n] = acc[i];
    }
    return;
  }
  if (ACT == kNoSecond || n < a.n_first) {
    const float scale = a.col_scale ? a.col_scale[n] : 1.f, bias = (a.bias ? a.bias[n] : 0.f) * scale, alpha = a.alpha * scale;
    float* c = a.C + (int64_t)p.base * a.ldc + n;
    if (a.residual) {
      // every read in front of the first write: the residual may be the output itself
      const float* res = a.residual + (int64_t)p.base * a.ldc + n;
      float r[16];
#pragma unroll
      for (int i = 0; i < 16; i++) r[i] = res[(int64_t)min(mb + 8 * (i >> 2) + (i & 3), p.rows - 1) * a.ldc];
#pragma unroll
      for (int i = 0; i < 16; i++) {
        const int m = mb + 8 * (i >> 2) + (i & 3);
        if (m < p.rows) c[(int64_t)m * a.ldc] = fmaf(acc[i], alpha, bias) + r[i];
      }
    } else {
#pragma unroll
      for (int i = 0; i < 16; i++) {
        const int m = mb + 8 * (i >> 2) + (i & 3);
        if (m < p.rows) c[(int64_t)m * a.ldc] = fmaf(acc[i], alpha, bias);
      }
    }
  } else {
    const int64_t at = (int64_t)p.base * a.ldc2 + (n - a.n_first);
    const int act = ACT == kAnyAct ? a.act : ACT;
#pragma unroll
    for (int i = 0; i < 16; i++) {
      const int m = mb + 8 * (i >> 2) + (i & 3);
      if (m < p.rows) put_c2(a, at + (int64_t)m * a.ldc2, dh::activate(acc[i] * a.alpha, act));
    }
  }
}
// The same for a gate tile and the up tile beside it (first weight row n0 of the gate block).
__device__ __forceinline__ void store_glu(const GemmArgs& a, const TilePlace& p, const f32x16_t& gate, const f32x16_t& up, int m0, int n0,
                                          int lane) {
  if (n0 >= a.N) return;
  const int col = (n0 >> 1) + (lane & 31), mb = m0 + 4 * (lane >> 5);
#pragma unroll
  for (int i = 0; i < 16; i++) {
    const int m = mb + 8 * (i >> 2) + (i & 3);
    if (m >= p.rows) continue;
    const int64_t r = p.base + m;
    const float w = a.rows.row_in ? a.rows.row_in[r] : 1.f;
    float y = dh::clamped_glu(w * gate[i], w * up[i], a.rows.limit);
    if (a.rows.row_out) y *= a.rows.row_out[r];
    put_c2(a, r * a.ldc2 + col, y);
  }
}

// WM x WN waves; a wave computes TM x TN accumulator tiles of 32 x 32.
template <int WM, int WN, int TM, int TN, bool F16, int ACT, bool GROUPED = false, bool GLU = false>
__global__ __launch_bounds__(64 * WM * WN, TM * TN >= 4 ? 2 : TM * TN == 2 ? 3 : 4) void gemm_16bit_kernel(const GemmArgs a) {
  static_assert(!GLU || TN == 2, "a wave's two tiles are the gate and the up value");
  constexpr int BM = 32 * WM * TM, BN = 32 * WN * TN, THREADS = 64 * WM * WN;
  constexpr int PA = BM * 8 / THREADS, PB = BN * 8 / THREADS;      // 16-byte pieces per thread and tile
  static_assert(BM * 8 % THREADS == 0 && BN * 8 % THREADS == 0, "whole pieces per thread");
  __shared__ __align__(16) u32x4_t lds[2][(BM + BN) * 8];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int wm = wave / WN, wn = wave % WN;
  const int tile = dh::xcd_contiguous(blockIdx.x, a.tiles_m * a.tiles_n);
  TilePlace place;
  if (!place_tile<GROUPED>(a, tile % a.tiles_m, BM, &place)) return;
  const int m0 = place.m0, n0 = (tile / a.tiles_m) * BN;

  // this thread's pieces: rows past the matrix repeat its last row (their products are never stored)
  const uint16_t* pa[PA];
  const uint16_t* pb[PB];
  int sa[PA], sb[PB];
#pragma unroll
  for (int r = 0; r < PA; r++) {
    const int p = tid + THREADS * r, row = p >> 3, c = p & 7;
    pa[r] = static_cast<const uint16_t*>(a.A) + source_row<GROUPED>(a, place, row) * a.lda + 8 * c;
    sa[r] = row * 8 + (c ^ (row & 7));
  }
#pragma unroll
  for (int r = 0; r < PB; r++) {
    const int p = tid + THREADS * r, row = p >> 3, c = p & 7;
    pb[r] = place.W + (int64_t)min(n0 + row, a.N - 1) * a.ldw + 8 * c;
    sb[r] = BM * 8 + row * 8 + (c ^ (row & 7));
  }
  u32x4_t ra[PA], rb[PB];
#define DH_GEMM_LOAD(kt_)                                                                                              \
  do {                                                                                                                 \
    _Pragma("unroll") for (int r = 0; r < PA; r++) ra[r] = *reinterpret_cast<const u32x4_t*>(pa[r] + 64 * (kt_));      \
    _Pragma("unroll") for (int r = 0; r < PB; r++) rb[r] = *reinterpret_cast<const u32x4_t*>(pb[r] + 64 * (kt_));      \
  } while (0)
#define DH_GEMM_STORE(b_)                                                                                              \
  do {                                                                                                                 \
    _Pragma("unroll") for (int r = 0; r < PA; r++) lds[b_][sa[r]] = ra[r];                                             \
    _Pragma("unroll") for (int r = 0; r < PB; r++) lds[b_][sb[r]] = rb[r];                                             \
  } while (0)

  f32x16_t acc[TM][TN];
#pragma unroll
  for (int i = 0; i < TM; i++)
#pragma unroll
    for (int j = 0; j < TN; j++)
#pragma unroll
      for (int e = 0; e < 16; e++) acc[i][j][e] = 0.f;

  const int k0 = blockIdx.y * a.k_slice;
  const int nk = min(a.k_slice, a.K - k0) >> 6;
#pragma unroll
  for (int r = 0; r < PA; r++) pa[r] += k0;
#pragma unroll
  for (int r = 0; r < PB; r++) pb[r] += k0;
  DH_GEMM_LOAD(0);
  DH_GEMM_STORE(0);
  __syncthreads();
  const int frow = lane & 31, fk = lane >> 5;
  for (int kt = 0; kt < nk; kt++) {
    const int buf = kt & 1;
    if (kt + 1 < nk) DH_GEMM_LOAD(kt + 1);
#pragma unroll
    for (int ks = 0; ks < 4; ks++) {
      u32x4_t fa[TM], fb[TN];
      const int piece = 2 * ks + fk;
#pragma unroll
      for (int i = 0; i < TM; i++) {
        const int row = 32 * (wm * TM + i) + frow;
        fa[i] = lds[buf][row * 8 + (piece ^ (row & 7))];
      }
#pragma unroll
      for (int j = 0; j < TN; j++) {
        const int row = 32 * (wn * TN + j) + frow;
        fb[j] = lds[buf][BM * 8 + row * 8 + (piece ^ (row & 7))];
      }
#pragma unroll
      for (int i = 0; i < TM; i++)
#pragma unroll
        for (int j = 0; j < TN; j++) {
          if constexpr (F16)
            acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(f16x8_t, fa[i]), __builtin_bit_cast(f16x8_t, fb[j]), acc[i][j], 0, 0, 0);
          else
            acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_t, fa[i]), __builtin_bit_cast(bf16x8_t, fb[j]), acc[i][j], 0, 0, 0);
        }
    }
    if (kt + 1 < nk) DH_GEMM_STORE(buf ^ 1);
    __syncthreads();
  }
#undef DH_GEMM_LOAD
#undef DH_GEMM_STORE
#pragma unroll
  for (int i = 0; i < TM; i++) {
    if constexpr (GLU) {
      store_glu(a, place, acc[i][0], acc[i][1], m0 + 32 * (wm * TM + i), n0 + 32 * wn * TN, lane);
    } else {
#pragma unroll
      for (int j = 0; j < TN; j++) store_tile<ACT>(a, place, acc[i][j], m0 + 32 * (wm * TM + i), n0 + 32 * (wn * TN + j), lane);
    }
  }
}

// The 32-bit product: four waves, a 64 x 64 TN tile, 32 k at a time.  Both tiles sit in LDS as f32 rows of 32 + 4
// words; a lane reads four consecutive k of its row and feeds four instructions with them (k-slot l >> 5 of
// instruction e stands for k = 8 s + 4 (l >> 5) + e on both sides).
template <int TN, bool GROUPED, bool GLU>
__global__ __launch_bounds__(256) void gemm_f32_kernel(const GemmArgs a) {
  static_assert(!GLU || TN == 2, "a wave's two tiles are the gate and the up value");
  constexpr int BM = 64, BN = 64 * TN, BK = 32, ROW = BK + 4;
  __shared__ __align__(16) float la[BM * ROW];
  __shared__ __align__(16) float lb[BN * ROW];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int wm = wave >> 1, wn = wave & 1;
  const int tile = dh::xcd_contiguous(blockIdx.x, a.tiles_m * a.tiles_n);
  TilePlace place;
  if (!place_tile<GROUPED>(a, tile % a.tiles_m, BM, &place)) return;
  const int m0 = place.m0, n0 = (tile / a.tiles_m) * BN;
  // A: 64 rows x 8 pieces of 4 floats, two per thread; W: 64 TN rows x 4 pieces of 8 elements, TN per thread
  const float* pa[2];
  const uint16_t* pb[TN];
#pragma unroll
  for (int r = 0; r < 2; r++) {
    const int p = tid + 256 * r;
    pa[r] = static_cast<const float*>(a.A) + source_row<GROUPED>(a, place, p >> 3) * a.lda + 4 * (p & 7);
  }
#pragma unroll
  for (int r = 0; r < TN; r++) pb[r] = place.W + (int64_t)min(n0 + 64 * r + (tid >> 2), a.N - 1) * a.ldw + 8 * (tid & 3);
  f32x4_t ra[2];
  u32x4_t rb[TN];
  f32x16_t acc[TN];
#pragma unroll
  for (int j = 0; j < TN; j++)
#pragma unroll
    for (int e = 0; e < 16; e++) acc[j][e] = 0.f;
  const int nk = a.K / BK;
#pragma unroll
  for (int r = 0; r < 2; r++) ra[r] = *reinterpret_cast<const f32x4_t*>(pa[r]);
#pragma unroll
  for (int r = 0; r < TN; r++) rb[r] = *reinterpret_cast<const u32x4_t*>(pb[r]);
  for (int kt = 0; kt < nk; kt++) {
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 2; r++) {
      const int p = tid + 256 * r;
      *reinterpret_cast<f32x4_t*>(&la[(p >> 3) * ROW + 4 * (p & 7)]) = ra[r];
    }
#pragma unroll
    for (int r = 0; r < TN; r++) {
      float* wb = &lb[(64 * r + (tid >> 2)) * ROW + 8 * (tid & 3)];
#pragma unroll
      for (int e = 0; e < 4; e++) {
        wb[2 * e] = dh::bf16_low(rb[r][e]);
        wb[2 * e + 1] = dh::bf16_high(rb[r][e]);
      }
    }
    __syncthreads();
    if (kt + 1 < nk) {
#pragma unroll
      for (int r = 0; r < 2; r++) ra[r] = *reinterpret_cast<const f32x4_t*>(pa[r] + BK * (kt + 1));
#pragma unroll
      for (int r = 0; r < TN; r++) rb[r] = *reinterpret_cast<const u32x4_t*>(pb[r] + BK * (kt + 1));
    }
#pragma unroll
    for (int s = 0; s < BK / 8; s++) {
      const int k = 8 * s + 4 * (lane >> 5);
      const f32x4_t fa = *reinterpret_cast<const f32x4_t*>(&la[(32 * wm + (lane & 31)) * ROW + k]);
#pragma unroll
      for (int j = 0; j < TN; j++) {
        const f32x4_t fb = *reinterpret_cast<const f32x4_t*>(&lb[(32 * (wn * TN + j) + (lane & 31)) * ROW + k]);
#pragma unroll
        for (int e = 0; e < 4; e++) acc[j] = __builtin_amdgcn_mfma_f32_32x32x2f32(fa[e], fb[e], acc[j], 0, 0, 0);
      }
    }
  }
  if constexpr (GLU) {
    store_glu(a, place, acc[0], acc[1], m0 + 32 * wm, n0 + 32 * wn * TN, lane);
  } else {
#pragma unroll
    for (int j = 0; j < TN; j++) store_tile<kAnyAct>(a, place, acc[j], m0 + 32 * wm, n0 + 32 * (wn * TN + j), lane);
  }
}

__global__ __launch_bounds__(256) void gemm_reduce_kernel(const GemmArgs a, int slices) {
  const int64_t total = (int64_t)a.M * a.N;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
    float s = 0.f;
#pragma unroll 4
    for (int k = 0; k < slices; k++) s += a.parts[k * total + i];
    put(a, (int)(i / a.N), (int)(i % a.N), s);
  }
}

template <int WM, int WN, int TM, int TN, bool F16, int ACT>
int launch_16bit(const char* op, GemmArgs a, int slices) {
  a.tiles_m = (int)dh::ceil_div(a.M, 32 * WM * TM);
  a.tiles_n = (int)dh::ceil_div(a.N, 32 * WN * TN);
  a.k_slice = a.K;
  if (slices > 1) {
    a.k_slice = (int)dh::ceil_div(a.K / 64, slices) * 64;
    slices = (int)dh::ceil_div(a.K, a.k_slice);
    size_t bytes = 0;
    a.parts = dh::splitk_workspace(&bytes);
  }
  hipLaunchKernelGGL((gemm_16bit_kernel<WM, WN, TM, TN, F16, ACT>), dim3(a.tiles_m * a.tiles_n, slices), dim3(64 * WM * WN), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  if (a.parts) {
    const unsigned grid = (unsigned)std::min<int64_t>(dh::ceil_div((int64_t)a.M * a.N, 256), 4096);
    hipLaunchKernelGGL(gemm_reduce_kernel, dim3(grid), dim3(256), 0, dh::stream(), a, slices);
    DH_CHECK_LAUNCH(op);
  }
  return 0;
}

template <int WM, int WN, int TM, int TN>
int launch_tile(const char* op, const GemmArgs& a, bool f16, int slices) {
  if (f16) return a.n_first == a.N ? launch_16bit<WM, WN, TM, TN, true, kNoSecond>(op, a, slices)
                  : a.act == DH_ACT_NONE ? launch_16bit<WM, WN, TM, TN, true, DH_ACT_NONE>(op, a, slices)
                                         : launch_16bit<WM, WN, TM, TN, true, kAnyAct>(op, a, slices);
  if (a.n_first == a.N) return launch_16bit<WM, WN, TM, TN, false, kNoSecond>(op, a, slices);
  if (a.act == DH_ACT_RELU2) return launch_16bit<WM, WN, TM, TN, false, DH_ACT_RELU2>(op, a, slices);
  if (a.act == DH_ACT_GELU_ERF) return launch_16bit<WM, WN, TM, TN, false, DH_ACT_GELU_ERF>(op, a, slices);
  return launch_16bit<WM, WN, TM, TN, false, kAnyAct>(op, a, slices);
}

// Expert products; the grouped ones launch as many row tiles as the table has room for.
template <bool GROUPED, bool GLU>
int launch_experts(const char* op, GemmArgs a, int a_dtype, int bm) {
  a.k_slice = a.K;
  if (a_dtype == DH_F32) {
    constexpr int TN = GLU ? 2 : 1;
    a.tiles_n = (int)dh::ceil_div(a.N, 64 * TN);
    if (!GROUPED) a.tiles_m = (int)dh::ceil_div(a.M, 64);
    hipLaunchKernelGGL((gemm_f32_kernel<TN, GROUPED, GLU>), dim3(a.tiles_m * a.tiles_n), dim3(256), 0, dh::stream(), a);
  } else {
    a.tiles_n = (int)dh::ceil_div(a.N, 128);
    if (!GROUPED) a.tiles_m = (int)dh::ceil_div(a.M, bm);
    if (bm == 128)
      hipLaunchKernelGGL((gemm_16bit_kernel<2, 2, 2, 2, false, kNoSecond, GROUPED, GLU>), dim3(a.tiles_m * a.tiles_n), dim3(256), 0, dh::stream(), a);
    else
      hipLaunchKernelGGL((gemm_16bit_kernel<2, 2, 1, 2, false, kNoSecond, GROUPED, GLU>), dim3(a.tiles_m * a.tiles_n), dim3(256), 0, dh::stream(), a);
  }
  DH_CHECK_LAUNCH(op);
  return 0;
}

}  // namespace

namespace dh {

int expert_tile_rows(int a_dtype, int rows, int groups) { return a_dtype == DH_F32 ? 64 : rows >= 96 * groups ? 128 : 64; }

int experts_glu(const char* op, const ExpertRows& rows, const void* A, int a_dtype, int64_t lda, const uint16_t* W, int64_t ldw, int M,
                int N, int K, void* out, int out_dtype, int64_t ld_out) {
  GemmArgs a{};
  a.A = A; a.W = W; a.lda = lda; a.ldw = ldw; a.M = M; a.N = N; a.K = K; a.alpha = 1.f;
  a.C2 = out; a.c2_dtype = out_dtype; a.ldc2 = ld_out; a.rows = rows;
  if (rows.tiles) {
    a.tiles_m = rows.max_tiles;
    return launch_experts<true, true>(op, a, a_dtype, rows.tile_rows);
  }
  const int bm = ceil_div(M, 128) * ceil_div(N, 128) >= num_cus() ? 128 : 64;
  return launch_experts<false, true>(op, a, a_dtype, bm);
}

int experts_down(const char* op, const ExpertRows& rows, const void* A, int a_dtype, int64_t lda, const uint16_t* W, int64_t ldw, int N,
                 int K, float* out, int64_t ld_out) {
  GemmArgs a{};
  a.A = A; a.W = W; a.lda = lda; a.ldw = ldw; a.N = N; a.K = K; a.alpha = 1.f;
  a.C = out; a.ldc = ld_out; a.n_first = N; a.rows = rows;
  a.tiles_m = rows.max_tiles;
  return launch_experts<true, false>(op, a, a_dtype, rows.tile_rows);
}

}  // namespace dh

extern "C" int dh_dense_matmul(const void* d_A, int a_dtype, int lda, const void* d_W, int ldw, int M, int N, int K,
                               float alpha, const float* d_bias, const float* d_residual, float* d_C, int ldc, int n_first,
                               void* d_C2, int c2_dtype, int ldc2, int activation) {
  return dh_dense_matmul_scaled(d_A, a_dtype, lda, d_W, ldw, M, N, K, alpha, d_bias, nullptr, d_residual, d_C, ldc, n_first, d_C2,
                                c2_dtype, ldc2, activation);
}

extern "C" int dh_dense_matmul_scaled(const void* d_A, int a_dtype, int lda, const void* d_W, int ldw, int M, int N, int K,
                                      float alpha, const float* d_bias, const float* d_col_scale, const float* d_residual,
                                      float* d_C, int ldc, int n_first, void* d_C2, int c2_dtype, int ldc2, int activation) {
  const char* op = "dh_dense_matmul";
  DH_REQUIRE_INIT(op);
  if (M <= 0 || N <= 0 || K <= 0) return dh::fail(1, "[%s] Dimensions must be positive: M=%d, N=%d, K=%d", op, M, N, K);
  if (K % 64) return dh::fail(1, "[%s] K=%d must be a multiple of 64 (zero-padded)", op, K);
  if (lda < K || ldw < K || lda % 8 || ldw % 8)
    return dh::fail(1, "[%s] row strides must be multiples of 8 and hold K=%d elements (lda=%d, ldw=%d)", op, K, lda, ldw);
  if (a_dtype != DH_BF16 && a_dtype != DH_F32 && a_dtype != DH_F16)
    return dh::fail(1, "[%s] activations must be bf16, f16 (with f16 weights) or f32, got dtype %d", op, a_dtype);
  if (n_first < 0 || n_first > N) return dh::fail(1, "[%s] n_first=%d is outside 0..%d", op, n_first, N);
  if (!d_A || !d_W || (n_first > 0 && !d_C) || (n_first < N && !d_C2)) return dh::fail(1, "[%s] null pointer", op);
  if (n_first > 0 && ldc < n_first) return dh::fail(1, "[%s] ldc=%d is shorter than %d columns", op, ldc, n_first);
  if (n_first < N && (ldc2 < N - n_first || (c2_dtype != DH_BF16 && c2_dtype != DH_F16 && c2_dtype != DH_F32)))
    return dh::fail(1, "[%s] the second output needs %d columns of bf16, f16 or f32 (ldc2=%d, dtype %d)", op, N - n_first, ldc2, c2_dtype);
  if ((reinterpret_cast<uintptr_t>(d_A) | reinterpret_cast<uintptr_t>(d_W)) & 15)
    return dh::fail(1, "[%s] activation and weight pointers must be 16-byte aligned", op);
  GemmArgs a{};
  a.A = d_A; a.W = static_cast<const uint16_t*>(d_W); a.lda = lda; a.ldw = ldw;
  a.M = M; a.N = N; a.K = K; a.alpha = alpha; a.bias = d_bias; a.residual = d_residual; a.col_scale = d_col_scale;
  a.C = d_C; a.ldc = ldc; a.n_first = n_first;
  a.C2 = d_C2; a.ldc2 = ldc2; a.c2_dtype = c2_dtype; a.act = activation;
  if (a_dtype == DH_F32) {
    a.tiles_m = (int)dh::ceil_div(M, 64);
    a.tiles_n = (int)dh::ceil_div(N, 64);
    hipLaunchKernelGGL((gemm_f32_kernel<1, false, false>), dim3(a.tiles_m * a.tiles_n), dim3(256), 0, dh::stream(), a);
    DH_CHECK_LAUNCH(op);
    return 0;
  }
  // 128 x 128 tiles (two workgroups per compute unit) where they fill the device, 64 x 64 otherwise.  (256 x 256 and
  // 256 x 128 tiles measured the same or slower at every shape tried: one workgroup per compute unit hides less.)
  const int cus = dh::num_cus();
  auto tiles = [&](int bm, int bn) { return dh::ceil_div(M, bm) * dh::ceil_div(N, bn); };
  static const int env_tile = dh::tuning_int("DH_DENSE_TILE", 0);
  static const int env_slices = dh::tuning_int("DH_DENSE_SLICES", 0);
  // slices of at least 1024 k, as many as fill the device, within the workspace
  size_t ws_bytes = 0;
  (void)dh::splitk_workspace(&ws_bytes);
  const int64_t most = std::max<int64_t>(1, std::min<int64_t>(K / 1024, (int64_t)(ws_bytes / ((size_t)M * N * sizeof(float)))));
  auto slices_for = [&](int64_t t, int per_cu) { return std::min(most, std::max<int64_t>(1, (int64_t)per_cu * cus / t)); };
  const bool big_enough = tiles(128, 128) >= cus || (M > 64 && tiles(128, 128) * most >= cus);
  const int pick = env_tile ? env_tile : big_enough ? 128 : 64;
  const int64_t t = tiles(pick, pick);
  const int slices = env_slices ? (int)std::min<int64_t>(env_slices, most) : t >= cus ? 1 : (int)slices_for(t, pick == 128 ? 2 : 4);
  const bool f16 = a_dtype == DH_F16;
  return pick == 128 ? launch_tile<2, 2, 2, 2>(op, a, f16, slices) : launch_tile<2, 2, 1, 1>(op, a, f16, slices);
}
