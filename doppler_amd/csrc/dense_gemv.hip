// Products of ONE f32 activation row with dense bf16 weights (decode), HBM-bound.
//
// The row sits in LDS as f32 (optionally RMS-normalised on its way there); a wave streams R weight rows at a time,
// 16 bytes per lane and load with the non-temporal hint, R * U loads of the next stage in flight while the current
// ones are multiplied (f32 fma on the widened weights, so the product is a 32-bit one).  The first stage is requested
// before the row is prepared and travels meanwhile.  The row is kept as two planes of 16-byte pieces (elements
// 0..3 and 4..7 of every eight) so that a wave's reads of either plane are consecutive.
//
// Outputs as in the multi-row product (dense_gemm.hip): columns below n_first with bias, column scale and residual, the rest
// through an activation; or the argmax over all of them (output head).
//
// The HEADS form reads the raw outputs of a layer's heads instead: each head divided by its root mean square, weighted and
// multiplied by the sigmoid of an output gate on its way into LDS.
#include <algorithm>
#include <cfloat>

#include "argmax_device.h"
#include "dense_device.h"

namespace {

using dh::Cand;

constexpr int kMaxK = 32768;
constexpr int kMaxHeads = 256;        // of the HEADS form

struct GemvArgs {
  const float* x;
  const float* norm_weight;   // null: the row as it is
  int hidden;                 // elements the norm's mean runs over
  float eps;
  const uint16_t* W;
  int64_t ldw;
  int N, K;
  float alpha;
  const float* bias;
  const float* residual;
  const float* col_scale;
  float* C;
  int n_first;
  float* C2;
  int act;
  const float* gate;          // HEADS form: one number per element; norm_weight has one too, eps is the heads'
  int heads, head_padded, head_size;
  int iters;                  // row groups per wave
  float* part_val;            // argmax: per-workgroup candidates
  uint32_t* part_idx;
};

template <int R, int U, int WAVES, bool ARGMAX, bool HEADS>
__global__ __launch_bounds__(64 * WAVES) void gemv_kernel(const GemvArgs a) {
  extern __shared__ __align__(16) float4 planes[];      // [2][K / 8]
  __shared__ float red[WAVES];
  __shared__ float sv[WAVES];
  __shared__ uint32_t si[WAVES];
  constexpr int THREADS = 64 * WAVES;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int np = a.K >> 3, nstages = (np + 64 * U - 1) / (64 * U);
  const int units = a.iters * nstages;

  uint4 cur[R][U], nxt[R][U];
  auto first_row = [&](int it) { return ((int64_t)(it * (int)gridDim.x + (int)blockIdx.x) * WAVES + wave) * R; };
  auto load = [&](int unit, uint4 (&dst)[R][U]) {
    const int it = unit / nstages, st = unit - it * nstages;
    const int64_t row0 = first_row(it);
#pragma unroll
    for (int r = 0; r < R; r++) {
      const uint4* w = reinterpret_cast<const uint4*>(a.W + min(row0 + r, (int64_t)a.N - 1) * a.ldw);
#pragma unroll
      for (int u = 0; u < U; u++) {
        const int p = lane + 64 * (u + U * st);
        dst[r][u] = p < np ? dh::stream_load_16(w + p) : make_uint4(0, 0, 0, 0);
      }
    }
  };
  load(0, cur);

  // ---- the activation row
  if constexpr (HEADS) {
    // weighted and gated on the way in; the squares are summed by eight lanes (whole heads: their sizes are multiples of 32), then by
    // head, and the row in LDS is scaled last: one trip to memory
    __shared__ float inv_s[kMaxHeads];
    __shared__ float squares[kMaxK / 32];
    const int hp = a.head_padded >> 2, live = a.heads * hp;       // 16-byte pieces of a head, of all heads
    constexpr int BATCH = 4;                              // pieces requested at once
    for (int i0 = tid; i0 < (a.K >> 2); i0 += THREADS * BATCH) {
      float4 v[BATCH], w[BATCH], g[BATCH];
#pragma unroll
      for (int b = 0; b < BATCH; b++) {
        const int i = i0 + THREADS * b;
        v[b] = w[b] = g[b] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (i < live) {
          v[b] = reinterpret_cast<const float4*>(a.x)[i];
          w[b] = reinterpret_cast<const float4*>(a.norm_weight)[i];
          g[b] = reinterpret_cast<const float4*>(a.gate)[i];
        }
      }
#pragma unroll
      for (int b = 0; b < BATCH; b++) {
        const int i = i0 + THREADS * b;
        if (i >= (a.K >> 2)) break;                       // sixteen lanes at a time: K is a multiple of 64
        float4 y = v[b];
        float ss = fmaf(y.x, y.x, fmaf(y.y, y.y, fmaf(y.z, y.z, y.w * y.w)));
        y.x = y.x * w[b].x * __frcp_rn(1.0f + __expf(-g[b].x)); y.y = y.y * w[b].y * __frcp_rn(1.0f + __expf(-g[b].y));
        y.z = y.z * w[b].z * __frcp_rn(1.0f + __expf(-g[b].z)); y.w = y.w * w[b].w * __frcp_rn(1.0f + __expf(-g[b].w));
        planes[(i & 1) * np + (i >> 1)] = y;
        ss = dh::group_combine<1, 8>(ss, dh::AddOp());
        if ((i & 7) == 0) squares[i >> 3] = ss;
      }
    }
    __syncthreads();
    for (int h = tid; h < a.heads; h += THREADS) {
      float ss = 0.f;
      for (int k = h * (hp >> 3); k < (h + 1) * (hp >> 3); k++) ss += squares[k];
      inv_s[h] = 1.0f / sqrtf(ss / (float)a.head_size + a.eps);
    }
    __syncthreads();
    for (int i = tid; i < live; i += THREADS) {
      const float f = inv_s[i / hp];
      float4& v = planes[(i & 1) * np + (i >> 1)];
      v.x *= f; v.y *= f; v.z *= f; v.w *= f;
    }
  } else {
    const float4* xg = reinterpret_cast<const float4*>(a.x);
    float inv = 1.f;
    if (a.norm_weight) {
      float ss = 0.f;
      for (int i = tid; i < (a.K >> 2); i += THREADS) {
        const float4 v = xg[i];
        ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
      }
      ss = dh::wave_sum_uniform(ss);
      if (lane == 0) red[wave] = ss;
      __syncthreads();
      float total = 0.f;
#pragma unroll
      for (int w = 0; w < WAVES; w++) total += red[w];
      inv = 1.0f / sqrtf(total / (float)a.hidden + a.eps);
    }
    for (int i = tid; i < (a.K >> 2); i += THREADS) {
      float4 v = xg[i];
      if (a.norm_weight) {
        const float4 w = reinterpret_cast<const float4*>(a.norm_weight)[i];
        v.x = v.x * inv * w.x; v.y = v.y * inv * w.y; v.z = v.z * inv * w.z; v.w = v.w * inv * w.w;
      }
      planes[(i & 1) * np + (i >> 1)] = v;
    }
  }
  __syncthreads();

  float acc[R];
#pragma unroll
  for (int r = 0; r < R; r++) acc[r] = 0.f;
  Cand best{-FLT_MAX, 0xFFFFFFFFu};
  int st = 0, it = 0;
  for (int unit = 0; unit < units; unit++) {
    if (unit + 1 < units) load(unit + 1, nxt);
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int p = min(lane + 64 * (u + U * st), np - 1);      // past the row the weights are zeros
      const float4 xa = planes[p], xb = planes[np + p];
#pragma unroll
      for (int r = 0; r < R; r++) {
        const uint4 w = cur[r][u];
        float s = acc[r];
        s = fmaf(xa.x, dh::bf16_low(w.x), s); s = fmaf(xa.y, dh::bf16_high(w.x), s);
        s = fmaf(xa.z, dh::bf16_low(w.y), s); s = fmaf(xa.w, dh::bf16_high(w.y), s);
        s = fmaf(xb.x, dh::bf16_low(w.z), s); s = fmaf(xb.y, dh::bf16_high(w.z), s);
        s = fmaf(xb.z, dh::bf16_low(w.w), s); s = fmaf(xb.w, dh::bf16_high(w.w), s);
        acc[r] = s;
      }
    }
    if (++st == nstages) {
      const int64_t row0 = first_row(it);
#pragma unroll
      for (int r = 0; r < R; r++) {
        const float v = dh::wave_sum_uniform(acc[r]) * a.alpha;
        acc[r] = 0.f;
        const int64_t n = row0 + r;
        if (lane == 0 && n < a.N) {
          if (n < a.n_first) {
            float y = v + (a.bias ? a.bias[n] : 0.f);
            if (a.col_scale) y *= a.col_scale[n];
            if (a.residual) y += a.residual[n];
            if (a.C) a.C[n] = y;
          } else {
            a.C2[n - a.n_first] = dh::activate(v, a.act);
          }
          if (ARGMAX && dh::beats(v, (uint32_t)n, best.v, best.i)) { best.v = v; best.i = (uint32_t)n; }
        }
      }
      st = 0;
      it++;
    }
#pragma unroll
    for (int r = 0; r < R; r++)
#pragma unroll
      for (int u = 0; u < U; u++) cur[r][u] = nxt[r][u];
  }
  if (ARGMAX) {
    if (lane == 0) { sv[wave] = best.v; si[wave] = best.i; }
    __syncthreads();
    if (tid == 0) {
      for (int w = 1; w < WAVES; w++)
        if (dh::beats(sv[w], si[w], best.v, best.i)) { best.v = sv[w]; best.i = si[w]; }
      a.part_val[blockIdx.x] = best.v;
      a.part_idx[blockIdx.x] = best.i;
    }
  }
}

template <int R, int U, int WAVES, bool ARGMAX, bool HEADS>
int launch(const char* op, GemvArgs a, int max_grid, int* parts) {
  auto kern = gemv_kernel<R, U, WAVES, ARGMAX, HEADS>;
  static bool attr_set = false;
  if (!attr_set) {
    DH_CHECK_HIP(op, hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize,
                                         kMaxK * 4));
    attr_set = true;
  }
  const int64_t groups = dh::ceil_div(a.N, R * WAVES);
  a.iters = (int)std::max<int64_t>(1, dh::ceil_div(groups, max_grid));
  const int grid = (int)dh::ceil_div(groups, a.iters);
  hipLaunchKernelGGL(kern, dim3(grid), dim3(64 * WAVES), (size_t)a.K * 4, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  if (parts) *parts = grid;
  return 0;
}

template <bool ARGMAX, bool HEADS = false>
int dispatch(const char* op, const GemvArgs& a, int* parts) {
  // workgroups that are resident at once share the activation row's preparation as widely as the LDS allows
  const int cus = dh::num_cus();
  static const int env_r = dh::tuning_int("DH_DENSE_GEMV_R", 0);
  if constexpr (HEADS) {
    // every workgroup reads three rows to prepare one: wide workgroups, as long as there is one for every compute unit
    static const int env_w = dh::tuning_int("DH_GEMV_HEADS_WAVES", 0);
    const int waves = env_w ? env_w : a.N >= 16 * cus ? 16 : a.N >= 8 * cus ? 8 : 4;
    if (a.K <= 8192 && waves == 16) return launch<1, 8, 16, ARGMAX, HEADS>(op, a, cus, parts);
    if (a.K <= 8192 && waves == 8) return launch<1, 8, 8, ARGMAX, HEADS>(op, a, 2 * cus, parts);
  }
  const bool two = env_r ? env_r == 2 : a.K <= 4096 && (int64_t)a.N >= (int64_t)64 * cus;
  if (a.K <= 8192) {
    const int max_grid = ARGMAX ? std::min(4 * cus, dh::kMaxParts) : 4 * cus;
    return two ? launch<2, 4, 4, ARGMAX, HEADS>(op, a, max_grid, parts) : launch<1, 8, 4, ARGMAX, HEADS>(op, a, max_grid, parts);
  }
  const int max_grid = a.K <= 16384 ? 2 * cus : cus;
  return launch<1, 8, 8, ARGMAX, HEADS>(op, a, std::min(max_grid, dh::kMaxParts), parts);
}

int check(const char* op, const float* x, const float* norm_weight, int hidden, float eps, const void* W, int ldw, int N, int K) {
  if (N <= 0 || K <= 0) return dh::fail(1, "[%s] Dimensions must be positive: N=%d, K=%d", op, N, K);
  if (K % 64 || K > kMaxK) return dh::fail(1, "[%s] K=%d must be a multiple of 64 and at most %d", op, K, kMaxK);
  if (ldw < K || ldw % 8) return dh::fail(1, "[%s] ldw=%d must be a multiple of 8 and hold K=%d elements", op, ldw, K);
  if (!x || !W) return dh::fail(1, "[%s] null pointer", op);
  if (norm_weight && (hidden <= 0 || hidden > K || !(eps >= 0.f)))
    return dh::fail(1, "[%s] the norm needs 0 < hidden <= K and eps >= 0 (hidden=%d, K=%d)", op, hidden, K);
  if ((reinterpret_cast<uintptr_t>(x) | reinterpret_cast<uintptr_t>(W) | reinterpret_cast<uintptr_t>(norm_weight)) & 15)
    return dh::fail(1, "[%s] activation, norm and weight pointers must be 16-byte aligned", op);
  return 0;
}

GemvArgs make_args(const float* x, const float* norm_weight, int hidden, float eps, const void* W, int ldw, int N, int K,
                   float alpha) {
  GemvArgs a{};
  a.x = x; a.norm_weight = norm_weight; a.hidden = hidden; a.eps = eps;
  a.W = static_cast<const uint16_t*>(W); a.ldw = ldw; a.N = N; a.K = K; a.alpha = alpha; a.n_first = N;
  a.act = DH_ACT_NONE;
  return a;
}

}  // namespace

extern "C" {

int dh_dense_gemv(const float* d_x, const float* d_norm_weight, int hidden, float eps, const void* d_W, int ldw, int N,
                  int K, float alpha, const float* d_bias, const float* d_residual, float* d_C, int n_first, float* d_C2,
                  int activation) {
  return dh_dense_gemv_scaled(d_x, d_norm_weight, hidden, eps, d_W, ldw, N, K, alpha, d_bias, nullptr, d_residual, d_C, n_first, d_C2,
                              activation);
}

int dh_dense_gemv_scaled(const float* d_x, const float* d_norm_weight, int hidden, float eps, const void* d_W, int ldw, int N,
                         int K, float alpha, const float* d_bias, const float* d_col_scale, const float* d_residual, float* d_C,
                         int n_first, float* d_C2, int activation) {
  const char* op = "dh_dense_gemv";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, d_x, d_norm_weight, hidden, eps, d_W, ldw, N, K)) return rc;
  if (n_first < 0 || n_first > N) return dh::fail(1, "[%s] n_first=%d is outside 0..%d", op, n_first, N);
  if ((n_first > 0 && !d_C) || (n_first < N && !d_C2)) return dh::fail(1, "[%s] null output pointer", op);
  if (d_x == d_C || d_x == d_C2) return dh::fail(1, "[%s] an output must not be the activation row", op);
  GemvArgs a = make_args(d_x, d_norm_weight, hidden, eps, d_W, ldw, N, K, alpha);
  a.bias = d_bias; a.col_scale = d_col_scale; a.residual = d_residual; a.C = d_C; a.n_first = n_first; a.C2 = d_C2; a.act = activation;
  return dispatch<false>(op, a, nullptr);
}

int dh_dense_gemv_heads(const float* d_x, const float* d_gate, const float* d_weight, int H, int padded, int size, float eps, const void* d_W,
                        int ldw, int N, int K, const float* d_col_scale, const float* d_residual, float* d_C) {
  const char* op = "dh_dense_gemv_heads";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, d_x, nullptr, 0, eps, d_W, ldw, N, K)) return rc;
  if (H <= 0 || H > kMaxHeads || size <= 0 || padded < size || padded % 32 || (int64_t)H * padded > K)
    return dh::fail(1, "[%s] %d heads (at most %d) of %d elements, %d apart (a multiple of 32), in a row of %d", op, H, kMaxHeads, size, padded, K);
  if (!d_gate || !d_weight || !d_C) return dh::fail(1, "[%s] null pointer", op);
  if ((reinterpret_cast<uintptr_t>(d_gate) | reinterpret_cast<uintptr_t>(d_weight)) & 15) return dh::fail(1, "[%s] gate and weight must be 16-byte aligned", op);
  if (d_x == d_C) return dh::fail(1, "[%s] the output must not be the activation row", op);
  GemvArgs a = make_args(d_x, d_weight, 0, eps, d_W, ldw, N, K, 1.f);
  a.gate = d_gate; a.heads = H; a.head_padded = padded; a.head_size = size;
  a.col_scale = d_col_scale; a.residual = d_residual; a.C = d_C;
  return dispatch<false, true>(op, a, nullptr);
}

int dh_dense_lmhead_argmax(const float* d_x, const float* d_norm_weight, int hidden, float eps, const void* d_W, int ldw,
                           int vocab, int K, float alpha, void* d_workspace, uint32_t* d_token_out, int output_index,
                           float* d_logits_out) {
  const char* op = "dh_dense_lmhead_argmax";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, d_x, d_norm_weight, hidden, eps, d_W, ldw, vocab, K)) return rc;
  if (!d_workspace || !d_token_out) return dh::fail(1, "[%s] null pointer", op);
  if (output_index < 0) return dh::fail(1, "[%s] outputIndex must be non-negative", op);
  GemvArgs a = make_args(d_x, d_norm_weight, hidden, eps, d_W, ldw, vocab, K, alpha);
  a.C = d_logits_out;
  a.part_val = static_cast<float*>(d_workspace);
  a.part_idx = reinterpret_cast<uint32_t*>(static_cast<char*>(d_workspace) + (size_t)dh::kMaxParts * 4);
  int parts = 0;
  if (int rc = dispatch<true>(op, a, &parts)) return rc;
  return dh::launch_argmax_final(op, a.part_val, a.part_idx, parts, d_token_out, output_index);
}

}  // extern "C"
