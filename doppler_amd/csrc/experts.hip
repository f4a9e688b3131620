// Mixtures of experts (dh_experts): every token uses the `top` experts with the largest router logits z, each weighted with
// sigmoid(z), and a shared expert weighted with sigmoid of one more logit.
//
//   expert(x) = W_down glu(W_gate x, W_up x),   glu(g, u) = g' sigmoid(1.702 g') (clamp(u, +-limit) + 1),  g' = min(g, limit)
//   out       = sum over chosen e of expert_e(s_e h) + sigmoid(z_shared) expert_shared(h)
//
// A weight multiplies its expert's input, so it scales the gate and up products in front of the clamps; the products
// themselves always read h.  The shared expert's weight scales its activations.
//
// Gate and up rows alternate in blocks of 32 (the matrix-core epilogue wants both of a column in one lane).
//
// Decode: experts_up_kernel chooses the experts itself (every workgroup, from the few logits), norms the row and streams the
// chosen gate and up rows; experts_down_kernel streams the chosen down matrices and the shared one side by side along k.
// Prefill: experts_route_kernel, experts_sort_kernel (rows sorted by expert, table of row tiles), grouped products on the
// matrix cores (dense_gemm.hip), experts_combine_kernel.
#include <algorithm>
#include <cfloat>

#include "argmax_device.h"
#include "experts.h"

namespace {

constexpr int kMaxTop = 32;
constexpr int kMaxExperts = 1024;

struct StepArgs {
  const float* x;
  const float* norm;
  const float* z;          // router logits [E], then the shared expert's
  const uint16_t* up;      // [E][2 ff][ld_in]
  const uint16_t* down;    // [E][hidden][ff]
  const uint16_t* shared_up;
  const uint16_t* shared_down;
  const float* ls;         // [hidden] or null
  float* act;              // [top ff + shared_ff]
  float* out;              // residual row, added to
  int hidden, K, E, top, ff, shared_ff;
  float eps, limit, shared_limit;
};

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// The top experts of a row of logits, by one wave: ids (and logits) in the order of their size, the lower id first among equals.
// Lane l holds experts l, l + 64, .., 64 SLOTS in all; the maximum is found by lane steps, its lowest holder from a ballot.
template <int SLOTS>
__device__ __forceinline__ void choose_upto(const float* z, int E, int top, int* ids, float* zs) {
  const int lane = threadIdx.x & 63;
  float v[SLOTS];
#pragma unroll
  for (int j = 0; j < SLOTS; j++) v[j] = lane + 64 * j < E ? z[lane + 64 * j] : -INFINITY;
  for (int t = 0; t < top; t++) {
    float best = v[0];
#pragma unroll
    for (int j = 1; j < SLOTS; j++) best = fmaxf(best, v[j]);
    const float mx = dh::group_combine<1, 64>(best, dh::MaxOp());
    int id = 0;                                          // logits that are not numbers: some expert, inside the tables
    bool found = false;
#pragma unroll
    for (int j = 0; j < SLOTS; j++) {
      const unsigned long long at = __builtin_amdgcn_ballot_w64(v[j] == mx && lane + 64 * j < E);
      if (!found && at != 0) {
        id = 64 * j + __builtin_ctzll(at);
        found = true;
      }
    }
    if (lane == 0) {
      ids[t] = id;
      zs[t] = mx;
    }
#pragma unroll
    for (int j = 0; j < SLOTS; j++)
      if (lane + 64 * j == id) v[j] = -INFINITY;
  }
}
__device__ __forceinline__ void choose(const float* z, int E, int top, int* ids, float* zs) {
  if (E <= 64) choose_upto<1>(z, E, top, ids, zs);
  else if (E <= 256) choose_upto<4>(z, E, top, ids, zs);
  else choose_upto<kMaxExperts / 64>(z, E, top, ids, zs);
}

// A wave takes a gate and an up row at a time; the row sits in LDS as two planes of 16-byte pieces, as in the dense GEMV.
template <int U>
__global__ __launch_bounds__(256) void experts_up_kernel(const StepArgs a, int iters) {
  extern __shared__ __align__(16) float4 planes[];       // [2][K / 8]
  __shared__ float red[4];
  __shared__ int ids[kMaxTop];
  __shared__ float zs[kMaxTop];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int np = a.K >> 3, nstages = (np + 64 * U - 1) / (64 * U);
  const float4* xg = reinterpret_cast<const float4*>(a.x);
  float ss = 0.f;
  for (int i = tid; i < (a.K >> 2); i += 256) {
    const float4 v = xg[i];
    ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
  }
  ss = dh::wave_sum_uniform(ss);
  if (lane == 0) red[wave] = ss;
  if (wave == 0) choose(a.z, a.E, a.top, ids, zs);
  __syncthreads();
  const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.hidden + a.eps);
  for (int i = tid; i < (a.K >> 2); i += 256) {
    float4 v = xg[i];
    const float4 w = reinterpret_cast<const float4*>(a.norm)[i];
    v.x = v.x * inv * w.x; v.y = v.y * inv * w.y; v.z = v.z * inv * w.z; v.w = v.w * inv * w.w;
    planes[(i & 1) * np + (i >> 1)] = v;
  }
  __syncthreads();
  const int total = a.top * a.ff + a.shared_ff;
  uint4 cur[2][U], nxt[2][U];
  auto load = [&](int unit, uint4 (&dst)[2][U]) {
    const int it = unit / nstages, st = unit - it * nstages;
    const int col = min((it * (int)gridDim.x + (int)blockIdx.x) * 4 + wave, total - 1);
    const bool shared = col >= a.top * a.ff;
    const int c = shared ? col - a.top * a.ff : col % a.ff;
    const uint16_t* m = shared ? a.shared_up : a.up + (int64_t)ids[col / a.ff] * 2 * a.ff * a.K;
#pragma unroll
    for (int r = 0; r < 2; r++) {
      const uint4* w = reinterpret_cast<const uint4*>(m + (int64_t)(64 * (c >> 5) + 32 * r + (c & 31)) * a.K);
#pragma unroll
      for (int u = 0; u < U; u++) {
        const int p = lane + 64 * (u + U * st);
        dst[r][u] = p < np ? dh::stream_load_16(w + p) : make_uint4(0, 0, 0, 0);
      }
    }
  };
  load(0, cur);
  float acc[2] = {0.f, 0.f};
  int st = 0, it = 0;
  for (int unit = 0; unit < iters * nstages; unit++) {
    if (unit + 1 < iters * nstages) load(unit + 1, nxt);
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int p = min(lane + 64 * (u + U * st), np - 1);
      const float4 xa = planes[p], xb = planes[np + p];
#pragma unroll
      for (int r = 0; r < 2; r++) {
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
      const float g = dh::wave_sum_uniform(acc[0]), u = dh::wave_sum_uniform(acc[1]);
      const int col = (it * (int)gridDim.x + (int)blockIdx.x) * 4 + wave;
      if (lane == 0 && col < total) {
        if (col >= a.top * a.ff) {
          a.act[col] = dh::clamped_glu(g, u, a.shared_limit) * sigmoid_f(a.z[a.E]);
        } else {
          const float s = sigmoid_f(zs[col / a.ff]);
          a.act[col] = dh::clamped_glu(s * g, s * u, a.limit);
        }
      }
      acc[0] = acc[1] = 0.f;
      st = 0;
      it++;
    }
#pragma unroll
    for (int r = 0; r < 2; r++)
#pragma unroll
      for (int u = 0; u < U; u++) cur[r][u] = nxt[r][u];
  }
}

// out[n] += ls[n] * [chosen down rows | shared down row] . act; a wave takes R rows at a time.
template <int R, int U>
__global__ __launch_bounds__(256) void experts_down_kernel(const StepArgs a, int iters) {
  extern __shared__ __align__(16) float4 planes[];       // [2][total / 8]
  __shared__ int ids[kMaxTop];
  __shared__ float zs[kMaxTop];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int np = (a.top * a.ff + a.shared_ff) >> 3, npe = a.ff >> 3, routed = a.top * npe;
  const int nstages = (np + 64 * U - 1) / (64 * U);
  if (wave == 0) choose(a.z, a.E, a.top, ids, zs);
  for (int i = tid; i < 2 * np; i += 256) planes[(i & 1) * np + (i >> 1)] = reinterpret_cast<const float4*>(a.act)[i];
  __syncthreads();
  uint4 cur[R][U], nxt[R][U];
  auto first_row = [&](int it) { return ((it * (int)gridDim.x + (int)blockIdx.x) * 4 + wave) * R; };
  auto load = [&](int unit, uint4 (&dst)[R][U]) {
    const int it = unit / nstages, st = unit - it * nstages, row0 = first_row(it);
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int p = lane + 64 * (u + U * st);
      const uint16_t* w = nullptr;
      int64_t ld = 0;
      if (p < routed) {
        w = a.down + (int64_t)ids[p / npe] * a.hidden * a.ff + 8 * (p % npe);
        ld = a.ff;
      } else if (p < np) {
        w = a.shared_down + 8 * (p - routed);
        ld = a.shared_ff;
      }
#pragma unroll
      for (int r = 0; r < R; r++)
        dst[r][u] = w ? dh::stream_load_16(reinterpret_cast<const uint4*>(w + (int64_t)min(row0 + r, a.hidden - 1) * ld)) : make_uint4(0, 0, 0, 0);
    }
  };
  load(0, cur);
  float acc[R];
#pragma unroll
  for (int r = 0; r < R; r++) acc[r] = 0.f;
  int st = 0, it = 0;
  for (int unit = 0; unit < iters * nstages; unit++) {
    if (unit + 1 < iters * nstages) load(unit + 1, nxt);
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int p = min(lane + 64 * (u + U * st), np - 1);
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
      const int row0 = first_row(it);
#pragma unroll
      for (int r = 0; r < R; r++) {
        const float v = dh::wave_sum_uniform(acc[r]);
        acc[r] = 0.f;
        const int n = row0 + r;
        if (lane == 0 && n < a.hidden) a.out[n] = fmaf(a.ls ? a.ls[n] : 1.f, v, a.out[n]);
      }
      st = 0;
      it++;
    }
#pragma unroll
    for (int r = 0; r < R; r++)
#pragma unroll
      for (int u = 0; u < U; u++) cur[r][u] = nxt[r][u];
  }
}

// ------------------------------------------------------------------ portions

// One wave per token.
__global__ __launch_bounds__(256) void experts_route_kernel(const float* __restrict__ z, int64_t ld_z, int T, int E, int top, int shared,
                                                            int* __restrict__ ids, float* __restrict__ weights, float* __restrict__ sg) {
  __shared__ int id_s[4][kMaxTop];
  __shared__ float z_s[4][kMaxTop];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, t = blockIdx.x * 4 + wave;
  if (t >= T) return;
  const float* row = z + (int64_t)t * ld_z;
  choose(row, E, top, id_s[wave], z_s[wave]);
  __builtin_amdgcn_wave_barrier();
  if (lane < top) {
    ids[(int64_t)t * top + lane] = id_s[wave][lane];
    weights[(int64_t)t * top + lane] = sigmoid_f(z_s[wave][lane]);
  }
  if (shared && lane == 0) sg[t] = sigmoid_f(row[E]);
}

// One workgroup: rows sorted by expert.  slot[i]: sorted place of choice i = token * top + k; row_token, row_weight by place.
__global__ __launch_bounds__(1024) void experts_sort_kernel(const int* __restrict__ ids, const float* __restrict__ weights, int n, int top,
                                                            int E, int tile_rows, int max_tiles, int* __restrict__ off, int* __restrict__ slot,
                                                            int* __restrict__ row_token, float* __restrict__ row_weight, int* __restrict__ tiles) {
  __shared__ int count[kMaxExperts];
  __shared__ int scan[kMaxExperts];
  __shared__ int tscan[kMaxExperts];
  const int tid = threadIdx.x;
  count[tid] = 0;
  __syncthreads();
  constexpr int BATCH = 8;                               // reads in flight per thread
  for (int i0 = tid; i0 < n; i0 += 1024 * BATCH) {
    int id[BATCH];
#pragma unroll
    for (int k = 0; k < BATCH; k++) id[k] = i0 + 1024 * k < n ? ids[i0 + 1024 * k] : -1;
#pragma unroll
    for (int k = 0; k < BATCH; k++)
      if (id[k] >= 0) atomicAdd(&count[id[k]], 1);
  }
  __syncthreads();
  const int mine = count[tid], my_tiles = (mine + tile_rows - 1) / tile_rows;
  scan[tid] = mine;
  tscan[tid] = my_tiles;
  __syncthreads();
  for (int o = 1; o < kMaxExperts; o <<= 1) {
    const int a = tid >= o ? scan[tid - o] : 0, b = tid >= o ? tscan[tid - o] : 0;
    __syncthreads();
    scan[tid] += a;
    tscan[tid] += b;
    __syncthreads();
  }
  const int first = scan[tid] - mine, first_tile = tscan[tid] - my_tiles, used = tscan[kMaxExperts - 1];
  if (tid < E) off[tid] = first;
  if (tid == E - 1) off[E] = n;
  for (int k = 0; k < my_tiles; k++) {
    tiles[2 * (first_tile + k)] = tid;
    tiles[2 * (first_tile + k) + 1] = k * tile_rows;
  }
  for (int k = used + tid; k < max_tiles; k += 1024) tiles[2 * k] = -1;
  count[tid] = first;                                    // next free place of the expert
  __syncthreads();
  for (int i0 = tid; i0 < n; i0 += 1024 * BATCH) {
    int id[BATCH];
    float w[BATCH];
#pragma unroll
    for (int k = 0; k < BATCH; k++) {
      const int i = i0 + 1024 * k;
      id[k] = i < n ? ids[i] : -1;
      w[k] = i < n ? weights[i] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < BATCH; k++) {
      const int i = i0 + 1024 * k;
      if (id[k] < 0) continue;
      const int at = atomicAdd(&count[id[k]], 1);        // any order inside a group: a row's results do not depend on its place
      slot[i] = at;
      row_token[at] = i / top;
      row_weight[at] = w[k];
    }
  }
}

// x[t] += ls * sum of the token's rows.  Four columns per thread.
__global__ __launch_bounds__(256) void experts_combine_kernel(const float* __restrict__ y, int64_t ld_y, const int* __restrict__ slot, int top,
                                                              const float* __restrict__ ls, float* __restrict__ x, int64_t ld_x, int hidden) {
  const int t = blockIdx.x, i = 4 * (blockIdx.y * 256 + threadIdx.x);
  if (i >= hidden) return;
  float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int k = 0; k < top; k++) {
    const float4 v = *reinterpret_cast<const float4*>(y + (int64_t)slot[(int64_t)t * top + k] * ld_y + i);
    s.x += v.x; s.y += v.y; s.z += v.z; s.w += v.w;
  }
  const float sv[4] = {s.x, s.y, s.z, s.w};
#pragma unroll
  for (int e = 0; e < 4; e++) {
    if (i + e >= hidden) break;
    float* o = x + (int64_t)t * ld_x + i + e;
    *o = fmaf(ls ? ls[i + e] : 1.f, sv[e], *o);
  }
}

size_t up256(size_t n) { return (n + 255) / 256 * 256; }
bool aligned(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

int check(const char* op, const dh_experts* s) {
  if (!s) return dh::fail(1, "[%s] null spec", op);
  if (s->hidden <= 0 || s->K < s->hidden || s->K % 64) return dh::fail(1, "[%s] hidden=%d in rows of %d (a multiple of 64)", op, s->hidden, s->K);
  if (s->experts <= 0 || s->experts > kMaxExperts || s->top <= 0 || s->top > kMaxTop || s->top > s->experts)
    return dh::fail(1, "[%s] %d of %d experts (at most %d of %d)", op, s->top, s->experts, kMaxTop, kMaxExperts);
  if (s->ff <= 0 || s->ff % 64 || s->shared_ff < 0 || s->shared_ff % 64) return dh::fail(1, "[%s] expert widths must be multiples of 64 (%d, shared %d)", op, s->ff, s->shared_ff);
  if (!s->d_router || !s->d_up || !s->d_down || !s->d_norm || (s->shared_ff && (!s->d_shared_up || !s->d_shared_down))) return dh::fail(1, "[%s] null pointer in the spec", op);
  if (!aligned(s->d_router) || !aligned(s->d_up) || !aligned(s->d_down) || !aligned(s->d_norm) || !aligned(s->d_shared_up) || !aligned(s->d_shared_down))
    return dh::fail(1, "[%s] weights must be 16-byte aligned", op);
  return 0;
}
int logits(const dh_experts* s) { return s->experts + (s->shared_ff ? 1 : 0); }

// Where a portion's intermediate rows lie in the workspace.
struct PortionSpace {
  size_t z, ids, weights, sg, off, slot, row_token, row_weight, tiles, act, shared_act, y, end;
  int ld_z, ld_y, max_tiles, tile_rows;
};
PortionSpace portion_space(const dh_experts* s, int operand, int T) {
  PortionSpace p{};
  const size_t n = (size_t)T * s->top, elem = operand == DH_F32 ? 4 : 2;
  p.ld_z = (logits(s) + 3) / 4 * 4;
  p.ld_y = (s->hidden + 3) / 4 * 4;
  p.tile_rows = dh::expert_tile_rows(operand, (int)n, s->experts);
  p.max_tiles = (int)(n / p.tile_rows + std::min<size_t>(n, s->experts));
  size_t at = 0;
  auto take = [&](size_t bytes) { const size_t r = at; at += up256(bytes); return r; };
  p.z = take((size_t)T * p.ld_z * 4);
  p.ids = take(n * 4); p.weights = take(n * 4); p.sg = take((size_t)T * 4);
  p.off = take((size_t)(s->experts + 1) * 4); p.slot = take(n * 4); p.row_token = take(n * 4); p.row_weight = take(n * 4);
  p.tiles = take((size_t)p.max_tiles * 8);
  p.act = take(n * s->ff * elem);
  p.shared_act = take((size_t)T * s->shared_ff * elem);
  p.y = take(n * p.ld_y * 4);
  p.end = at;
  return p;
}

}  // namespace

extern "C" {

size_t dh_experts_step_workspace_bytes(const dh_experts* s) {
  if (!s) return 256;
  return up256((size_t)logits(s) * 4) + up256(((size_t)s->top * s->ff + s->shared_ff) * 4);
}

int dh_experts_step(const dh_experts* spec, float* d_x, void* d_workspace) {
  const char* op = "dh_experts_step";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (!d_x || !d_workspace) return dh::fail(1, "[%s] null pointer", op);
  if (!aligned(d_x) || !aligned(d_workspace)) return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  const int64_t total = (int64_t)spec->top * spec->ff + spec->shared_ff;
  if (spec->K > 32768 || total > 32768) return dh::fail(1, "[%s] rows of %d and %lld elements: at most 32768 fit one workgroup", op, spec->K, (long long)total);
  float* z = static_cast<float*>(d_workspace);
  float* act = reinterpret_cast<float*>(static_cast<char*>(d_workspace) + up256((size_t)logits(spec) * 4));
  if (int rc = dh_dense_gemv(d_x, spec->d_norm, spec->hidden, spec->eps, spec->d_router, spec->K, logits(spec), spec->K, 1.f, nullptr, nullptr, z,
                             logits(spec), nullptr, DH_ACT_NONE))
    return rc;
  StepArgs a{};
  a.x = d_x; a.norm = spec->d_norm; a.z = z;
  a.up = static_cast<const uint16_t*>(spec->d_up); a.down = static_cast<const uint16_t*>(spec->d_down);
  a.shared_up = static_cast<const uint16_t*>(spec->d_shared_up); a.shared_down = static_cast<const uint16_t*>(spec->d_shared_down);
  a.ls = spec->d_layer_scale; a.act = act; a.out = d_x;
  a.hidden = spec->hidden; a.K = spec->K; a.E = spec->experts; a.top = spec->top; a.ff = spec->ff; a.shared_ff = spec->shared_ff;
  a.eps = spec->eps; a.limit = spec->limit; a.shared_limit = spec->shared_limit;
  static bool attr_set = false;
  if (!attr_set) {
    for (const void* k : {reinterpret_cast<const void*>(experts_up_kernel<4>), reinterpret_cast<const void*>(experts_down_kernel<1, 8>)})
      DH_CHECK_HIP(op, hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, 32768 * 4));
    attr_set = true;
  }
  auto plan = [&](int64_t units, int64_t k, int* iters) {
    const int64_t most = (k <= 8192 ? 4 : k <= 16384 ? 2 : 1) * (int64_t)dh::num_cus();
    *iters = (int)std::max<int64_t>(1, dh::ceil_div(units, most));
    return dim3((unsigned)dh::ceil_div(units, *iters));
  };
  int iters = 1;
  dim3 grid = plan(dh::ceil_div(total, 4), spec->K, &iters);
  hipLaunchKernelGGL(experts_up_kernel<4>, grid, dim3(256), (size_t)spec->K * 4, dh::stream(), a, iters);
  DH_CHECK_LAUNCH(op);
  grid = plan(dh::ceil_div(spec->hidden, 4), total, &iters);
  hipLaunchKernelGGL((experts_down_kernel<1, 8>), grid, dim3(256), (size_t)total * 4, dh::stream(), a, iters);
  DH_CHECK_LAUNCH(op);
  return 0;
}

size_t dh_experts_prefill_workspace_bytes(const dh_experts* s, int operand, int T) { return s && T > 0 ? portion_space(s, operand, T).end : 256; }

int dh_experts_prefill(const dh_experts* spec, const void* d_h, int operand, float* d_x, int ld_x, void* d_workspace, int T) {
  const char* op = "dh_experts_prefill";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (T <= 0 || ld_x < spec->hidden) return dh::fail(1, "[%s] %d rows %d apart", op, T, ld_x);
  if (operand != DH_BF16 && operand != DH_F32) return dh::fail(1, "[%s] activations must be bf16 or f32, got dtype %d", op, operand);
  if (!d_h || !d_x || !d_workspace) return dh::fail(1, "[%s] null pointer", op);
  if (!aligned(d_h) || !aligned(d_workspace)) return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  if ((int64_t)T * spec->top > (1 << 24)) return dh::fail(1, "[%s] %d tokens are too many for one portion", op, T);
  const PortionSpace p = portion_space(spec, operand, T);
  char* w = static_cast<char*>(d_workspace);
  auto f32 = [&](size_t at) { return reinterpret_cast<float*>(w + at); };
  auto i32 = [&](size_t at) { return reinterpret_cast<int*>(w + at); };
  const int n = T * spec->top;
  if (int rc = dh_dense_matmul(d_h, operand, spec->K, spec->d_router, spec->K, T, logits(spec), spec->K, 1.f, nullptr, nullptr, f32(p.z), p.ld_z,
                               logits(spec), nullptr, 0, 0, DH_ACT_NONE))
    return rc;
  hipLaunchKernelGGL(experts_route_kernel, dim3((unsigned)dh::ceil_div(T, 4)), dim3(256), 0, dh::stream(), f32(p.z), (int64_t)p.ld_z, T, spec->experts,
                     spec->top, spec->shared_ff > 0 ? 1 : 0, i32(p.ids), f32(p.weights), f32(p.sg));
  DH_CHECK_LAUNCH(op);
  hipLaunchKernelGGL(experts_sort_kernel, dim3(1), dim3(1024), 0, dh::stream(), i32(p.ids), f32(p.weights), n, spec->top, spec->experts, p.tile_rows,
                     p.max_tiles, i32(p.off), i32(p.slot), i32(p.row_token), f32(p.row_weight), i32(p.tiles));
  DH_CHECK_LAUNCH(op);
  dh::ExpertRows rows{};
  rows.tiles = i32(p.tiles); rows.group_off = i32(p.off); rows.row_index = i32(p.row_token); rows.w_stride = (int64_t)2 * spec->ff * spec->K;
  rows.max_tiles = p.max_tiles; rows.tile_rows = p.tile_rows; rows.row_in = f32(p.row_weight); rows.limit = spec->limit;
  if (int rc = dh::experts_glu(op, rows, d_h, operand, spec->K, static_cast<const uint16_t*>(spec->d_up), spec->K, n, 2 * spec->ff, spec->K, w + p.act,
                               operand, spec->ff))
    return rc;
  rows.row_index = nullptr; rows.row_in = nullptr; rows.w_stride = (int64_t)spec->hidden * spec->ff;
  if (int rc = dh::experts_down(op, rows, w + p.act, operand, spec->ff, static_cast<const uint16_t*>(spec->d_down), spec->ff, spec->hidden, spec->ff,
                                f32(p.y), p.ld_y))
    return rc;
  hipLaunchKernelGGL(experts_combine_kernel, dim3(T, (unsigned)dh::ceil_div(spec->hidden, 1024)), dim3(256), 0, dh::stream(), f32(p.y), (int64_t)p.ld_y,
                     i32(p.slot), spec->top, spec->d_layer_scale, d_x, (int64_t)ld_x, spec->hidden);
  DH_CHECK_LAUNCH(op);
  if (spec->shared_ff) {
    dh::ExpertRows one{};
    one.row_out = f32(p.sg); one.limit = spec->shared_limit;
    if (int rc = dh::experts_glu(op, one, d_h, operand, spec->K, static_cast<const uint16_t*>(spec->d_shared_up), spec->K, T, 2 * spec->shared_ff, spec->K,
                                 w + p.shared_act, operand, spec->shared_ff))
      return rc;
    return dh_dense_matmul_scaled(w + p.shared_act, operand, spec->shared_ff, spec->d_shared_down, spec->shared_ff, T, spec->hidden, spec->shared_ff, 1.f,
                                  nullptr, spec->d_layer_scale, d_x, d_x, ld_x, spec->hidden, nullptr, 0, 0, DH_ACT_NONE);
  }
  return 0;
}

}  // extern "C"
