// Attention over a low-rank latent (dh_latent): a token's cache row is [latent c | rotated key part], one for all heads.
//
//   k_h = [W_uk,h c | k_rot],  v_h = W_uv,h c,  q_h = [unrotated | rotated],  softmax over a sliding window
//
// Prefill expands the visible rows into per-head keys and values with two matrix products and runs the flash kernel on
// them (the rotated part comes straight from the cache rows).  Decode never expands: the query is carried into the latent
// space instead, where all heads share one row per key,
//
//   latent_query_kernel    q'_h = [W_uk,h^T q_h | rotated q_h], 32-bit; also norms, rotates and appends the token's cache row
//   latent_mfma_kernel     16 heads x 64 keys per workgroup and pass: S^T = K Q'^T with the key rows as they lie in memory, Q'
//                          as f16 high part + residual; O'^T = C^T P^T with the latents transposed through LDS and P as high
//                          part + residual.  Key splits as in the other decode attention.
//   latent_plain_kernel    the same for f32 caches and latents of more than 512 elements, on the vector units
//   latent_value_kernel    merges a head's splits and applies W_uv,h
#include <algorithm>
#include <cfloat>

#include "attention_keys.h"
#include "dense_device.h"

namespace {

using dh::DynKeys;
using dh::KeyRange;
using dh::f16x8_t;
using dh::f32x4_t;
using dh::u32x4_t;

constexpr float kLog2e = 1.4426950408889634f;
constexpr int kKeys = 64;            // keys per pass
constexpr int kVRow = kKeys + 8;     // halves per transposed latent row in LDS
// Word of a transposed row that holds a key pair: groups of four words trade places by row, so that lanes that write eight rows
// apart meet different banks; a group (what a fragment read takes) stays whole.
__device__ __forceinline__ int v_word(int row, int pair) { return (row * kVRow >> 1) + (pair ^ (4 * ((row >> 3) & 7))); }

struct LatentArgs {
  float* rows;             // projection rows [T][ld_row]
  void* cache;             // [row][C + R]
  float* q;                // [H][C + R] queries in latent space, scale and log2(e) folded in
  _Float16* q16;           // the same as f16: [H][C + R] high parts, then as many residuals
  float* parts;            // [H][nsplit of the launch][C + 4]: sums, running maximum, running denominator
  float* out;              // [H][VD]
  const uint16_t* uk_t;    // [H][C][D]
  const uint16_t* uv;      // [H][VD][C]
  const float* norm;
  const float* cos;
  const float* sin;
  int64_t ld_row;
  int H, D, R, VD, rank, C, rot_dim, dkv_off;
  int pos0, kbeg, kend, nsplit;
  float scale, eps;
  DynKeys dyn;
};

__device__ __forceinline__ int step_position(const LatentArgs& a) { return a.dyn.kv_len_ptr ? max(0, min((int)*a.dyn.kv_len_ptr, a.dyn.max_kv_len) - 1) : a.pos0; }

// The interleaved pair 2 j, 2 j + 1 of a rotated part, turned.
__device__ __forceinline__ float2 rotated(const LatentArgs& a, const float* x, int64_t pos, int j) {
  const int half = a.rot_dim >> 1;
  if (j >= half) return make_float2(0.f, 0.f);
  const float c = a.cos[pos * half + j], s = a.sin[pos * half + j], u = x[2 * j], v = x[2 * j + 1];
  return make_float2(u * c - v * s, v * c + u * s);
}

// The token's cache row from its raw projection: 256 threads.
template <typename KV>
__device__ void write_cache_row(const LatentArgs& a, const float* raw, int64_t pos, float* red) {
  const int tid = threadIdx.x;
  float ss = 0.f;
  for (int i = tid; i < a.rank; i += 256) ss = fmaf(raw[i], raw[i], ss);
  ss = dh::wave_sum_uniform(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.rank + a.eps);
  KV* row = static_cast<KV*>(a.cache) + pos * (a.C + a.R);
  for (int i = tid; i < a.C; i += 256) row[i] = (KV)(i < a.rank ? raw[i] * inv * a.norm[i] : 0.f);
  for (int j = tid; j < a.R / 2; j += 256) {
    const float2 r = rotated(a, raw + a.C, pos, j);
    row[a.C + 2 * j] = (KV)r.x;
    row[a.C + 2 * j + 1] = (KV)r.y;
  }
}

// A portion: queries rotated in place, cache rows written.  One workgroup per token.
template <typename KV>
__global__ __launch_bounds__(256) void latent_rows_kernel(const LatentArgs a) {
  __shared__ float red[4];
  const int64_t pos = (int64_t)a.pos0 + blockIdx.x;
  float* row = a.rows + (int64_t)blockIdx.x * a.ld_row;
  const int half = a.rot_dim >> 1;
  for (int i = threadIdx.x; i < a.H * half; i += 256) {
    float* x = row + (int64_t)(i / half) * (a.D + a.R) + a.D;
    const int j = i % half;
    const float2 r = rotated(a, x, pos, j);
    x[2 * j] = r.x;
    x[2 * j + 1] = r.y;
  }
  if (a.dkv_off >= 0) write_cache_row<KV>(a, row + a.dkv_off, pos, red);
}

// s + eight bf16 elements times a vector in LDS.
__device__ __forceinline__ float piece_dot(const u32x4_t v, const float* x, float s) {
  const float4 xa = *reinterpret_cast<const float4*>(x), xb = *reinterpret_cast<const float4*>(x + 4);
  s = fmaf(xa.x, dh::bf16_low(v[0]), s); s = fmaf(xa.y, dh::bf16_high(v[0]), s);
  s = fmaf(xa.z, dh::bf16_low(v[1]), s); s = fmaf(xa.w, dh::bf16_high(v[1]), s);
  s = fmaf(xb.x, dh::bf16_low(v[2]), s); s = fmaf(xb.y, dh::bf16_high(v[2]), s);
  s = fmaf(xb.z, dh::bf16_low(v[3]), s); s = fmaf(xb.w, dh::bf16_high(v[3]), s);
  return s;
}

__device__ __forceinline__ void put_query(const LatentArgs& a, int64_t at, float v) {
  a.q[at] = v;
  if (a.q16) {
    const _Float16 hi = (_Float16)v;
    a.q16[at] = hi;
    a.q16[(int64_t)a.H * (a.C + a.R) + at] = (_Float16)(v - (float)hi);
  }
}

// Grid = (slices of 64 latent elements, heads + 1): head h's query carried into the latent space; row H appends the cache row.
template <typename KV, int L>
__global__ __launch_bounds__(256) void latent_query_kernel(const LatentArgs a) {
  __shared__ __align__(16) float qs[512];
  __shared__ float red[4];
  constexpr int ROWS = 64 / L, PASSES = 16 / ROWS;       // L lanes hold a row of D <= 8 L elements
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.y, piece = lane % L;
  const int64_t pos = step_position(a);
  if (h == a.H) {
    if (blockIdx.x == 0 && a.dkv_off >= 0) write_cache_row<KV>(a, a.rows + a.dkv_off, pos, red);
    return;
  }
  u32x4_t w[PASSES];
#pragma unroll
  for (int pass = 0; pass < PASSES; pass++) {
    const int row = 64 * blockIdx.x + (4 * pass + wave) * ROWS + lane / L;      // C is a multiple of 64
    w[pass] = u32x4_t{0u, 0u, 0u, 0u};
    if (8 * piece < a.D) w[pass] = *reinterpret_cast<const u32x4_t*>(a.uk_t + ((int64_t)h * a.C + row) * a.D + 8 * piece);
  }
  const float* q = a.rows + (int64_t)h * (a.D + a.R);
  const float f = a.scale * kLog2e;
  for (int i = tid; i < a.D; i += 256) qs[i] = q[i] * f;
  const int64_t base = (int64_t)h * (a.C + a.R);
  if (blockIdx.x == 0) {
    for (int j = tid; j < a.R / 2; j += 256) {
      const float2 r = rotated(a, q + a.D, pos, j);
      put_query(a, base + a.C + 2 * j, r.x * f);
      put_query(a, base + a.C + 2 * j + 1, r.y * f);
    }
  }
  __syncthreads();
#pragma unroll
  for (int pass = 0; pass < PASSES; pass++) {
    const int row = 64 * blockIdx.x + (4 * pass + wave) * ROWS + lane / L;
    const float s = dh::group_combine<1, L>(8 * piece < a.D ? piece_dot(w[pass], qs + 8 * piece, 0.f) : 0.f, dh::AddOp());
    if (piece == 0) put_query(a, base + row, s);
  }
}

__device__ __forceinline__ KeyRange key_range(const LatentArgs& a) {
  if (a.dyn.kv_len_ptr) return dh::dyn_key_range(a.dyn);
  KeyRange r;
  r.kbeg = a.kbeg; r.kend = a.kend; r.nsplit = a.nsplit; r.start_pos = a.pos0;
  return r;
}

// Grid = (groups of 16 heads, key splits).  NT * 64 >= C latent elements; wave w sums latent tiles w, w + 4, ...
template <int NT>
__global__ __launch_bounds__(256) void latent_mfma_kernel(const LatentArgs a) {
  extern __shared__ __align__(16) _Float16 lds[];
  __shared__ float m_lds[4][16];
  __shared__ float l_lds[4][16];
  const int CR = a.C + a.R, qrow = CR + 8;
  _Float16* q_hi = lds;
  _Float16* q_lo = q_hi + 16 * qrow;
  _Float16* v_lds = q_lo + 16 * qrow;
  _Float16* p_hi = v_lds + a.C * kVRow;
  _Float16* p_lo = p_hi + 16 * kVRow;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, head = lane & 15, g = lane >> 4;
  const int h0 = 16 * blockIdx.x, split = blockIdx.y;
  const KeyRange kr = key_range(a);
  if (split >= kr.nsplit) return;
  const int ntiles = (kr.kend - kr.kbeg + kKeys - 1) / kKeys;
  const _Float16* cache = static_cast<const _Float16*>(a.cache);
  const int64_t residual = (int64_t)a.H * CR;
  // latents to be transposed: key pairs 8 wave + 4 i + (lane >> 4), sixteen neighbouring pieces of a row per group of lanes
  const int piece0 = lane & 15, pair0 = 8 * wave + (lane >> 4);
  constexpr int NP = (NT + 1) / 2;                       // pieces per lane: 16 NP pieces hold C elements
  constexpr int KF = 2 * NT + 2;                         // key fragments in registers: rotated parts of up to 64 elements
  const int steps = CR >> 5;
  u32x4_t v[NP][2][2];
  f16x8_t kf[KF];
  auto key_row = [&](int k0) { return cache + (int64_t)min(k0 + 16 * wave + head, kr.kend - 1) * CR + 8 * g; };
  // a tile's latents by key pairs (to be transposed) and key fragments; keys past the end repeat the last one (their
  // probabilities are zero)
  auto load = [&](int k0) {
    const _Float16* krow = key_row(k0);
#pragma unroll
    for (int s = 0; s < KF; s++)
      if (s < steps) kf[s] = *reinterpret_cast<const f16x8_t*>(krow + 32 * s);
#pragma unroll
    for (int j = 0; j < NP; j++) {
      const int col = 8 * (piece0 + 16 * j);
      if (col >= a.C) continue;
#pragma unroll
      for (int i = 0; i < 2; i++)
#pragma unroll
        for (int s = 0; s < 2; s++)
          v[j][i][s] = *reinterpret_cast<const u32x4_t*>(cache + (int64_t)min(k0 + 2 * (pair0 + 4 * i) + s, kr.kend - 1) * CR + col);
    }
  };
  if (split < ntiles) load(kr.kbeg + split * kKeys);
  for (int i = tid; i < 16 * (CR >> 3); i += 256) {
    const int hh = i / (CR >> 3), p = i % (CR >> 3);
    u32x4_t hi = {0u, 0u, 0u, 0u}, lo = hi;
    if (h0 + hh < a.H) {
      hi = *reinterpret_cast<const u32x4_t*>(a.q16 + (int64_t)(h0 + hh) * CR + 8 * p);
      lo = *reinterpret_cast<const u32x4_t*>(a.q16 + residual + (int64_t)(h0 + hh) * CR + 8 * p);
    }
    *reinterpret_cast<u32x4_t*>(q_hi + hh * qrow + 8 * p) = hi;
    *reinterpret_cast<u32x4_t*>(q_lo + hh * qrow + 8 * p) = lo;
  }
  f32x4_t acc[NT];
#pragma unroll
  for (int t = 0; t < NT; t++) acc[t] = {0.f, 0.f, 0.f, 0.f};
  float m_run = -FLT_MAX, l_run = 0.f;
  __syncthreads();
  for (int c = split; c < ntiles; c += kr.nsplit) {
    const int k0 = kr.kbeg + c * kKeys;
    f32x4_t st = {0.f, 0.f, 0.f, 0.f};
    auto score = [&](const f16x8_t& ka, int s) {
      st = __builtin_amdgcn_mfma_f32_16x16x32_f16(ka, *reinterpret_cast<const f16x8_t*>(q_hi + head * qrow + 32 * s + 8 * g), st, 0, 0, 0);
      st = __builtin_amdgcn_mfma_f32_16x16x32_f16(ka, *reinterpret_cast<const f16x8_t*>(q_lo + head * qrow + 32 * s + 8 * g), st, 0, 0, 0);
    };
#pragma unroll
    for (int s = 0; s < KF; s++)
      if (s < steps) score(kf[s], s);
    for (int s = KF; s < steps; s++) score(*reinterpret_cast<const f16x8_t*>(key_row(k0) + 32 * s), s);
    // this lane: head `head`, keys k0 + 16 wave + 4 g + i
    float mx = -FLT_MAX;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      if (k0 + 16 * wave + 4 * g + i >= kr.kend) st[i] = -INFINITY;
      mx = fmaxf(mx, st[i]);
    }
    mx = dh::group_combine<16, 64>(mx, dh::MaxOp());
    if (g == 0) m_lds[wave][head] = mx;
#pragma unroll
    for (int j = 0; j < NP; j++) {
      const int col = 8 * (piece0 + 16 * j);
      if (col >= a.C) continue;
#pragma unroll
      for (int i = 0; i < 2; i++)
#pragma unroll
        for (int e = 0; e < 8; e++) {
          const uint32_t word = __builtin_amdgcn_perm(v[j][i][1][e >> 1], v[j][i][0][e >> 1], (e & 1) ? 0x07060302u : 0x05040100u);
          reinterpret_cast<uint32_t*>(v_lds)[v_word(col + e, pair0 + 4 * i)] = word;
        }
    }
    if (c + kr.nsplit < ntiles) load(k0 + kr.nsplit * kKeys);
    __syncthreads();
    const float m_new = fmaxf(m_run, fmaxf(fmaxf(m_lds[0][head], m_lds[1][head]), fmaxf(m_lds[2][head], m_lds[3][head])));
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    l_run *= alpha;
    _Float16 ph[4], pl[4];
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const float p = __builtin_amdgcn_exp2f(st[i] - m_new);
      l_run += p;
      ph[i] = (_Float16)p;
      pl[i] = (_Float16)(p - (float)ph[i]);
    }
    const int at = head * kVRow + 16 * wave + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      p_hi[at + i] = ph[i];
      p_lo[at + i] = pl[i];
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < NT; t++) {
      const int tile = wave + 4 * t;
      if (16 * tile >= a.C) break;
      acc[t] *= alpha;
#pragma unroll
      for (int kb = 0; kb < 2; kb++) {
        const f16x8_t va = *reinterpret_cast<const f16x8_t*>(reinterpret_cast<const uint32_t*>(v_lds) + v_word(16 * tile + head, 16 * kb + 4 * g));
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_f16(va, *reinterpret_cast<const f16x8_t*>(p_hi + head * kVRow + 32 * kb + 8 * g), acc[t], 0, 0, 0);
        acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_f16(va, *reinterpret_cast<const f16x8_t*>(p_lo + head * kVRow + 32 * kb + 8 * g), acc[t], 0, 0, 0);
      }
    }
    __syncthreads();
  }
  l_run = dh::group_combine<16, 64>(l_run, dh::AddOp());
  if (g == 0) l_lds[wave][head] = l_run;
  __syncthreads();
  if (h0 + head >= a.H) return;
  float* part = a.parts + ((int64_t)(h0 + head) * a.nsplit + split) * (a.C + 4);
#pragma unroll
  for (int t = 0; t < NT; t++) {
    const int tile = wave + 4 * t;
    if (16 * tile >= a.C) break;
    *reinterpret_cast<f32x4_t*>(part + 16 * tile + 4 * g) = acc[t];
  }
  if (wave == 0 && g == 0) {
    part[a.C] = m_run;
    part[a.C + 1] = l_lds[0][head] + l_lds[1][head] + l_lds[2][head] + l_lds[3][head];
  }
}

// Grid = (heads, key splits); four threads per key for the scores, one thread per latent element (and 256 more) for the sums.
template <typename KV>
__global__ __launch_bounds__(256) void latent_plain_kernel(const LatentArgs a) {
  extern __shared__ __align__(16) float fl[];
  __shared__ float p_lds[kKeys];
  __shared__ float red[4];
  const int CR = a.C + a.R, tid = threadIdx.x, h = blockIdx.x, split = blockIdx.y;
  const KeyRange kr = key_range(a);
  if (split >= kr.nsplit) return;
  const int ntiles = (kr.kend - kr.kbeg + kKeys - 1) / kKeys;
  const KV* cache = static_cast<const KV*>(a.cache);
  float* q = fl;                                         // [CR]
  float* sum = fl + CR;                                  // [C]
  for (int i = tid; i < CR; i += 256) q[i] = a.q[(int64_t)h * CR + i];
  for (int i = tid; i < a.C; i += 256) sum[i] = 0.f;
  float m_run = -FLT_MAX, l_run = 0.f;
  __syncthreads();
  for (int c = split; c < ntiles; c += kr.nsplit) {
    const int k0 = kr.kbeg + c * kKeys, key = k0 + (tid >> 2), live = min(kKeys, kr.kend - k0);
    float s = 0.f;
    const KV* row = cache + (int64_t)min(key, kr.kend - 1) * CR;
    for (int i = 4 * (tid & 3); i < CR; i += 16) {
#pragma unroll
      for (int e = 0; e < 4; e++) s = fmaf(q[i + e], (float)row[i + e], s);
    }
    s = dh::group_combine<1, 4>(s, dh::AddOp());
    if (key >= kr.kend) s = -INFINITY;
    float mx = dh::group_combine<4, 64>(s, dh::MaxOp());
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    const float m_new = fmaxf(m_run, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
    m_run = m_new;
    if ((tid & 3) == 0) p_lds[tid >> 2] = __builtin_amdgcn_exp2f(s - m_new);
    __syncthreads();
    float l = 0.f;
    for (int k = 0; k < live; k++) l += p_lds[k];
    l_run = l_run * alpha + l;
    for (int i = tid; i < a.C; i += 256) {
      float v = sum[i] * alpha;
      for (int k = 0; k < live; k++) v = fmaf(p_lds[k], (float)cache[(int64_t)(k0 + k) * CR + i], v);
      sum[i] = v;
    }
    __syncthreads();
  }
  float* part = a.parts + ((int64_t)h * a.nsplit + split) * (a.C + 4);
  for (int i = tid; i < a.C; i += 256) part[i] = sum[i];
  if (tid == 0) {
    part[a.C] = m_run;
    part[a.C + 1] = l_run;
  }
}

// Grid = (slices of 32 value elements, heads).  The slice's weights are requested first and travel while the splits are merged.
template <int L, bool LONG>
__global__ __launch_bounds__(256) void latent_value_kernel(const LatentArgs a) {
  extern __shared__ __align__(16) float fl[];            // [C] the head's latent, [splits] factors
  __shared__ float4 sums[256];
  float* o = fl;
  float* f = fl + a.C;
  constexpr int ROWS = 64 / L, PASSES = 8 / ROWS;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.y, piece = lane % L;
  auto weights = [&](int pass) {
    const int row = 32 * blockIdx.x + (4 * pass + wave) * ROWS + lane / L;
    return a.uv + ((int64_t)h * a.VD + min(row, a.VD - 1)) * a.C;
  };
  u32x4_t w[PASSES];
#pragma unroll
  for (int pass = 0; pass < PASSES; pass++) {
    w[pass] = u32x4_t{0u, 0u, 0u, 0u};
    if (8 * piece < a.C) w[pass] = *reinterpret_cast<const u32x4_t*>(weights(pass) + 8 * piece);
  }
  const int nsplit = key_range(a).nsplit, stride = a.C + 4;
  const float* base = a.parts + (int64_t)h * a.nsplit * stride;
  // four latent elements per thread, the splits dealt to the groups of C / 4 threads; the first ones of a thread are requested here
  constexpr int AHEAD = 8;
  const int cols = a.C >> 2, groups = LONG ? 1 : 256 / cols, group = LONG ? 0 : tid / cols, col = 4 * (LONG ? tid : tid % cols);
  float4 part[AHEAD];
  if (!LONG && group < groups) {
#pragma unroll
    for (int k = 0; k < AHEAD; k++)
      if (group + groups * k < nsplit) part[k] = *reinterpret_cast<const float4*>(base + (int64_t)(group + groups * k) * stride + col);
  }
  // every wave finds the common maximum and denominator by itself
  float M = -FLT_MAX;
  for (int s = lane; s < nsplit; s += 64) M = fmaxf(M, base[(int64_t)s * stride + a.C]);
  M = dh::group_combine<1, 64>(M, dh::MaxOp());
  float den = 0.f;
  for (int s = lane; s < nsplit; s += 64) {
    const float e = __builtin_amdgcn_exp2f(base[(int64_t)s * stride + a.C] - M);
    if (wave == 0) f[s] = e;
    den = fmaf(e, base[(int64_t)s * stride + a.C + 1], den);
  }
  den = dh::wave_sum_uniform(den);
  const float inv = den > 0.f ? 1.0f / den : 0.f;
  __syncthreads();
  if (LONG) {
    for (int i = tid; i < a.C; i += 256) {
      float v = 0.f;
#pragma unroll 8
      for (int s = 0; s < nsplit; s++) v = fmaf(f[s], base[(int64_t)s * stride + i], v);
      o[i] = v * inv;
    }
  } else {
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    auto add = [&](const float4& p, float e) {
      v.x = fmaf(e, p.x, v.x); v.y = fmaf(e, p.y, v.y); v.z = fmaf(e, p.z, v.z); v.w = fmaf(e, p.w, v.w);
    };
    if (group < groups) {
#pragma unroll
      for (int k = 0; k < AHEAD; k++)
        if (group + groups * k < nsplit) add(part[k], f[group + groups * k]);
      for (int s = group + groups * AHEAD; s < nsplit; s += groups) add(*reinterpret_cast<const float4*>(base + (int64_t)s * stride + col), f[s]);
      sums[tid] = make_float4(v.x * inv, v.y * inv, v.z * inv, v.w * inv);
    }
    __syncthreads();
    if (tid < cols) {
      float4 t = sums[tid];
      for (int k = 1; k < groups; k++) {
        const float4 u = sums[tid + k * cols];
        t.x += u.x; t.y += u.y; t.z += u.z; t.w += u.w;
      }
      *reinterpret_cast<float4*>(o + 4 * tid) = t;
    }
  }
  __syncthreads();
#pragma unroll
  for (int pass = 0; pass < PASSES; pass++) {
    const int row = 32 * blockIdx.x + (4 * pass + wave) * ROWS + lane / L;
    float s = 8 * piece < a.C ? piece_dot(w[pass], o + 8 * piece, 0.f) : 0.f;
    if (LONG) {
      for (int p = piece + L; p < (a.C >> 3); p += L) s = piece_dot(*reinterpret_cast<const u32x4_t*>(weights(pass) + 8 * p), o + 8 * p, s);
    }
    s = dh::group_combine<1, L>(s, dh::AddOp());
    if (piece == 0 && row < a.VD) a.out[(int64_t)h * a.VD + row] = s;
  }
}

int check(const char* op, const dh_latent* s) {
  if (!s) return dh::fail(1, "[%s] null spec", op);
  if (s->H <= 0 || s->D <= 0 || s->D % 8 || s->VD <= 0 || s->VD % 8 || s->R <= 0 || s->R % 32 || s->D + s->R > 512 || s->VD > 512)
    return dh::fail(1, "[%s] head parts must be multiples of 8 (rotated: of 32), 512 in all: heads %d, own %d, rotated %d, values %d", op, s->H, s->D, s->R, s->VD);
  if (s->rank <= 0 || s->rank > s->C || s->C % 64) return dh::fail(1, "[%s] latent of %d elements in rows of %d (a multiple of 64)", op, s->rank, s->C);
  if (s->rot_dim < 0 || s->rot_dim % 2 || s->rot_dim > s->R) return dh::fail(1, "[%s] rot_dim=%d must be even and fit %d elements", op, s->rot_dim, s->R);
  if (s->window < 0) return dh::fail(1, "[%s] window must be non-negative", op);
  if (s->cache_dtype != DH_F16 && s->cache_dtype != DH_F32) return dh::fail(1, "[%s] caches must be f16 or f32, got dtype %d", op, s->cache_dtype);
  const int64_t q = (int64_t)s->H * (s->D + s->R);
  if (s->ld_row % 4 || s->ld_row < q || (s->dkv_offset >= 0 && (s->dkv_offset % 4 || s->dkv_offset < q || s->ld_row < s->dkv_offset + s->C + s->R)))
    return dh::fail(1, "[%s] a projection row of %d floats does not hold its parts", op, s->ld_row);
  if (!s->d_cos || !s->d_sin || !s->d_uk || !s->d_uv || !s->d_uk_t || !s->d_uv_rows || (s->dkv_offset >= 0 && !s->d_latent_norm)) return dh::fail(1, "[%s] null pointer in the spec", op);
  if ((reinterpret_cast<uintptr_t>(s->d_uk) | reinterpret_cast<uintptr_t>(s->d_uv) | reinterpret_cast<uintptr_t>(s->d_uk_t) |
       reinterpret_cast<uintptr_t>(s->d_uv_rows)) & 15)
    return dh::fail(1, "[%s] weights must be 16-byte aligned", op);
  return 0;
}

LatentArgs make_args(const dh_latent* s, const float* rows, void* cache) {
  LatentArgs a{};
  a.rows = const_cast<float*>(rows); a.cache = cache;
  a.uk_t = static_cast<const uint16_t*>(s->d_uk_t); a.uv = static_cast<const uint16_t*>(s->d_uv_rows);
  a.norm = s->d_latent_norm; a.cos = s->d_cos; a.sin = s->d_sin;
  a.ld_row = s->ld_row;
  a.H = s->H; a.D = s->D; a.R = s->R; a.VD = s->VD; a.rank = s->rank; a.C = s->C; a.rot_dim = s->rot_dim; a.dkv_off = s->dkv_offset;
  a.scale = s->scale; a.eps = s->eps;
  return a;
}

bool on_matrix_cores(const dh_latent* s) { return s->cache_dtype == DH_F16 && s->C <= 512; }
int one_per_cu(const dh_latent* s) { return dh::attn_one_per_cu(dh::num_cus(), on_matrix_cores(s) ? (int)dh::ceil_div(s->H, 16) : s->H); }
size_t up256(size_t n) { return (n + 255) / 256 * 256; }
size_t query_bytes(const dh_latent* s) { return up256((size_t)s->H * (s->C + s->R) * 8); }     // f32 and two f16 copies
size_t expanded_bytes(const dh_latent* s, int64_t keys, int size) { return up256((size_t)keys * s->H * size * (s->cache_dtype == DH_F16 ? 2 : 4)); }

template <int NT>
int launch_mfma(const char* op, const LatentArgs& a, dim3 grid) {
  auto kern = latent_mfma_kernel<NT>;
  static bool attr_set = false;
  if (!attr_set) {
    DH_CHECK_HIP(op, hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
    attr_set = true;
  }
  const size_t lds = ((size_t)32 * (a.C + a.R + 8) + (size_t)a.C * kVRow + 32 * kVRow) * 2;
  if (lds > 150 * 1024) return dh::fail(1, "[%s] %zu bytes of LDS are needed", op, lds);
  hipLaunchKernelGGL(kern, grid, dim3(256), lds, dh::stream(), a);
  return 0;
}
template <typename KV>
void launch_query(const LatentArgs& a, dim3 grid) {
  if (a.D <= 64) hipLaunchKernelGGL((latent_query_kernel<KV, 8>), grid, dim3(256), 0, dh::stream(), a);
  else if (a.D <= 128) hipLaunchKernelGGL((latent_query_kernel<KV, 16>), grid, dim3(256), 0, dh::stream(), a);
  else hipLaunchKernelGGL((latent_query_kernel<KV, 64>), grid, dim3(256), 0, dh::stream(), a);
}

}  // namespace

extern "C" {

int dh_latent_rows(const dh_latent* spec, float* d_rows, void* d_cache, int T, int start_pos) {
  const char* op = "dh_latent_rows";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (T <= 0 || start_pos < 0) return dh::fail(1, "[%s] seqLen must be positive and startPos non-negative", op);
  if (!d_rows || !d_cache) return dh::fail(1, "[%s] null pointer", op);
  LatentArgs a = make_args(spec, d_rows, d_cache);
  a.pos0 = start_pos;
  if (spec->cache_dtype == DH_F16) hipLaunchKernelGGL(latent_rows_kernel<_Float16>, dim3(T), dim3(256), 0, dh::stream(), a);
  else hipLaunchKernelGGL(latent_rows_kernel<float>, dim3(T), dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  return 0;
}

size_t dh_latent_prefill_workspace_bytes(const dh_latent* s, int T, int start_pos) {
  if (!s || T <= 0 || start_pos < 0) return 256;
  const int64_t first = s->window > 0 ? std::max(0, start_pos - s->window + 1) : 0, keys = start_pos + T - first;
  return expanded_bytes(s, keys, s->D) + expanded_bytes(s, keys, s->VD);
}

int dh_latent_prefill(const dh_latent* spec, const float* d_rows, const void* d_cache, void* d_workspace, void* d_out, int out_dtype,
                      int ld_out, int T, int start_pos) {
  const char* op = "dh_latent_prefill";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (T <= 0 || start_pos < 0) return dh::fail(1, "[%s] seqLen must be positive and startPos non-negative", op);
  if (!d_rows || !d_cache || !d_workspace || !d_out) return dh::fail(1, "[%s] null pointer", op);
  const bool half = spec->cache_dtype == DH_F16;
  const int first = spec->window > 0 ? std::max(0, start_pos - spec->window + 1) : 0, keys = start_pos + T - first;
  const int CR = spec->C + spec->R, nk = spec->H * spec->D, nv = spec->H * spec->VD;
  const char* rows = static_cast<const char*>(d_cache) + (size_t)first * CR * (half ? 2 : 4);
  void* K = d_workspace;
  void* V = static_cast<char*>(d_workspace) + expanded_bytes(spec, keys, spec->D);
  for (int i = 0; i < 2; i++) {
    const void* w = i ? spec->d_uv : spec->d_uk;
    const int n = i ? nv : nk;
    void* out = i ? V : K;
    const int rc = half ? dh_dense_matmul(rows, DH_F16, CR, w, spec->C, keys, n, spec->C, 1.f, nullptr, nullptr, nullptr, 0, 0, out, DH_F16, n, DH_ACT_NONE)
                        : dh_dense_matmul(rows, DH_F32, CR, w, spec->C, keys, n, spec->C, 1.f, nullptr, nullptr, static_cast<float*>(out), n, n, nullptr, 0, 0, DH_ACT_NONE);
    if (rc) return rc;
  }
  dh_attn_spec s{};
  s.H = s.Hkv = spec->H; s.D = spec->D; s.VD = s.value_dim = spec->VD; s.window = spec->window; s.cache_dtype = spec->cache_dtype;
  s.gate_offset = -1; s.ld_qkv = spec->ld_row; s.scale = spec->scale;
  if (s.ld_qkv < nv) return dh::fail(1, "[%s] a projection row of %d floats is shorter than the values", op, s.ld_qkv);
  return dh_attn_spec_prefill_shared(&s, d_rows, K, rows + (size_t)spec->C * (half ? 2 : 4), spec->R, CR, V, d_out, out_dtype, ld_out, T,
                                     start_pos - first);
}

size_t dh_latent_decode_workspace_bytes(const dh_latent* s, int max_kv_len) {
  if (!s || max_kv_len <= 0) return 256;
  const size_t splits = std::min<size_t>((size_t)dh::ceil_div(max_kv_len, dh::kAttnTileKeys), 1024);
  return query_bytes(s) + up256((size_t)s->H * splits * (s->C + 4) * sizeof(float));
}

int dh_latent_decode(const dh_latent* spec, const float* d_row, void* d_cache, float* d_out, int pos, const uint32_t* d_kv_len,
                     int max_kv_len, void* d_workspace) {
  const char* op = "dh_latent_decode";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (pos < 0) return dh::fail(1, "[%s] the position must be non-negative", op);
  if (d_kv_len && max_kv_len <= 0) return dh::fail(1, "[%s] max_kv_len must be positive with the key count on the device", op);
  if (!d_row || !d_cache || !d_out || !d_workspace) return dh::fail(1, "[%s] null pointer", op);
  if ((reinterpret_cast<uintptr_t>(d_row) | reinterpret_cast<uintptr_t>(d_cache) | reinterpret_cast<uintptr_t>(d_workspace)) & 15)
    return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  LatentArgs a = make_args(spec, d_row, d_cache);
  const bool mfma = on_matrix_cores(spec);
  a.q = static_cast<float*>(d_workspace);
  a.q16 = mfma ? reinterpret_cast<_Float16*>(a.q + (size_t)spec->H * (spec->C + spec->R)) : nullptr;
  a.parts = reinterpret_cast<float*>(static_cast<char*>(d_workspace) + query_bytes(spec));
  a.out = d_out; a.pos0 = pos;
  const int per_cu = one_per_cu(spec);
  if (d_kv_len) {
    a.dyn.kv_len_ptr = d_kv_len; a.dyn.max_kv_len = max_kv_len; a.dyn.causal = 1; a.dyn.start_pos = -1;
    a.dyn.sliding_window = spec->window; a.dyn.kv_start = 0; a.dyn.qkv = 1; a.dyn.one_per_cu = per_cu;
    a.nsplit = dh::max_splits_upto(per_cu, spec->window > 0 ? std::min(max_kv_len, spec->window) : max_kv_len);
  } else {
    a.kend = pos + 1;
    a.kbeg = spec->window > 0 ? std::max(0, pos - spec->window + 1) : 0;
    a.nsplit = dh::splits_for(per_cu, a.kend - a.kbeg);
  }
  const dim3 qgrid((unsigned)(spec->C / 64), (unsigned)spec->H + 1);
  if (spec->cache_dtype == DH_F16) launch_query<_Float16>(a, qgrid);
  else launch_query<float>(a, qgrid);
  DH_CHECK_LAUNCH(op);
  if (mfma) {
    const dim3 grid((unsigned)dh::ceil_div(spec->H, 16), (unsigned)a.nsplit);
    const int rc = spec->C <= 64 ? launch_mfma<1>(op, a, grid) : spec->C <= 128 ? launch_mfma<2>(op, a, grid)
                   : spec->C <= 256 ? launch_mfma<4>(op, a, grid) : launch_mfma<8>(op, a, grid);
    if (rc) return rc;
  } else {
    const dim3 grid((unsigned)spec->H, (unsigned)a.nsplit);
    const size_t lds = (size_t)(2 * spec->C + spec->R) * sizeof(float);
    if (lds > 60 * 1024) return dh::fail(1, "[%s] a latent of %d elements is not served", op, spec->rank);
    if (spec->cache_dtype == DH_F16) hipLaunchKernelGGL(latent_plain_kernel<_Float16>, grid, dim3(256), lds, dh::stream(), a);
    else hipLaunchKernelGGL(latent_plain_kernel<float>, grid, dim3(256), lds, dh::stream(), a);
  }
  DH_CHECK_LAUNCH(op);
  const dim3 vgrid((unsigned)dh::ceil_div(spec->VD, 32), (unsigned)spec->H);
  const size_t lds = (size_t)(spec->C + a.nsplit) * sizeof(float);
  if (spec->C <= 64) hipLaunchKernelGGL((latent_value_kernel<8, false>), vgrid, dim3(256), lds, dh::stream(), a);
  else if (spec->C <= 128) hipLaunchKernelGGL((latent_value_kernel<16, false>), vgrid, dim3(256), lds, dh::stream(), a);
  else if (spec->C <= 512) hipLaunchKernelGGL((latent_value_kernel<64, false>), vgrid, dim3(256), lds, dh::stream(), a);
  else hipLaunchKernelGGL((latent_value_kernel<64, true>), vgrid, dim3(256), lds, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  return 0;
}

}  // extern "C"
