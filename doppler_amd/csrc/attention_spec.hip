// Attention with a logarithmic distance bias, a sliding window, normed values, an output gate and key and value heads
// of different sizes (dh_attn_spec): decode steps, and prefill for what the matrix-core kernel
// (attention_prefill.hip) does not serve (f32 caches, heads of more than 128 elements).
//
// attn_spec_kernel: grid = (kv head x query-head group, key split, query token), four waves.  Keys advance in chunks;
// every wave takes its own keys of a chunk and keeps its own online-softmax state, so the loop has no barrier.
// L lanes share a key: lane (slot, piece) holds elements 8 piece .. 8 piece + 7 of its key's row and of its value
// row.  Scores are f32 dot products summed over the L lanes with DPP steps, so the lane that multiplies a value piece
// already holds its key's probability.  Partial results meet in LDS at the end: slots, then waves.
//
// A decode step's key and value come raw from its projection row: every workgroup norms and rounds them as the
// cache would hold them, uses them in place of the (not yet written) cache row, and the workgroup that owns the
// last chunk appends them.
#include <algorithm>
#include <cfloat>

#include "attention_keys.h"
#include "attention_spec.h"
#include "dense_device.h"

namespace {

using dh::DynKeys;
using dh::KeyRange;

constexpr float kLog2e = 1.4426950408889634f;

struct SpecArgs {
  const float* qkv;     // projection rows [T][ld_qkv]
  void* K;
  void* V;
  float* O;             // f32 output rows (or null)
  uint16_t* O16;        // bf16 output rows
  float* ws;            // [H][nsplit of the launch][VD + 2]
  int64_t ld_qkv, ld_out;
  int H, Hkv, G, D, VD, value_dim;      // D: key elements of a head, its own and the shared ones
  int own_d;                            // its own
  const void* KS;                       // rows of the shared ones, ld_shared apart
  int64_t ld_shared;
  int k_off, v_off, gate_off;
  int pos0;             // position of the first query token
  int window, kbeg, kend, nsplit;
  int append, value_norm, direct;
  float scale, value_eps;
  const float* r1;
  const float* r2;
  DynKeys dyn;
};

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

// Eight elements as the cache holds them, widened.
template <typename KV>
struct Piece;
template <>
struct Piece<__half> {
  dh::f16x8_t h;
  __device__ __forceinline__ void load(const __half* p) { h = *reinterpret_cast<const dh::f16x8_t*>(p); }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int i = 0; i < 8; i++) h[i] = (_Float16)0.f;
  }
  __device__ __forceinline__ void set(const float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 8; i++) h[i] = (_Float16)v[i];
  }
  __device__ __forceinline__ float get(int i) const { return (float)h[i]; }
  __device__ __forceinline__ void store(__half* p) const { *reinterpret_cast<dh::f16x8_t*>(p) = h; }
};
template <>
struct Piece<float> {
  float f[8];
  __device__ __forceinline__ void load(const float* p) {
    const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
    f[0] = a.x; f[1] = a.y; f[2] = a.z; f[3] = a.w; f[4] = b.x; f[5] = b.y; f[6] = b.z; f[7] = b.w;
  }
  __device__ __forceinline__ void zero() {
#pragma unroll
    for (int i = 0; i < 8; i++) f[i] = 0.f;
  }
  __device__ __forceinline__ void set(const float (&v)[8]) {
#pragma unroll
    for (int i = 0; i < 8; i++) f[i] = v[i];
  }
  __device__ __forceinline__ float get(int i) const { return f[i]; }
  __device__ __forceinline__ void store(float* p) const {
    reinterpret_cast<float4*>(p)[0] = make_float4(f[0], f[1], f[2], f[3]);
    reinterpret_cast<float4*>(p)[1] = make_float4(f[4], f[5], f[6], f[7]);
  }
};

__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
  const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}

// The value row's factor 1 / rms: the L lanes of a group hold its pieces (zeros past VD).
template <int L>
__device__ __forceinline__ float value_factor(const float (&v)[8], int value_dim, float eps) {
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < 8; i++) ss = fmaf(v[i], v[i], ss);
  ss = dh::group_combine<1, L>(ss, dh::AddOp());
  return 1.0f / sqrtf(ss / (float)value_dim + eps);
}

template <typename KV, int L, int GT>
__global__ __launch_bounds__(256) void attn_spec_kernel(const SpecArgs a_in) {
  SpecArgs a = a_in;
  constexpr int SLOTS = 64 / L;                        // keys a wave handles per pass
  constexpr int NP = L >= 16 ? 4 : L / 4;              // passes per chunk
  constexpr int WK = SLOTS * NP;                       // keys per wave and chunk
  constexpr int CH = 4 * WK;                           // keys per chunk
  __shared__ float o_lds[4][GT][8 * L];
  __shared__ float ml_lds[4][GT][2];

  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int slot = lane / L, piece = lane % L;
  const int groups = (a.G + GT - 1) / GT;
  const int kvh = blockIdx.x / groups, hg = blockIdx.x % groups;
  const int h0 = kvh * a.G + hg * GT, gn = min(GT, a.G - hg * GT);
  const int split = blockIdx.y, t = blockIdx.z;
  const int ws_stride = a.nsplit;
  int pos = a.pos0 + t, kbeg = a.kbeg, kend = a.kend, nsplit = a.nsplit;
  if (a.dyn.kv_len_ptr != nullptr) {
    const KeyRange r = dh::dyn_key_range(a.dyn);
    if (split >= r.nsplit) return;                     // surplus workgroups of the largest key count
    pos = r.start_pos; kbeg = r.kbeg; kend = r.kend; nsplit = r.nsplit;
  } else if (!a.append) {
    kend = pos + 1;                                    // every query token has its own key range
    kbeg = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  }
  const float* row = a.qkv + (int64_t)t * a.ld_qkv;
  const bool own = 8 * piece < a.own_d;
  const KV* Kc = own ? static_cast<const KV*>(a.K) + (int64_t)kvh * a.own_d + 8 * piece : static_cast<const KV*>(a.KS) + 8 * piece - a.own_d;
  const KV* Vc = static_cast<const KV*>(a.V) + (int64_t)kvh * a.VD + 8 * piece;
  const int64_t kstride = own ? (int64_t)a.Hkv * a.own_d : a.ld_shared, vstride = (int64_t)a.Hkv * a.VD;
  const bool has_k = 8 * piece < a.D, has_v = 8 * piece < a.VD;
  const int nchunks = (kend - kbeg + CH - 1) / CH;

  Piece<KV> kn[NP], vn[NP], knew, vnew;
  auto load = [&](int c) {
#pragma unroll
    for (int n = 0; n < NP; n++) {
      // keys past the end repeat the last one; the appended one is not in the cache yet
      const int key = min(kbeg + c * CH + wave * WK + n * SLOTS + slot, kend - 1 - a.append);
      kn[n].zero();
      vn[n].zero();
      if (key >= kbeg) {
        if (has_k) kn[n].load(Kc + key * kstride);
        if (has_v) vn[n].load(Vc + key * vstride);
      }
    }
  };
  if (split < nchunks) load(split);

  // ---- query pieces, scale and log2(e) folded in; heads past the group read nothing and score zero
  float q[GT][8], r1[GT], r2[GT];
#pragma unroll
  for (int g = 0; g < GT; g++) {
#pragma unroll
    for (int i = 0; i < 8; i++) q[g][i] = 0.f;
    r1[g] = r2[g] = 0.f;
    if (g < gn) {
      if (has_k) load8(row + (int64_t)(h0 + g) * a.D + 8 * piece, q[g]);
      if (a.r1) {
        r1[g] = a.r1[h0 + g];
        r2[g] = a.r2[h0 + g];
      }
    }
#pragma unroll
    for (int i = 0; i < 8; i++) q[g][i] *= a.scale * kLog2e;
  }
  if (a.append) {
    float kv[8] = {}, vv[8] = {};
    if (has_k) load8(row + a.k_off + (int64_t)kvh * a.D + 8 * piece, kv);
    if (has_v) load8(row + a.v_off + (int64_t)kvh * a.VD + 8 * piece, vv);
    if (a.value_norm) {
      const float f = value_factor<L>(vv, a.value_dim, a.value_eps);
#pragma unroll
      for (int i = 0; i < 8; i++) vv[i] *= f;
    }
    knew.set(kv);
    vnew.set(vv);
    if (split == (nchunks - 1) % nsplit && hg == 0 && wave == 0 && slot == 0) {
      if (has_k) knew.store(static_cast<KV*>(a.K) + (int64_t)kvh * a.D + 8 * piece + pos * kstride);
      if (has_v) vnew.store(static_cast<KV*>(a.V) + (int64_t)kvh * a.VD + 8 * piece + pos * vstride);
    }
  }

  float m[GT], l[GT], acc[GT][8];
#pragma unroll
  for (int g = 0; g < GT; g++) {
    m[g] = -FLT_MAX;
    l[g] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; i++) acc[g][i] = 0.f;
  }
  for (int c = split; c < nchunks; c += nsplit) {
    Piece<KV> kf[NP], vf[NP];
    float s[GT][NP];
#pragma unroll
    for (int n = 0; n < NP; n++) {
      kf[n] = kn[n];
      vf[n] = vn[n];
    }
    if (c + nsplit < nchunks) load(c + nsplit);
    if (kbeg + c * CH + wave * WK >= kend) continue;   // wave-uniform: none of this wave's keys exist
#pragma unroll
    for (int n = 0; n < NP; n++) {
      const int key = kbeg + c * CH + wave * WK + n * SLOTS + slot;
      if (a.append && key == pos) {
        kf[n] = knew;
        vf[n] = vnew;
      }
      const float dist = (float)(pos - key);
#pragma unroll
      for (int g = 0; g < GT; g++) {
        float d = 0.f;
#pragma unroll
        for (int i = 0; i < 8; i++) d = fmaf(q[g][i], kf[n].get(i), d);
        d = dh::group_combine<1, L>(d, dh::AddOp());
        // in units of log2(e): r1 ln(1 + r2 x) log2(e) = r1 log2(1 + r2 x)
        if (a.r1) d = fmaf(-r1[g], __builtin_amdgcn_logf(fmaf(r2[g], dist, 1.0f)), d);
        s[g][n] = key < kend ? d : -INFINITY;
      }
    }
#pragma unroll
    for (int g = 0; g < GT; g++) {
      float mx = s[g][0];
#pragma unroll
      for (int n = 1; n < NP; n++) mx = fmaxf(mx, s[g][n]);
      mx = dh::group_combine<L, 64>(mx, dh::MaxOp());
      const float m_new = fmaxf(m[g], mx);
      const float alpha = __builtin_amdgcn_exp2f(m[g] - m_new);
      m[g] = m_new;
      l[g] *= alpha;
#pragma unroll
      for (int i = 0; i < 8; i++) acc[g][i] *= alpha;
#pragma unroll
      for (int n = 0; n < NP; n++) {
        const float p = __builtin_amdgcn_exp2f(s[g][n] - m_new);
        l[g] += p;
#pragma unroll
        for (int i = 0; i < 8; i++) acc[g][i] = fmaf(p, vf[n].get(i), acc[g][i]);
      }
    }
  }

  // ---- slots meet by lane steps, waves in LDS
#pragma unroll
  for (int g = 0; g < GT; g++) {
    l[g] = dh::group_combine<L, 64>(l[g], dh::AddOp());
#pragma unroll
    for (int i = 0; i < 8; i++) {
      // the mirrors reverse the pieces of a row: they serve uniform groups only, so pieces are added lane by lane
      float v = acc[g][i];
#pragma unroll
      for (int off = L; off < 64; off <<= 1) v += __shfl_xor(v, off, 64);
      if (slot == 0) o_lds[wave][g][8 * piece + i] = v;
    }
    if (lane == 0) {
      ml_lds[wave][g][0] = m[g];
      ml_lds[wave][g][1] = l[g];
    }
  }
  __syncthreads();
  for (int o = tid; o < gn * a.VD; o += 256) {
    const int g = o / a.VD, d = o - g * a.VD, h = h0 + g;
    float M = ml_lds[0][g][0];
#pragma unroll
    for (int w = 1; w < 4; w++) M = fmaxf(M, ml_lds[w][g][0]);
    float num = 0.f, den = 0.f;
#pragma unroll
    for (int w = 0; w < 4; w++) {
      const float f = __builtin_amdgcn_exp2f(ml_lds[w][g][0] - M);
      num = fmaf(f, o_lds[w][g][d], num);
      den = fmaf(f, ml_lds[w][g][1], den);
    }
    if (a.direct) {
      float y = den > 0.f ? num / den : 0.f;
      if (a.gate_off >= 0) y *= sigmoid_f(row[a.gate_off + h]);
      const int64_t at = (int64_t)t * a.ld_out + (int64_t)h * a.VD + d;
      if (a.O16) a.O16[at] = dh::f32_to_bf16_bits(y);
      else a.O[at] = y;
    } else {
      float* w = a.ws + ((int64_t)h * ws_stride + split) * (a.VD + 2);
      w[d] = num;
      if (d == 0) {
        w[a.VD] = M;
        w[a.VD + 1] = den;
      }
    }
  }
}

// One workgroup per query head: the splits' partial outputs, rescaled to their common maximum, gated.
__global__ __launch_bounds__(256) void attn_spec_merge_kernel(const float* __restrict__ ws, float* __restrict__ O,
                                                              const float* __restrict__ gate, int VD, int nsplit,
                                                              const DynKeys dyn) {
  __shared__ float f_s[1024];
  __shared__ float red[4];
  const int h = blockIdx.x, tid = threadIdx.x, wave = tid >> 6;
  const float* base = ws + (int64_t)h * nsplit * (VD + 2);
  if (dyn.kv_len_ptr != nullptr) nsplit = dh::dyn_key_range(dyn).nsplit;
  float M = -FLT_MAX;
  for (int s = tid; s < nsplit; s += 256) M = fmaxf(M, base[(int64_t)s * (VD + 2) + VD]);
  M = dh::group_combine<1, 64>(M, dh::MaxOp());
  if ((tid & 63) == 0) red[wave] = M;
  __syncthreads();
  M = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
  __syncthreads();
  float den = 0.f;
  for (int s = tid; s < nsplit; s += 256) {
    const float f = __builtin_amdgcn_exp2f(base[(int64_t)s * (VD + 2) + VD] - M);
    f_s[s] = f;
    den = fmaf(f, base[(int64_t)s * (VD + 2) + VD + 1], den);
  }
  den = dh::wave_sum_uniform(den);
  if ((tid & 63) == 0) red[wave] = den;
  __syncthreads();
  den = red[0] + red[1] + red[2] + red[3];
  const float inv = (den > 0.f ? 1.0f / den : 0.f) * (gate ? sigmoid_f(gate[h]) : 1.0f);
  for (int d = tid; d < VD; d += 256) {
    float num = 0.f;
#pragma unroll 8
    for (int s = 0; s < nsplit; s++) num = fmaf(f_s[s], base[(int64_t)s * (VD + 2) + d], num);
    O[(int64_t)h * VD + d] = num * inv;
  }
}

// Keys and values of T projection rows into the caches: one wave per (token, kv head).
template <typename KV>
__global__ __launch_bounds__(256) void kv_write_kernel(const SpecArgs a, int T) {
  const int lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= (int64_t)T * a.Hkv) return;              // wave-uniform
  const int t = (int)(item / a.Hkv), kvh = (int)(item % a.Hkv);
  const float* row = a.qkv + (int64_t)t * a.ld_qkv;
  float k[8] = {}, v[8] = {};
  if (8 * lane < a.D) load8(row + a.k_off + (int64_t)kvh * a.D + 8 * lane, k);
  if (8 * lane < a.VD) load8(row + a.v_off + (int64_t)kvh * a.VD + 8 * lane, v);
  if (a.value_norm) {
    const float f = value_factor<64>(v, a.value_dim, a.value_eps);
#pragma unroll
    for (int i = 0; i < 8; i++) v[i] *= f;
  }
  Piece<KV> pk, pv;
  pk.set(k);
  pv.set(v);
  const int64_t at = (int64_t)(a.pos0 + t) * a.Hkv + kvh;
  if (8 * lane < a.D) pk.store(static_cast<KV*>(a.K) + at * a.D + 8 * lane);
  if (8 * lane < a.VD) pv.store(static_cast<KV*>(a.V) + at * a.VD + 8 * lane);
}

typedef void (*SpecKernel)(const SpecArgs);
template <typename KV, int L>
SpecKernel pick_heads(int gt) {
  switch (gt) {
    case 1: return attn_spec_kernel<KV, L, 1>;
    case 2: return attn_spec_kernel<KV, L, 2>;
    case 4: return attn_spec_kernel<KV, L, 4>;
    default:
      if constexpr (L < 64) return attn_spec_kernel<KV, L, 8>;
      else return attn_spec_kernel<KV, L, 4>;
  }
}
template <typename KV>
SpecKernel pick_lanes(int lanes, int gt) {
  switch (lanes) {
    case 8: return pick_heads<KV, 8>(gt);
    case 16: return pick_heads<KV, 16>(gt);
    case 32: return pick_heads<KV, 32>(gt);
    default: return pick_heads<KV, 64>(gt);
  }
}

int lanes_for(int D, int VD) {
  const int n = std::max(D, VD);
  return n <= 64 ? 8 : n <= 128 ? 16 : n <= 256 ? 32 : 64;
}
int heads_at_once(int G, int lanes) {
  const int gt = G <= 1 ? 1 : G <= 2 ? 2 : G <= 4 ? 4 : 8;
  return lanes == 64 ? std::min(gt, 4) : gt;      // wide heads: fewer of them at once fit the registers
}

SpecArgs make_args(const dh_attn_spec* s, const float* qkv, void* K, void* V) {
  SpecArgs a{};
  a.qkv = qkv; a.K = K; a.V = V;
  a.ld_qkv = s->ld_qkv;
  a.H = s->H; a.Hkv = s->Hkv; a.G = s->H / s->Hkv; a.D = s->D; a.VD = s->VD; a.value_dim = s->value_dim;
  a.k_off = s->k_offset; a.v_off = s->v_offset; a.gate_off = s->gate_offset;
  a.own_d = s->D;
  a.window = s->window; a.value_norm = s->value_norm; a.scale = s->scale; a.value_eps = s->value_eps;
  a.r1 = s->d_bias_r1; a.r2 = s->d_bias_r2;
  return a;
}

int launch_spec(const char* op, const dh_attn_spec* s, const SpecArgs& a, int T) {
  const int lanes = lanes_for(a.D, a.VD), gt = heads_at_once(a.G, lanes);
  const dim3 grid((unsigned)(s->Hkv * dh::ceil_div(a.G, gt)), (unsigned)a.nsplit, (unsigned)T);
  SpecKernel k = s->cache_dtype == DH_F16 ? pick_lanes<__half>(lanes, gt) : pick_lanes<float>(lanes, gt);
  hipLaunchKernelGGL(k, grid, dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  return 0;
}

}  // namespace

namespace dh {

int attn_spec_check(const char* op, const dh_attn_spec* s) {
  if (!s) return fail(1, "[%s] null spec", op);
  if (s->H <= 0 || s->Hkv <= 0 || s->H % s->Hkv) return fail(1, "[%s] numHeads=%d must be a positive multiple of numKVHeads=%d", op, s->H, s->Hkv);
  if (s->D <= 0 || s->D > 512 || s->D % 8 || s->VD <= 0 || s->VD > 512 || s->VD % 8)
    return fail(1, "[%s] head sizes must be multiples of 8 up to 512 (keys %d, values %d)", op, s->D, s->VD);
  if (s->value_dim <= 0 || s->value_dim > s->VD) return fail(1, "[%s] value_dim=%d is outside 1..%d", op, s->value_dim, s->VD);
  if (s->window < 0) return fail(1, "[%s] window must be non-negative", op);
  if (s->cache_dtype != DH_F16 && s->cache_dtype != DH_F32) return fail(1, "[%s] caches must be f16 or f32, got dtype %d", op, s->cache_dtype);
  if ((s->k_offset | s->v_offset | s->ld_qkv) & 3) return fail(1, "[%s] projection offsets and stride must be multiples of 4", op);
  const int64_t need = std::max<int64_t>(std::max<int64_t>((int64_t)s->H * s->D, s->k_offset + (int64_t)s->Hkv * s->D),
                                         std::max<int64_t>(s->v_offset + (int64_t)s->Hkv * s->VD, s->gate_offset >= 0 ? (int64_t)s->gate_offset + s->H : 0));
  if (s->k_offset < 0 || s->v_offset < 0 || s->ld_qkv < need) return fail(1, "[%s] a projection row of %d floats does not hold its heads", op, s->ld_qkv);
  if ((s->d_bias_r1 == nullptr) != (s->d_bias_r2 == nullptr)) return fail(1, "[%s] the distance bias needs both of its parameters", op);
  return 0;
}

int attn_spec_prefill_general(const char* op, const dh_attn_spec* s, const float* d_qkv, const void* K, const void* V,
                              void* d_out, int out_dtype, int ld_out, int T, int start_pos, const SharedKey& shared) {
  SpecArgs a = make_args(s, d_qkv, const_cast<void*>(K), const_cast<void*>(V));
  a.O = out_dtype == DH_F32 ? static_cast<float*>(d_out) : nullptr;
  a.O16 = out_dtype == DH_BF16 ? static_cast<uint16_t*>(d_out) : nullptr;
  a.ld_out = ld_out; a.nsplit = 1; a.direct = 1;
  a.D += shared.dim; a.KS = shared.rows; a.ld_shared = shared.ld;
  // the grid's third dimension holds at most 65535 query tokens
  for (int t0 = 0; t0 < T; t0 += 32768) {
    SpecArgs b = a;
    b.qkv = a.qkv + (int64_t)t0 * a.ld_qkv;
    b.pos0 = start_pos + t0;
    if (b.O) b.O += (int64_t)t0 * ld_out;
    if (b.O16) b.O16 += (int64_t)t0 * ld_out;
    if (int rc = launch_spec(op, s, b, std::min(32768, T - t0))) return rc;
  }
  return 0;
}

}  // namespace dh

extern "C" {

size_t dh_attn_spec_workspace_bytes(int H, int VD, int max_kv_len) {
  if (H <= 0 || VD <= 0 || max_kv_len <= 0) return 256;
  const size_t splits = std::min<size_t>((size_t)dh::ceil_div(max_kv_len, dh::kAttnTileKeys), 1024);
  return std::max<size_t>(256, (size_t)H * splits * (VD + 2) * sizeof(float));
}

int dh_attn_spec_kv_write(const dh_attn_spec* spec, const float* d_qkv, void* d_cache_k, void* d_cache_v, int T,
                          int start_pos) {
  const char* op = "dh_attn_spec_kv_write";
  DH_REQUIRE_INIT(op);
  if (int rc = dh::attn_spec_check(op, spec)) return rc;
  if (T <= 0 || start_pos < 0) return dh::fail(1, "[%s] seqLen must be positive and startPos non-negative", op);
  if (!d_qkv || !d_cache_k || !d_cache_v) return dh::fail(1, "[%s] null pointer", op);
  if ((reinterpret_cast<uintptr_t>(d_qkv) | reinterpret_cast<uintptr_t>(d_cache_k) | reinterpret_cast<uintptr_t>(d_cache_v)) & 15)
    return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  SpecArgs a = make_args(spec, d_qkv, d_cache_k, d_cache_v);
  a.pos0 = start_pos;
  const unsigned grid = (unsigned)dh::ceil_div((int64_t)T * spec->Hkv, 4);
  if (spec->cache_dtype == DH_F16) hipLaunchKernelGGL(kv_write_kernel<__half>, dim3(grid), dim3(256), 0, dh::stream(), a, T);
  else hipLaunchKernelGGL(kv_write_kernel<float>, dim3(grid), dim3(256), 0, dh::stream(), a, T);
  DH_CHECK_LAUNCH(op);
  return 0;
}

int dh_attn_spec_decode(const dh_attn_spec* spec, const float* d_qkv, void* d_cache_k, void* d_cache_v, float* d_out,
                        int pos, const uint32_t* d_kv_len, int max_kv_len, void* d_workspace) {
  const char* op = "dh_attn_spec_decode";
  DH_REQUIRE_INIT(op);
  if (int rc = dh::attn_spec_check(op, spec)) return rc;
  if (pos < 0) return dh::fail(1, "[%s] the position must be non-negative", op);
  if (d_kv_len && max_kv_len <= 0) return dh::fail(1, "[%s] max_kv_len must be positive with the key count on the device", op);
  if (!d_qkv || !d_cache_k || !d_cache_v || !d_out || !d_workspace) return dh::fail(1, "[%s] null pointer", op);
  if ((reinterpret_cast<uintptr_t>(d_qkv) | reinterpret_cast<uintptr_t>(d_cache_k) | reinterpret_cast<uintptr_t>(d_cache_v)) & 15)
    return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  SpecArgs a = make_args(spec, d_qkv, d_cache_k, d_cache_v);
  a.O = d_out; a.ld_out = (int64_t)spec->H * spec->VD; a.ws = static_cast<float*>(d_workspace);
  a.append = 1; a.pos0 = pos;
  const int one_per_cu = dh::attn_one_per_cu(dh::num_cus(), spec->Hkv);
  if (d_kv_len) {
    a.dyn.kv_len_ptr = d_kv_len; a.dyn.max_kv_len = max_kv_len; a.dyn.causal = 1; a.dyn.start_pos = -1;
    a.dyn.sliding_window = spec->window; a.dyn.kv_start = 0; a.dyn.qkv = 1; a.dyn.one_per_cu = one_per_cu;
    const int keys = spec->window > 0 ? std::min(max_kv_len, spec->window) : max_kv_len;
    a.nsplit = dh::max_splits_upto(one_per_cu, keys);
  } else {
    a.kend = pos + 1;
    a.kbeg = spec->window > 0 ? std::max(0, pos - spec->window + 1) : 0;
    a.nsplit = dh::splits_for(one_per_cu, a.kend - a.kbeg);
    a.direct = a.nsplit == 1;
  }
  if (int rc = launch_spec(op, spec, a, 1)) return rc;
  if (!a.direct) {
    hipLaunchKernelGGL(attn_spec_merge_kernel, dim3(spec->H), dim3(256), 0, dh::stream(), a.ws, d_out,
                       spec->gate_offset >= 0 ? d_qkv + spec->gate_offset : nullptr, spec->VD, a.nsplit, a.dyn);
    DH_CHECK_LAUNCH(op);
  }
  return 0;
}

}  // extern "C"
