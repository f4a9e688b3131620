// Matrix memory with exponential gates (dh_mlstm): per head a state S [dim][vdim], a normaliser n [dim] and a running maximum m,
//
//   m' = max(f + m, i);  S' = e^(f + m - m') S + e^(i - m') k v^T;  n' likewise with k alone
//   o  = S'^T q / (max(|n' . q|, e^-m') + 1e-6)
//   i  = cap tanh(z_i / cap),  f = log sigmoid(cap tanh(z_f / cap)),  m starts at 0
//
// everything in 32-bit.  S is updated in place; n and m live in two slots, and a step at position p reads slot p & 1 and
// writes the other, so that every workgroup of a head can read them while one writes.  At position 0 the state counts as zero,
// whatever the buffers hold.
//
// Decode: mlstm_step_kernel, one workgroup per (head, 32 value columns).
// Prefill cuts a portion into chunks of 64 tokens.  With F the running sum of f (kept in double: its differences are the
// exponents), m is known for every token from a max-plus scan, and a chunk's outputs are a product with the state before it plus a
// masked product inside it:
//
//   mlstm_gates_kernel     F, i, m of every token; one workgroup per head
//   mlstm_chunks_kernel    what every chunk adds to the state behind it, sum_s e^(F_end - F_s + i_s - m_end) k_s v_s^T: independent of
//                          one another, because m is known
//   mlstm_scan_kernel      the state in front of every chunk, S_(c+1) = e^(F_end - F_start + m_start - m_end) S_c + what chunk c adds,
//                          element by element and in place
//   mlstm_outputs_kernel   o of (chunk, head, value columns): Q K^T and Q S in one walk over dim, decay mask, then (Q K^T) V
//
// on the 32-bit matrix-core instruction v_mfma_f32_32x32x2_f32.  head_norm_gate_kernel then divides every head's output by its root
// mean square and applies the weight and the output gate.
#include <algorithm>
#include <cfloat>

#include "dense_device.h"

namespace {

using dh::f32x16_t;
using dh::f32x4_t;

constexpr int kChunk = 64;           // tokens per chunk
constexpr int kCols = 32;            // value columns per workgroup of a step
constexpr float kDenominatorEps = 1e-6f;

struct MemArgs {
  const float* rows;       // projection rows [T][ld_row]: q heads, k heads, v heads, .., i, f
  float* S;                // [H][DP][VP]
  float* n;                // [2][H][DP]
  float* m;                // [2][H]
  float* out;              // [T][ld_out] raw head outputs
  int64_t ld_row, ld_out;
  int H, DP, VP, k_off, v_off, i_off, f_off;
  float gate_cap, q_scale;
  int pos, T, chunks;
  const uint32_t* kv_len;
  // portions: gates [H][T], states in front of chunks
  double* F;
  float* i;
  float* mt;               // m after every token
  float* mc;               // [H][chunks + 1] m in front of every chunk, and at the end
  float* keep;             // [H][chunks] what a chunk leaves of the state in front of it
  float* Sc;               // [chunks + 1][H][DP][VP]
  float* nc;               // [chunks + 1][H][DP]
};

__device__ __forceinline__ float log_input_gate(const MemArgs& a, float z) { return a.gate_cap * tanhf(z / a.gate_cap); }
__device__ __forceinline__ float log_forget_gate(const MemArgs& a, float z) {
  const float t = a.gate_cap * tanhf(z / a.gate_cap);
  return fminf(t, 0.f) - log1pf(expf(-fabsf(t)));
}

// Eight lanes x four columns, 32 rows at a time.
__global__ __launch_bounds__(256) void mlstm_step_kernel(const MemArgs a) {
  __shared__ float red[4];
  __shared__ float4 o_lds[4][8];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.y, col = kCols * blockIdx.x + 4 * (tid & 7);
  const int pos = a.kv_len ? max(0, (int)*a.kv_len - 1) : a.pos;
  const bool first = pos == 0;
  const int from = pos & 1, to = from ^ 1;
  const float* q = a.rows + (int64_t)h * a.DP;
  const float* k = a.rows + a.k_off + (int64_t)h * a.DP;
  const float li = log_input_gate(a, a.rows[a.i_off + h]), lf = log_forget_gate(a, a.rows[a.f_off + h]);
  const float m_old = first ? 0.f : a.m[from * a.H + h];
  const float m_new = fmaxf(lf + m_old, li);
  const float keep = first ? 0.f : expf(lf + m_old - m_new), put = expf(li - m_new);

  const float4 v = *reinterpret_cast<const float4*>(a.rows + a.v_off + (int64_t)h * a.VP + col);
  float* S = a.S + (int64_t)h * a.DP * a.VP + col;
  float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll 4
  for (int r = tid >> 3; r < a.DP; r += 32) {
    float4* at = reinterpret_cast<float4*>(S + (int64_t)r * a.VP);
    float4 s = first ? make_float4(0.f, 0.f, 0.f, 0.f) : *at;
    const float kp = put * k[r], qr = q[r];
    s.x = fmaf(keep, s.x, kp * v.x); s.y = fmaf(keep, s.y, kp * v.y);
    s.z = fmaf(keep, s.z, kp * v.z); s.w = fmaf(keep, s.w, kp * v.w);
    *at = s;
    acc.x = fmaf(qr, s.x, acc.x); acc.y = fmaf(qr, s.y, acc.y);
    acc.z = fmaf(qr, s.z, acc.z); acc.w = fmaf(qr, s.w, acc.w);
  }
  float dot = 0.f;
  const float* n_old = a.n + ((int64_t)from * a.H + h) * a.DP;
  float* n_new = a.n + ((int64_t)to * a.H + h) * a.DP;
  for (int r = tid; r < a.DP; r += 256) {
    const float n = fmaf(keep, first ? 0.f : n_old[r], put * k[r]);
    dot = fmaf(n, q[r], dot);
    if (blockIdx.x == 0) n_new[r] = n;
  }
  if (blockIdx.x == 0 && tid == 0) a.m[to * a.H + h] = m_new;
  // lanes that hold the same columns lie 8 apart
#pragma unroll
  for (int off = 8; off < 64; off <<= 1) {
    acc.x += __shfl_xor(acc.x, off, 64); acc.y += __shfl_xor(acc.y, off, 64);
    acc.z += __shfl_xor(acc.z, off, 64); acc.w += __shfl_xor(acc.w, off, 64);
  }
  dot = dh::wave_sum_uniform(dot);
  if (lane < 8) o_lds[wave][lane] = acc;
  if (lane == 0) red[wave] = dot;
  __syncthreads();
  if (tid < 8) {
    const float nq = (red[0] + red[1] + red[2] + red[3]) * a.q_scale;
    const float f = a.q_scale / (fmaxf(fabsf(nq), expf(-m_new)) + kDenominatorEps);
    float4 o = o_lds[0][tid];
#pragma unroll
    for (int w = 1; w < 4; w++) { o.x += o_lds[w][tid].x; o.y += o_lds[w][tid].y; o.z += o_lds[w][tid].z; o.w += o_lds[w][tid].w; }
    *reinterpret_cast<float4*>(a.out + (int64_t)h * a.VP + col) = make_float4(o.x * f, o.y * f, o.z * f, o.w * f);
  }
}

// (F, M): a stretch of tokens takes m to max(m + F, M).
struct MaxPlus {
  double F, M;
};
__device__ __forceinline__ MaxPlus then(const MaxPlus& x, const MaxPlus& y) { return {x.F + y.F, fmax(x.M + y.F, y.M)}; }

__global__ __launch_bounds__(1024) void mlstm_gates_kernel(const MemArgs a) {
  __shared__ double sF[1024];
  __shared__ double sM[1024];
  const int tid = threadIdx.x, h = blockIdx.x;
  const int per = (a.T + 1023) / 1024, t0 = min(tid * per, a.T), t1 = min(t0 + per, a.T);
  const float m_in = a.pos == 0 ? 0.f : a.m[(a.pos & 1) * a.H + h];
  double* F = a.F + (int64_t)h * a.T;
  float* li = a.i + (int64_t)h * a.T;
  float* mt = a.mt + (int64_t)h * a.T;
  float* mc = a.mc + (int64_t)h * (a.chunks + 1);
  MaxPlus run = {0.0, -1e30};
  for (int t = t0; t < t1; t++) {
    const float* row = a.rows + (int64_t)t * a.ld_row;
    const float f = log_forget_gate(a, row[a.f_off + h]), i = log_input_gate(a, row[a.i_off + h]);
    run = then(run, {(double)f, (double)i});
    F[t] = (double)f;                                   // becomes the running sum below
    li[t] = i;
  }
  sF[tid] = run.F;
  sM[tid] = run.M;
  __syncthreads();
  for (int off = 1; off < 1024; off <<= 1) {            // inclusive scan over the threads' stretches
    MaxPlus mine = {sF[tid], sM[tid]};
    if (tid >= off) mine = then({sF[tid - off], sM[tid - off]}, mine);
    __syncthreads();
    sF[tid] = mine.F;
    sM[tid] = mine.M;
    __syncthreads();
  }
  const MaxPlus before = tid > 0 ? MaxPlus{sF[tid - 1], sM[tid - 1]} : MaxPlus{0.0, -1e30};
  double sum = before.F, m = fmax((double)m_in + before.F, before.M);
  for (int t = t0; t < t1; t++) {
    if (t % kChunk == 0) mc[t / kChunk] = (float)m;
    const double f = F[t];
    sum += f;
    m = fmax(m + f, (double)li[t]);
    F[t] = sum;
    mt[t] = (float)m;
    if (t == a.T - 1) {
      mc[a.chunks] = (float)m;
      a.m[((a.pos + a.T) & 1) * a.H + h] = (float)m;
    }
  }
  __syncthreads();
  for (int c = tid; c < a.chunks; c += 1024) {
    const double start = c > 0 ? F[c * kChunk - 1] : 0.0, end = F[min((c + 1) * kChunk, a.T) - 1];
    a.keep[(int64_t)h * a.chunks + c] = expf((float)(end - start + (double)mc[c] - (double)mc[c + 1]));
  }
}

// Grid = (64 x 64 tiles of a head's state, heads, chunks); wave w: rows 32 (w >> 1), columns 32 (w & 1) of the tile.
__global__ __launch_bounds__(256) void mlstm_chunks_kernel(const MemArgs a) {
  constexpr int ROW = 64 + 4;
  __shared__ __align__(16) float ks[kChunk * ROW];     // weighted keys [token][dim]
  __shared__ __align__(16) float vs[kChunk * ROW];     // values [token][column]
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, h = blockIdx.y, c = blockIdx.z;
  const int tiles_v = (a.VP + 63) / 64, d0 = 64 * (blockIdx.x / tiles_v), v0 = 64 * (blockIdx.x % tiles_v);
  const double* F = a.F + (int64_t)h * a.T;
  const int first = c * kChunk, count = min(kChunk, a.T - first);
  const double F_end = F[first + count - 1];
  const float m_end = a.mc[(int64_t)h * (a.chunks + 1) + c + 1];
  f32x4_t kr[4], vr[4];
  float w[4];
#pragma unroll
  for (int r = 0; r < 4; r++) {
    const int p = tid + 256 * r, tok = first + min(p >> 4, count - 1), x = 4 * (p & 15);
    const float* row = a.rows + (int64_t)tok * a.ld_row;
    kr[r] = vr[r] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (d0 + x < a.DP) kr[r] = *reinterpret_cast<const f32x4_t*>(row + a.k_off + (int64_t)h * a.DP + d0 + x);
    if (v0 + x < a.VP) vr[r] = *reinterpret_cast<const f32x4_t*>(row + a.v_off + (int64_t)h * a.VP + v0 + x);
    w[r] = (p >> 4) < count ? expf((float)(F_end - F[tok] + (double)a.i[(int64_t)h * a.T + tok] - (double)m_end)) : 0.f;
  }
#pragma unroll
  for (int r = 0; r < 4; r++) {
    const int p = tid + 256 * r, tok = p >> 4, x = 4 * (p & 15);
    kr[r] *= w[r];
    *reinterpret_cast<f32x4_t*>(&ks[tok * ROW + x]) = kr[r];
    *reinterpret_cast<f32x4_t*>(&vs[tok * ROW + x]) = vr[r];
  }
  __syncthreads();
  const int wd = 32 * (wave >> 1), wv = 32 * (wave & 1);
  if (d0 + wd < a.DP && v0 + wv < a.VP) {              // wave-uniform (sizes are multiples of 32)
    f32x16_t acc;
#pragma unroll
    for (int e = 0; e < 16; e++) acc[e] = 0.f;
#pragma unroll 8
    for (int j = 0; j < kChunk / 2; j++) {
      const int tok = 2 * j + (lane >> 5);
      acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ks[tok * ROW + wd + (lane & 31)], vs[tok * ROW + wv + (lane & 31)], acc, 0, 0, 0);
    }
    // accumulator element e of a lane: state row 8 (e / 4) + 4 (lane >> 5) + e % 4, column lane & 31
    float* U = a.Sc + ((int64_t)(c + 1) * a.H + h) * a.DP * a.VP + (int64_t)(d0 + wd + 4 * (lane >> 5)) * a.VP + v0 + wv + (lane & 31);
#pragma unroll
    for (int e = 0; e < 16; e++) U[(int64_t)(8 * (e >> 2) + (e & 3)) * a.VP] = acc[e];
  }
  if (v0 == 0 && tid < 64 && d0 + tid < a.DP) {
    float s = 0.f;
#pragma unroll 8
    for (int t = 0; t < kChunk; t++) s += ks[t * ROW + tid];
    a.nc[((int64_t)(c + 1) * a.H + h) * a.DP + d0 + tid] = s;
  }
}

// Grid = (groups of 1024 elements of a head's [S | n], heads), four per thread; slot 0 of Sc and nc is filled here.
__global__ __launch_bounds__(256) void mlstm_scan_kernel(const MemArgs a) {
  constexpr int AHEAD = 16;
  const int h = blockIdx.y, size = a.DP * a.VP;
  const int64_t i = 4 * ((int64_t)blockIdx.x * 256 + threadIdx.x);
  if (i >= size + a.DP) return;
  const bool is_n = i >= size;
  const int64_t stride = is_n ? (int64_t)a.H * a.DP : (int64_t)a.H * size;
  float* at = is_n ? a.nc + (int64_t)h * a.DP + (i - size) : a.Sc + (int64_t)h * size + i;
  const int64_t slots = (int64_t)a.H * a.DP;
  const float* from = is_n ? a.n + (a.pos & 1) * slots + (int64_t)h * a.DP + (i - size) : a.S + (int64_t)h * size + i;
  float* to = is_n ? a.n + ((a.pos + a.T) & 1) * slots + (int64_t)h * a.DP + (i - size) : a.S + (int64_t)h * size + i;
  const float* keep = a.keep + (int64_t)h * a.chunks;
  f32x4_t s = {0.f, 0.f, 0.f, 0.f};
  if (a.pos > 0) s = *reinterpret_cast<const f32x4_t*>(from);
  *reinterpret_cast<f32x4_t*>(at) = s;
  for (int c0 = 0; c0 < a.chunks; c0 += AHEAD) {
    f32x4_t u[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; k++)
      if (c0 + k < a.chunks) u[k] = *reinterpret_cast<const f32x4_t*>(at + (c0 + k + 1) * stride);
#pragma unroll
    for (int k = 0; k < AHEAD; k++) {
      const int c = c0 + k;
      if (c < a.chunks) {
        s = s * keep[c] + u[k];
        if (c + 1 < a.chunks) *reinterpret_cast<f32x4_t*>(at + (c + 1) * stride) = s;
      }
    }
  }
  *reinterpret_cast<f32x4_t*>(to) = s;
}

// Grid = (chunks, heads, groups of 64 TN value columns); wave w: tokens 32 (w >> 1), columns 32 TN (w & 1) + 0 .. 32 TN - 1.
template <int TN>
__global__ __launch_bounds__(256) void mlstm_outputs_kernel(const MemArgs a) {
  constexpr int BV = 64 * TN, BD = 32, ROW = BD + 4, VROW = BV + 4, PROW = kChunk + 4;
  __shared__ __align__(16) float qs[kChunk * ROW];
  __shared__ __align__(16) float ks[kChunk * ROW];
  __shared__ __align__(16) float sv[kChunk * VROW];    // state rows, later the values
  __shared__ __align__(16) float ps[kChunk * PROW];
  __shared__ double Fl[kChunk];
  __shared__ float il[kChunk];
  __shared__ float ml[kChunk];
  __shared__ float inter[kChunk];                      // what the state before the chunk has decayed to, per token
  __shared__ float nq[kChunk];                         // n_start . q
  __shared__ float nl[BD];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, c = blockIdx.x, h = blockIdx.y, v0 = BV * blockIdx.z;
  const int first = c * kChunk, count = min(kChunk, a.T - first);
  const int wt = 32 * (wave >> 1), wc = 32 * TN * (wave & 1), ws = 32 * (wave & 1);
  const float* Sc = a.Sc + ((int64_t)c * a.H + h) * a.DP * a.VP;
  const float* nc = a.nc + ((int64_t)c * a.H + h) * a.DP;
  if (tid < kChunk) {
    const int t = first + min(tid, count - 1);
    const double F_start = first > 0 ? a.F[(int64_t)h * a.T + first - 1] : 0.0, F = a.F[(int64_t)h * a.T + t];
    const float m = a.mt[(int64_t)h * a.T + t];
    Fl[tid] = F;
    il[tid] = a.i[(int64_t)h * a.T + t];
    ml[tid] = m;
    inter[tid] = expf((float)(F - F_start + (double)a.mc[(int64_t)h * (a.chunks + 1) + c] - (double)m));
  }
  f32x16_t p, o[TN];
#pragma unroll
  for (int e = 0; e < 16; e++) p[e] = 0.f;
#pragma unroll
  for (int j = 0; j < TN; j++)
#pragma unroll
    for (int e = 0; e < 16; e++) o[j][e] = 0.f;
  float dot = 0.f;                                     // token tid >> 2, every fourth dim from tid & 3 on

  f32x4_t qr[2], kr[2], sr[2 * TN];
  float nr = 0.f;
  auto load = [&](int d0) {
#pragma unroll
    for (int r = 0; r < 2; r++) {
      const int x = tid + 256 * r, tok = first + min(x >> 3, count - 1), d = d0 + 4 * (x & 7);
      const float* row = a.rows + (int64_t)tok * a.ld_row + (int64_t)h * a.DP + d;
      qr[r] = *reinterpret_cast<const f32x4_t*>(row);
      kr[r] = *reinterpret_cast<const f32x4_t*>(row + a.k_off);
    }
#pragma unroll
    for (int r = 0; r < 2 * TN; r++) {
      const int x = tid + 256 * r, d = d0 + x / (BV / 4), v = v0 + 4 * (x % (BV / 4));
      sr[r] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (v < a.VP) sr[r] = *reinterpret_cast<const f32x4_t*>(Sc + (int64_t)d * a.VP + v);
    }
    if (tid < BD) nr = nc[d0 + tid];
  };
  load(0);
  for (int d0 = 0; d0 < a.DP; d0 += BD) {
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 2; r++) {
      const int x = tid + 256 * r;
      qr[r] *= a.q_scale;
      *reinterpret_cast<f32x4_t*>(&qs[(x >> 3) * ROW + 4 * (x & 7)]) = qr[r];
      *reinterpret_cast<f32x4_t*>(&ks[(x >> 3) * ROW + 4 * (x & 7)]) = kr[r];
    }
#pragma unroll
    for (int r = 0; r < 2 * TN; r++) {
      const int x = tid + 256 * r;
      *reinterpret_cast<f32x4_t*>(&sv[x / (BV / 4) * VROW + 4 * (x % (BV / 4))]) = sr[r];
    }
    if (tid < BD) nl[tid] = nr;
    __syncthreads();
    if (d0 + BD < a.DP) load(d0 + BD);
#pragma unroll
    for (int s = 0; s < BD / 8; s++) {
      const int d = 8 * s + 4 * (lane >> 5);
      const f32x4_t fq = *reinterpret_cast<const f32x4_t*>(&qs[(wt + (lane & 31)) * ROW + d]);
      const f32x4_t fk = *reinterpret_cast<const f32x4_t*>(&ks[(ws + (lane & 31)) * ROW + d]);
#pragma unroll
      for (int e = 0; e < 4; e++) p = __builtin_amdgcn_mfma_f32_32x32x2f32(fq[e], fk[e], p, 0, 0, 0);
#pragma unroll
      for (int j = 0; j < TN; j++)
#pragma unroll
        for (int e = 0; e < 4; e++)
          o[j] = __builtin_amdgcn_mfma_f32_32x32x2f32(fq[e], sv[(d + e) * VROW + wc + 32 * j + (lane & 31)], o[j], 0, 0, 0);
    }
#pragma unroll
    for (int d = 0; d < BD; d += 4) dot = fmaf(qs[(tid >> 2) * ROW + d + (tid & 3)], nl[d + (tid & 3)], dot);
  }
  dot = dh::group_combine<1, 4>(dot, dh::AddOp());
  if ((tid & 3) == 0) nq[tid >> 2] = dot;
  // decayed scores: accumulator element e holds token wt + 8 (e / 4) + 4 (lane >> 5) + e % 4, earlier token ws + (lane & 31)
  {
    const int s = ws + (lane & 31);
    const double base = (double)il[s] - Fl[s];
#pragma unroll
    for (int e = 0; e < 16; e++) {
      const int t = wt + 8 * (e >> 2) + 4 * (lane >> 5) + (e & 3);
      const float w = s <= t && s < count ? expf((float)(Fl[t] + base - (double)ml[t])) : 0.f;
      ps[t * PROW + s] = w * p[e];
    }
  }
  __syncthreads();                                     // scores are there; the last state rows have been consumed
#pragma unroll
  for (int r = 0; r < 4 * TN; r++) {
    const int x = tid + 256 * r, tok = first + min(x / (BV / 4), count - 1), v = v0 + 4 * (x % (BV / 4));
    f32x4_t vv = {0.f, 0.f, 0.f, 0.f};
    if (v < a.VP) vv = *reinterpret_cast<const f32x4_t*>(a.rows + (int64_t)tok * a.ld_row + a.v_off + (int64_t)h * a.VP + v);
    *reinterpret_cast<f32x4_t*>(&sv[x / (BV / 4) * VROW + 4 * (x % (BV / 4))]) = vv;
  }
  // a token's normaliser and with it the factor of its outputs
  float sum = 0.f;
  for (int s = tid & 3; s < kChunk; s += 4) sum += ps[(tid >> 2) * PROW + s];
  sum = dh::group_combine<1, 4>(sum, dh::AddOp());
#pragma unroll
  for (int e = 0; e < 16; e++) {
    const float f = inter[wt + 8 * (e >> 2) + 4 * (lane >> 5) + (e & 3)];
#pragma unroll
    for (int j = 0; j < TN; j++) o[j][e] *= f;
  }
  __syncthreads();
  if ((tid & 3) == 0) {
    const int t = tid >> 2;
    nq[t] = 1.0f / (fmaxf(fabsf(fmaf(inter[t], nq[t], sum)), expf(-ml[t])) + kDenominatorEps);
  }
#pragma unroll
  for (int s = 0; s < kChunk / 8; s++) {
    const int d = 8 * s + 4 * (lane >> 5);
    const f32x4_t fp = *reinterpret_cast<const f32x4_t*>(&ps[(wt + (lane & 31)) * PROW + d]);
#pragma unroll
    for (int j = 0; j < TN; j++)
#pragma unroll
      for (int e = 0; e < 4; e++)
        o[j] = __builtin_amdgcn_mfma_f32_32x32x2f32(fp[e], sv[(d + e) * VROW + wc + 32 * j + (lane & 31)], o[j], 0, 0, 0);
  }
  __syncthreads();
#pragma unroll
  for (int j = 0; j < TN; j++) {
    const int v = v0 + wc + 32 * j + (lane & 31);
    if (v >= a.VP) continue;
#pragma unroll
    for (int e = 0; e < 16; e++) {
      const int t = wt + 8 * (e >> 2) + 4 * (lane >> 5) + (e & 3);
      if (t < count) a.out[(int64_t)(first + t) * a.ld_out + (int64_t)h * a.VP + v] = o[j][e] * nq[t];
    }
  }
}

// One wave per (row, head): y = x / rms(x over size) * weight * sigmoid(gate).
template <typename OUT>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const float* __restrict__ x, int64_t ld_x, const float* __restrict__ gate,
                                                             int64_t ld_gate, const float* __restrict__ w, OUT* __restrict__ out,
                                                             int64_t ld_out, int rows, int H, int VP, int size, float eps) {
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= (int64_t)rows * H) return;
  const int64_t t = item / H;
  const int h = (int)(item % H);
  const float* xr = x + t * ld_x + (int64_t)h * VP;
  float ss = 0.f;
  for (int i = 4 * lane; i < VP; i += 256) {
    const float4 v = *reinterpret_cast<const float4*>(xr + i);
    ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
  }
  ss = dh::wave_sum_uniform(ss);
  const float inv = 1.0f / sqrtf(ss / (float)size + eps);
  for (int i = 4 * lane; i < VP; i += 256) {
    const float4 v = *reinterpret_cast<const float4*>(xr + i);
    const float4 g = *reinterpret_cast<const float4*>(gate + t * ld_gate + (int64_t)h * VP + i);
    const float4 c = *reinterpret_cast<const float4*>(w + (int64_t)h * VP + i);
    const float y[4] = {v.x * inv * c.x / (1.0f + expf(-g.x)), v.y * inv * c.y / (1.0f + expf(-g.y)),
                        v.z * inv * c.z / (1.0f + expf(-g.z)), v.w * inv * c.w / (1.0f + expf(-g.w))};
    OUT* o = out + t * ld_out + (int64_t)h * VP + i;
    if constexpr (sizeof(OUT) == 2) {
      uint2 two;
      two.x = (uint32_t)dh::f32_to_bf16_bits(y[0]) | ((uint32_t)dh::f32_to_bf16_bits(y[1]) << 16);
      two.y = (uint32_t)dh::f32_to_bf16_bits(y[2]) | ((uint32_t)dh::f32_to_bf16_bits(y[3]) << 16);
      *reinterpret_cast<uint2*>(o) = two;
    } else {
      *reinterpret_cast<float4*>(o) = make_float4(y[0], y[1], y[2], y[3]);
    }
  }
}

int check(const char* op, const dh_mlstm* s) {
  if (!s) return dh::fail(1, "[%s] null spec", op);
  if (s->H <= 0 || s->dim <= 0 || s->vdim <= 0 || s->DP < s->dim || s->VP < s->vdim || s->DP % 32 || s->VP % 32)
    return dh::fail(1, "[%s] heads %d of %d x %d in padded sizes %d x %d (multiples of 32)", op, s->H, s->dim, s->vdim, s->DP, s->VP);
  if (!(s->gate_cap > 0.f)) return dh::fail(1, "[%s] the gate cap must be positive", op);
  const int64_t nq = (int64_t)s->H * s->DP, nv = (int64_t)s->H * s->VP;
  if ((s->ld_row | s->k_offset | s->v_offset) % 4 || s->k_offset < nq || s->v_offset < 0 || s->i_offset < 0 || s->f_offset < 0 ||
      s->ld_row < std::max<int64_t>(std::max<int64_t>(s->k_offset + nq, s->v_offset + nv), (int64_t)std::max(s->i_offset, s->f_offset) + s->H))
    return dh::fail(1, "[%s] a projection row of %d floats does not hold its parts", op, s->ld_row);
  return 0;
}
size_t up256(size_t n) { return (n + 255) / 256 * 256; }

MemArgs make_args(const dh_mlstm* s, const float* rows, float* state, float* out) {
  MemArgs a{};
  a.rows = rows; a.S = state; a.n = state + (size_t)s->H * s->DP * s->VP; a.m = a.n + (size_t)2 * s->H * s->DP; a.out = out;
  a.ld_row = s->ld_row; a.H = s->H; a.DP = s->DP; a.VP = s->VP;
  a.k_off = s->k_offset; a.v_off = s->v_offset; a.i_off = s->i_offset; a.f_off = s->f_offset;
  a.gate_cap = s->gate_cap; a.q_scale = 1.0f / sqrtf((float)s->dim);
  return a;
}
bool aligned(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

}  // namespace

extern "C" {

size_t dh_mlstm_state_bytes(const dh_mlstm* s) {
  if (!s) return 0;
  return up256(((size_t)s->H * s->DP * s->VP + (size_t)2 * s->H * s->DP + (size_t)2 * s->H) * sizeof(float));
}

int dh_mlstm_step(const dh_mlstm* spec, const float* d_row, void* d_state, float* d_out, int pos, const uint32_t* d_kv_len) {
  const char* op = "dh_mlstm_step";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (pos < 0) return dh::fail(1, "[%s] the position must be non-negative", op);
  if (!d_row || !d_state || !d_out) return dh::fail(1, "[%s] null pointer", op);
  if (!aligned(d_row) || !aligned(d_state) || !aligned(d_out)) return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  MemArgs a = make_args(spec, d_row, static_cast<float*>(d_state), d_out);
  a.pos = pos; a.kv_len = d_kv_len;
  hipLaunchKernelGGL(mlstm_step_kernel, dim3(spec->VP / kCols, spec->H), dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  return 0;
}

size_t dh_mlstm_prefill_workspace_bytes(const dh_mlstm* s, int T) {
  if (!s || T <= 0) return 256;
  const size_t chunks = (size_t)dh::ceil_div(T, kChunk), HT = (size_t)s->H * T;
  return up256(HT * 8) + 2 * up256(HT * 4) + 2 * up256((size_t)s->H * (chunks + 1) * 4) + up256((chunks + 1) * s->H * s->DP * 4) +
         up256((chunks + 1) * s->H * s->DP * s->VP * 4);
}

int dh_mlstm_prefill(const dh_mlstm* spec, const float* d_rows, void* d_state, void* d_workspace, float* d_out, int ld_out, int T,
                     int start_pos) {
  const char* op = "dh_mlstm_prefill";
  DH_REQUIRE_INIT(op);
  if (int rc = check(op, spec)) return rc;
  if (T <= 0 || start_pos < 0) return dh::fail(1, "[%s] seqLen must be positive and startPos non-negative", op);
  if (ld_out < spec->H * spec->VP || ld_out % 4) return dh::fail(1, "[%s] ld_out=%d must be a multiple of 4 and hold %d elements", op, ld_out, spec->H * spec->VP);
  if (!d_rows || !d_state || !d_workspace || !d_out) return dh::fail(1, "[%s] null pointer", op);
  if (!aligned(d_rows) || !aligned(d_state) || !aligned(d_out) || !aligned(d_workspace)) return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  MemArgs a = make_args(spec, d_rows, static_cast<float*>(d_state), d_out);
  a.pos = start_pos; a.T = T; a.chunks = (int)dh::ceil_div(T, kChunk); a.ld_out = ld_out;
  char* w = static_cast<char*>(d_workspace);
  auto take = [&](size_t bytes) { char* p = w; w += up256(bytes); return p; };
  const size_t HT = (size_t)spec->H * T;
  a.F = reinterpret_cast<double*>(take(HT * 8));
  a.i = reinterpret_cast<float*>(take(HT * 4));
  a.mt = reinterpret_cast<float*>(take(HT * 4));
  a.mc = reinterpret_cast<float*>(take((size_t)spec->H * (a.chunks + 1) * 4));
  a.keep = reinterpret_cast<float*>(take((size_t)spec->H * (a.chunks + 1) * 4));
  a.nc = reinterpret_cast<float*>(take((size_t)(a.chunks + 1) * spec->H * spec->DP * 4));
  a.Sc = reinterpret_cast<float*>(take((size_t)(a.chunks + 1) * spec->H * spec->DP * spec->VP * 4));
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(spec->H), dim3(1024), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  const int tiles = (int)(dh::ceil_div(spec->DP, 64) * dh::ceil_div(spec->VP, 64));
  // the grid's third dimension holds at most 65535 chunks
  if (a.chunks > 65535) return dh::fail(1, "[%s] %d tokens are too many for one portion", op, T);
  hipLaunchKernelGGL(mlstm_chunks_kernel, dim3(tiles, spec->H, a.chunks), dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  hipLaunchKernelGGL(mlstm_scan_kernel, dim3((unsigned)dh::ceil_div((int64_t)spec->DP * spec->VP + spec->DP, 1024), spec->H), dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  // wide column groups repeat Q K^T less often; narrow ones where those would not fill the device
  const bool wide = spec->VP > 64 && (int64_t)a.chunks * spec->H * dh::ceil_div(spec->VP, 128) >= dh::num_cus();
  if (wide) hipLaunchKernelGGL(mlstm_outputs_kernel<2>, dim3(a.chunks, spec->H, (unsigned)dh::ceil_div(spec->VP, 128)), dim3(256), 0, dh::stream(), a);
  else hipLaunchKernelGGL(mlstm_outputs_kernel<1>, dim3(a.chunks, spec->H, (unsigned)dh::ceil_div(spec->VP, 64)), dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  return 0;
}

int dh_head_norm_gate(const float* d_x, int ld_x, const float* d_gate, int ld_gate, const float* d_weight, void* d_out, int out_dtype,
                      int ld_out, int rows, int H, int padded, int size, float eps) {
  const char* op = "dh_head_norm_gate";
  DH_REQUIRE_INIT(op);
  if (rows <= 0 || H <= 0 || size <= 0 || padded < size || padded % 4) return dh::fail(1, "[%s] %d rows of %d heads of %d elements (padded to %d)", op, rows, H, size, padded);
  if ((ld_x | ld_gate | ld_out) % 4 || std::min(ld_x, std::min(ld_gate, ld_out)) < H * padded)
    return dh::fail(1, "[%s] row strides must be multiples of 4 and hold %d elements (%d, %d, %d)", op, H * padded, ld_x, ld_gate, ld_out);
  if (out_dtype != DH_BF16 && out_dtype != DH_F32) return dh::fail(1, "[%s] output must be bf16 or f32, got dtype %d", op, out_dtype);
  if (!d_x || !d_gate || !d_weight || !d_out) return dh::fail(1, "[%s] null pointer", op);
  if (!aligned(d_x) || !aligned(d_gate) || !aligned(d_weight) || !aligned(d_out)) return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  const dim3 grid((unsigned)dh::ceil_div((int64_t)rows * H, 4));
  if (out_dtype == DH_BF16)
    hipLaunchKernelGGL(head_norm_gate_kernel<uint16_t>, grid, dim3(256), 0, dh::stream(), d_x, ld_x, d_gate, ld_gate, d_weight,
                       static_cast<uint16_t*>(d_out), ld_out, rows, H, padded, size, eps);
  else
    hipLaunchKernelGGL(head_norm_gate_kernel<float>, grid, dim3(256), 0, dh::stream(), d_x, ld_x, d_gate, ld_gate, d_weight,
                       static_cast<float*>(d_out), ld_out, rows, H, padded, size, eps);
  DH_CHECK_LAUNCH(op);
  return 0;
}

}  // extern "C"
