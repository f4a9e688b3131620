// Token embedding sums and row norms of the dense-weight decoders.
#include <algorithm>

#include "dense_device.h"

namespace {

struct EmbedArgs {
  const uint32_t* ids;
  const uint32_t* prev;
  const uint16_t* embed;
  const uint16_t* bigram;
  const uint16_t* pos;
  float* out;
  int64_t buckets, mul_prev, mul_cur;
  int vocab, max_positions, ld_out, hidden, start_pos;
  const uint32_t* kv_len;
};

// Grid = (tokens, slices of 2048 columns): eight columns per thread with 16-byte loads where the rows are aligned for
// them, else one column at a time.  Rows that do not exist (id or position out of range) count as zeros, so no id read on
// the device can send a load outside the tables.
template <bool VEC>
__global__ __launch_bounds__(256) void embed_sum_kernel(const EmbedArgs a) {
  const int t = blockIdx.x;
  const int64_t p = a.kv_len ? (int64_t)*a.kv_len - 1 : (int64_t)a.start_pos + t;
  const uint32_t id = a.ids[t];
  const uint16_t* e = id < (uint32_t)a.vocab ? a.embed + (int64_t)id * a.hidden : nullptr;
  const uint16_t* b = nullptr;
  if (a.bigram) {
    int64_t row = a.buckets;
    if (p > 0) {
      const uint32_t prev = t > 0 ? a.ids[t - 1] : *a.prev;
      row = ((int64_t)prev * a.mul_prev + (int64_t)id * a.mul_cur) % a.buckets;
      if (row < 0) row += a.buckets;
    }
    b = a.bigram + row * a.hidden;
  }
  const uint16_t* q = a.pos && p >= 0 && p < a.max_positions ? a.pos + p * a.hidden : nullptr;
  float* o = a.out + (int64_t)t * a.ld_out;
  const int first = 2048 * blockIdx.y;
  if (VEC) {
    const int i = first + 8 * threadIdx.x;
    if (i >= a.hidden) return;
    const dh::u32x4_t none = {0u, 0u, 0u, 0u};
    const dh::u32x4_t ev = e ? *reinterpret_cast<const dh::u32x4_t*>(e + i) : none;
    const dh::u32x4_t bv = b ? *reinterpret_cast<const dh::u32x4_t*>(b + i) : none;
    const dh::u32x4_t qv = q ? *reinterpret_cast<const dh::u32x4_t*>(q + i) : none;
    float v[8];
#pragma unroll
    for (int w = 0; w < 4; w++) {
      v[2 * w] = dh::bf16_low(ev[w]) + dh::bf16_low(bv[w]) + dh::bf16_low(qv[w]);
      v[2 * w + 1] = dh::bf16_high(ev[w]) + dh::bf16_high(bv[w]) + dh::bf16_high(qv[w]);
    }
    reinterpret_cast<float4*>(o + i)[0] = make_float4(v[0], v[1], v[2], v[3]);
    reinterpret_cast<float4*>(o + i)[1] = make_float4(v[4], v[5], v[6], v[7]);
    return;
  }
  const int last = min(first + 2048, a.hidden);
  for (int i = first + threadIdx.x; i < last; i += 256) {
    float v = e ? dh::bf16_bits_to_f32(e[i]) : 0.f;
    if (b) v += dh::bf16_bits_to_f32(b[i]);
    if (q) v += dh::bf16_bits_to_f32(q[i]);
    o[i] = v;
  }
}

// One workgroup per output row; the row stays in registers between the two passes (up to 8 x 1024 elements).
template <bool BF16>
__global__ __launch_bounds__(256) void rmsnorm_rows_kernel(const float* __restrict__ x, int ld_x, const uint32_t* rows,
                                                           const float* __restrict__ w, void* __restrict__ out, int ld_out,
                                                           int hidden, float eps) {
  __shared__ float red[4];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const float* xr = x + (int64_t)(rows ? rows[blockIdx.x] : blockIdx.x) * ld_x;
  const bool vec = (ld_x & 3) == 0 && (hidden & 3) == 0 && hidden <= 8192;
  float4 xv[8];
  float ss = 0.f;
  if (vec) {
#pragma unroll
    for (int j = 0; j < 8; j++) {
      const int i = 4 * (tid + 256 * j);
      xv[j] = i < hidden ? *reinterpret_cast<const float4*>(xr + i) : make_float4(0.f, 0.f, 0.f, 0.f);
      ss = fmaf(xv[j].x, xv[j].x, ss); ss = fmaf(xv[j].y, xv[j].y, ss);
      ss = fmaf(xv[j].z, xv[j].z, ss); ss = fmaf(xv[j].w, xv[j].w, ss);
    }
  } else {
    for (int i = tid; i < hidden; i += 256) ss = fmaf(xr[i], xr[i], ss);
  }
  ss = dh::wave_sum_uniform(ss);
  if (lane == 0) red[wave] = ss;
  __syncthreads();
  const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)hidden + eps);
  const int64_t base = (int64_t)blockIdx.x * ld_out;
  auto put = [&](int i, float v) {
    if (BF16) static_cast<uint16_t*>(out)[base + i] = dh::f32_to_bf16_bits(v);
    else static_cast<float*>(out)[base + i] = v;
  };
  if (vec) {
#pragma unroll
    for (int j = 0; j < 8; j++) {
      const int i = 4 * (tid + 256 * j);
      if (i >= hidden) continue;
      const float4 wv = *reinterpret_cast<const float4*>(w + i);
      const float y[4] = {xv[j].x * inv * wv.x, xv[j].y * inv * wv.y, xv[j].z * inv * wv.z, xv[j].w * inv * wv.w};
      if (BF16 && (ld_out & 3) == 0) {
        uint2 two;
        two.x = (uint32_t)dh::f32_to_bf16_bits(y[0]) | ((uint32_t)dh::f32_to_bf16_bits(y[1]) << 16);
        two.y = (uint32_t)dh::f32_to_bf16_bits(y[2]) | ((uint32_t)dh::f32_to_bf16_bits(y[3]) << 16);
        *reinterpret_cast<uint2*>(static_cast<uint16_t*>(out) + base + i) = two;
      } else {
#pragma unroll
        for (int e = 0; e < 4; e++) put(i + e, y[e]);
      }
    }
  } else {
    for (int i = tid; i < hidden; i += 256) put(i, xr[i] * inv * w[i]);
  }
  for (int i = hidden + tid; i < ld_out; i += 256) put(i, 0.f);
}

}  // namespace

extern "C" {

int dh_embed_sum(const uint32_t* d_ids, int index_offset, const uint32_t* d_prev, const void* d_embed, int vocab,
                 const void* d_bigram, int64_t buckets, int64_t mul_prev, int64_t mul_cur, const void* d_pos,
                 int max_positions, float* d_out, int ld_out, int T, int hidden, int start_pos, const uint32_t* d_kv_len) {
  const char* op = "dh_embed_sum";
  DH_REQUIRE_INIT(op);
  if (T <= 0 || hidden <= 0 || vocab <= 0) return dh::fail(1, "[%s] Dimensions must be positive: T=%d, hidden=%d, vocab=%d", op, T, hidden, vocab);
  if (index_offset < 0 || start_pos < 0) return dh::fail(1, "[%s] indexOffset and startPos must be non-negative", op);
  if (ld_out < hidden) return dh::fail(1, "[%s] ld_out=%d is shorter than hidden=%d", op, ld_out, hidden);
  if (!d_ids || !d_embed || !d_out) return dh::fail(1, "[%s] null pointer", op);
  if (d_kv_len && T != 1) return dh::fail(1, "[%s] the device key count serves one token, got T=%d", op, T);
  if (d_bigram && buckets <= 0) return dh::fail(1, "[%s] buckets must be positive", op);
  if (d_bigram && !d_prev && (start_pos > 0 || d_kv_len)) return dh::fail(1, "[%s] the token before position %d is needed", op, start_pos);
  if (d_pos && (max_positions <= 0 || (!d_kv_len && start_pos + T > max_positions)))
    return dh::fail(1, "[%s] positions %d..%d are outside the table of %d", op, start_pos, start_pos + T - 1, max_positions);
  EmbedArgs a{};
  a.ids = d_ids + index_offset; a.prev = d_prev;
  a.embed = static_cast<const uint16_t*>(d_embed); a.bigram = static_cast<const uint16_t*>(d_bigram);
  a.pos = static_cast<const uint16_t*>(d_pos);
  a.out = d_out; a.buckets = buckets; a.mul_prev = mul_prev; a.mul_cur = mul_cur;
  a.vocab = vocab; a.max_positions = max_positions; a.ld_out = ld_out; a.hidden = hidden; a.start_pos = start_pos;
  a.kv_len = d_kv_len;
  const bool vec = hidden % 8 == 0 && ld_out % 4 == 0 &&
                   ((reinterpret_cast<uintptr_t>(d_embed) | reinterpret_cast<uintptr_t>(d_bigram) | reinterpret_cast<uintptr_t>(d_pos) |
                     reinterpret_cast<uintptr_t>(d_out)) & 15) == 0;
  const dim3 grid((unsigned)T, (unsigned)dh::ceil_div(hidden, 2048));
  if (vec) hipLaunchKernelGGL(embed_sum_kernel<true>, grid, dim3(256), 0, dh::stream(), a);
  else hipLaunchKernelGGL(embed_sum_kernel<false>, grid, dim3(256), 0, dh::stream(), a);
  DH_CHECK_LAUNCH(op);
  return 0;
}

int dh_rmsnorm_rows(const float* d_x, int ld_x, const uint32_t* d_rows, const float* d_weight, void* d_out, int out_dtype,
                    int ld_out, int n, int hidden, float eps) {
  const char* op = "dh_rmsnorm_rows";
  DH_REQUIRE_INIT(op);
  if (n <= 0 || hidden <= 0) return dh::fail(1, "[%s] Dimensions must be positive: rows=%d, hidden=%d", op, n, hidden);
  if (ld_x < hidden || ld_out < hidden) return dh::fail(1, "[%s] row strides must hold hidden=%d elements (%d, %d)", op, hidden, ld_x, ld_out);
  if (out_dtype != DH_BF16 && out_dtype != DH_F32) return dh::fail(1, "[%s] output must be bf16 or f32, got dtype %d", op, out_dtype);
  if (!d_x || !d_weight || !d_out) return dh::fail(1, "[%s] null pointer", op);
  if ((reinterpret_cast<uintptr_t>(d_x) | reinterpret_cast<uintptr_t>(d_weight) | reinterpret_cast<uintptr_t>(d_out)) & 15)
    return dh::fail(1, "[%s] pointers must be 16-byte aligned", op);
  if (out_dtype == DH_BF16)
    hipLaunchKernelGGL(rmsnorm_rows_kernel<true>, dim3(n), dim3(256), 0, dh::stream(), d_x, ld_x, d_rows, d_weight, d_out, ld_out, hidden, eps);
  else
    hipLaunchKernelGGL(rmsnorm_rows_kernel<false>, dim3(n), dim3(256), 0, dh::stream(), d_x, ld_x, d_rows, d_weight, d_out, ld_out, hidden, eps);
  DH_CHECK_LAUNCH(op);
  return 0;
}

}  // extern "C"
