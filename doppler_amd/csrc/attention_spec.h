// Shared by the two files that serve dh_attn_spec (attention_spec.hip, attention_prefill.hip).
#pragma once
#include "dh_common.h"

namespace dh {
// Host-side validation of a spec: 0, or fail().
int attn_spec_check(const char* op, const dh_attn_spec* s);
// Key elements that all heads of a token share (a rotated part beside every head's own): head keys are [D own | dim shared],
// row r of the shared part lies ld elements behind row r - 1.  dim 0: none.
struct SharedKey {
  const void* rows;
  int dim;
  int64_t ld;
};
// T queries with the any-shape kernel (the cache rows up to each query's own are written).
int attn_spec_prefill_general(const char* op, const dh_attn_spec* s, const float* d_qkv, const void* K, const void* V,
                              void* d_out, int out_dtype, int ld_out, int T, int start_pos, const SharedKey& shared);
}  // namespace dh
