// Shared by the two files that serve dh_attn_spec (attention_spec.hip, attention_prefill.hip).
#pragma once
#include "dh_common.h"

namespace dh {
// Host-side validation of a spec: 0, or fail().
int attn_spec_check(const char* op, const dh_attn_spec* s);
// T queries with the any-shape kernel (the cache rows up to each query's own are written).
int attn_spec_prefill_general(const char* op, const dh_attn_spec* s, const float* d_qkv, const void* K, const void* V,
                              void* d_out, int out_dtype, int ld_out, int T, int start_pos);
}  // namespace dh
