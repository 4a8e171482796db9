// What the split-key attention kernels share.
#pragma once

#include "serving_common.h"

namespace cai {
namespace serving {

// Optional parameters beyond the common ones.
struct ScalarExtras {
  const float* sink_logits = nullptr;
  const float* dist_bias = nullptr;
  int dist_rows = 0;
  const void* ksum = nullptr;
  const void* vsum = nullptr;
  int sum_shift = 0, sum_block = 1;
  float* cross_out = nullptr;
  int chunk = 0;
  const float* key_fac = nullptr;
  int vrep = 1;
  float* out32 = nullptr;
};

template <int CTRL>
DEV_INLINE float dpp_add(float v) {
  const int moved = __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, false);
  return v + __builtin_bit_cast(float, moved);
}

// First position a query at `pos` sees: its block of `chunk` positions, its window, or position 0.
DEV_INLINE int first_visible(int pos, int window, int chunk) {
  if (chunk > 0) return pos - pos % chunk;
  return window > 0 ? max(0, pos - window + 1) : 0;
}

// The form of the split-key kernel that keeps a block's rows in registers (row_attention.hip); false when the shape or
// the options are not its.
bool launch_row_attention(at::Tensor& out, const at::Tensor& q, const at::Tensor& kpool, const at::Tensor& vpool,
                          const at::Tensor& block_tables, const at::Tensor& tok_seq, const at::Tensor& positions,
                          const float* slopes, const c10::optional<at::Tensor>& gate, long gate_stride, double scale,
                          int64_t window, int64_t keep_first, double softcap, bool sink, int page_shift, long vrow,
                          long vhead, const ScalarExtras& x);

}  // namespace serving
}  // namespace cai
