// What the kernels of the delta rule with one decay per head share (host side).
#pragma once

#include "../serving_common.h"

namespace cai {
namespace serving {

constexpr int DELTA_CHUNK = 64;      // tokens per chunk of the chunked form
constexpr int DELTA_CHUNK_MAX_D = 128;

// q, k [N, G, D] float32 dense (unit length, q scaled); gates [N, H, 2] = (beta, decay); v [N, H, Dv], dense rows at
// v.stride(0). Sequential scan, one pass over the tokens of every sequence.
void delta_head_scan(at::Tensor& out, const at::Tensor& q, const at::Tensor& k, const at::Tensor& gates, const at::Tensor& v,
                     at::Tensor& state, const at::Tensor& cu, const at::Tensor& start, const at::Tensor& slots);

// The same in chunks of DELTA_CHUNK tokens on the matrix cores; v float32, gates [N, H, 2] = (beta, log decay).
void delta_head_chunks(at::Tensor& out, const at::Tensor& q, const at::Tensor& k, const at::Tensor& gates,
                       const at::Tensor& v, at::Tensor& state, const at::Tensor& start, const at::Tensor& slots,
                       const at::Tensor& chunks, const at::Tensor& seq_chunks);

// Sets every sequence's convolution tail to its last K - 1 inputs (x [N, C], tail [slots, K - 1, C] float32).
void refresh_conv_tail(const at::Tensor& x, at::Tensor& tail, const at::Tensor& cu, const at::Tensor& start,
                       const at::Tensor& slots, int K);

}  // namespace serving
}  // namespace cai
