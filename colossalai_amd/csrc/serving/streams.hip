// Parallel residual streams ("hyper-connections"): instead of one residual row a token carries S rows
// x_1 .. x_S (float32). A sublayer reads u = sum_s in[s] x_s and, from its output y,
// x_t <- sum_s mix[s, t] x_s + out[t] y for all t at once from the old rows.
//   streams_start  : the (scaled) embedding row becomes every stream, and the first sublayer's input
//                    rms_norm(u) * w is formed in the same launch;
//   streams_update : the write of one sublayer, in place, and the read + norm of the next one
//                    (or of the output, with in = 1 everywhere) in one pass over the streams.
#include "serving_common.h"

namespace cai {
namespace serving {

DEV_INLINE void load4(const float* p, float* o) {
  const float4v a = *reinterpret_cast<const float4v*>(p);
  o[0] = a[0]; o[1] = a[1]; o[2] = a[2]; o[3] = a[3];
}
DEV_INLINE void load4(const bf16s* p, float* o) {
  const short4v a = *reinterpret_cast<const short4v*>(p);
#pragma unroll
  for (int e = 0; e < 4; ++e) o[e] = bf2f((bf16s)a[e]);
}
DEV_INLINE void store4(float* p, const float* v) { *reinterpret_cast<float4v*>(p) = float4v{v[0], v[1], v[2], v[3]}; }
DEV_INLINE void store4(bf16s* p, const float* v) {
  short4v a;
#pragma unroll
  for (int e = 0; e < 4; ++e) a[e] = (short)f2bf(v[e]);
  *reinterpret_cast<short4v*>(p) = a;
}

constexpr int STREAMS_MAX = 8;  // streams the register form is built for; more take the general form

// One block per token; a thread owns the same four neighbouring channels of all S streams, CH times 1024 channels
// apart. Every stream element is read once and written once; u stays in registers over the block's reduction.
template <typename TY, typename TO, int S, int CH>
__global__ __launch_bounds__(256) void streams_update_rows_kernel(
    TO* __restrict__ h, float* __restrict__ x, const TY* __restrict__ y, const float* __restrict__ mix,
    const float* __restrict__ w_out, const float* __restrict__ w_in, const float* __restrict__ w, int W, float eps) {
  __shared__ float red[8];
  const long row = blockIdx.x;
  float mx[S][S], wo[S], wi[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    wo[s] = w_out[s];
    wi[s] = w_in != nullptr ? w_in[s] : 1.0f;
#pragma unroll
    for (int t = 0; t < S; ++t) mx[s][t] = mix[s * S + t];
  }
  float* xr = x + row * S * (long)W;
  float u[CH][4];
  float ssq = 0.0f;
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (threadIdx.x + 256 * c) * 4;
    if (i < W) {
      float old[S][4], yv[4];
#pragma unroll
      for (int s = 0; s < S; ++s) load4(xr + (long)s * W + i, old[s]);
      load4(y + row * (long)W + i, yv);
#pragma unroll
      for (int e = 0; e < 4; ++e) u[c][e] = 0.0f;
#pragma unroll
      for (int t = 0; t < S; ++t) {
        float nv[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) nv[e] = wo[t] * yv[e];
#pragma unroll
        for (int s = 0; s < S; ++s)
#pragma unroll
          for (int e = 0; e < 4; ++e) nv[e] += mx[s][t] * old[s][e];
        store4(xr + (long)t * W + i, nv);
#pragma unroll
        for (int e = 0; e < 4; ++e) u[c][e] += wi[t] * nv[e];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) ssq += u[c][e] * u[c][e];
    }
  }
  if (h == nullptr) return;
  ssq = block_reduce_sum(ssq, red);
  const float inv = 1.0f / sqrtf(ssq / (float)W + eps);
#pragma unroll
  for (int c = 0; c < CH; ++c) {
    const int i = (threadIdx.x + 256 * c) * 4;
    if (i < W) {
      float wv[4];
      load4(w + i, wv);
#pragma unroll
      for (int e = 0; e < 4; ++e) wv[e] *= u[c][e] * inv;
      store4(h + row * (long)W + i, wv);
    }
  }
}

// Any width and up to 32 streams: a thread owns single channels (all streams of them), u is formed again from the
// rows it has written.
template <typename TY, typename TO>
__global__ __launch_bounds__(256) void streams_update_kernel(
    TO* __restrict__ h, float* __restrict__ x, const TY* __restrict__ y, const float* __restrict__ mix,
    const float* __restrict__ w_out, const float* __restrict__ w_in, const float* __restrict__ w, int W, int S, float eps) {
  __shared__ float red[8];
  const long row = blockIdx.x;
  float* xr = x + row * S * (long)W;
  float old[32];
  float ssq = 0.0f;
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    for (int s = 0; s < S; ++s) old[s] = xr[(long)s * W + i];
    const float yv = ldf(y + row * (long)W + i);
    float u = 0.0f;
    for (int t = 0; t < S; ++t) {
      float nv = w_out[t] * yv;
      for (int s = 0; s < S; ++s) nv += mix[s * S + t] * old[s];
      xr[(long)t * W + i] = nv;
      u += (w_in != nullptr ? w_in[t] : 1.0f) * nv;
    }
    ssq += u * u;
  }
  if (h == nullptr) return;
  ssq = block_reduce_sum(ssq, red);
  const float inv = 1.0f / sqrtf(ssq / (float)W + eps);
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    float u = 0.0f;
    for (int t = 0; t < S; ++t) u += (w_in != nullptr ? w_in[t] : 1.0f) * xr[(long)t * W + i];
    stf(h + row * (long)W + i, u * inv * w[i]);
  }
}

c10::optional<at::Tensor> streams_update(at::Tensor x, at::Tensor y, at::Tensor mix, at::Tensor w_out,
                                         c10::optional<at::Tensor> w_in, c10::optional<at::Tensor> weight, double eps,
                                         at::ScalarType out_dtype) {
  check_act(y, "y");
  TORCH_CHECK(x.is_cuda() && is_f32(x) && x.dim() == 3 && x.is_contiguous(), "streams must be contiguous float32 [N, S, W]");
  const long N = x.size(0);
  const int S = (int)x.size(1), W = (int)x.size(2);
  TORCH_CHECK(S >= 1 && S <= 32, "between 1 and 32 streams");
  TORCH_CHECK(y.is_contiguous() && y.dim() == 2 && y.size(0) == N && y.size(1) == W, "y must be contiguous [N, W]");
  TORCH_CHECK(out_dtype == at::kFloat || out_dtype == at::kBFloat16);
  at::Tensor mx = f32c(mix), wo = f32c(w_out), wi, w, h;
  TORCH_CHECK(mx.is_cuda() && mx.dim() == 2 && mx.size(0) == S && mx.size(1) == S && wo.is_cuda() && wo.numel() == S,
              "mix must be [S, S], out [S]");
  const float* wip = nullptr;
  const float* wp = nullptr;
  if (w_in.has_value()) {
    wi = f32c(*w_in);
    TORCH_CHECK(wi.is_cuda() && wi.numel() == S, "in must be [S]");
    wip = wi.data_ptr<float>();
  }
  if (weight.has_value()) {
    w = f32c(*weight);
    TORCH_CHECK(w.is_cuda() && w.numel() == W, "the norm's weight must be [W]");
    wp = w.data_ptr<float>();
    h = at::empty({N, W}, y.options().dtype(out_dtype));
  }
  if (N > 0) {
    const at::Tensor& like = weight.has_value() ? h : y;  // without a norm nothing is written through h
    auto al16 = [](const void* p) { return p == nullptr || reinterpret_cast<uintptr_t>(p) % 16 == 0; };
    const bool rows = S <= STREAMS_MAX && W % 4 == 0 && W <= 8192 && al16(x.data_ptr()) && al16(y.data_ptr()) && al16(wp);
#define STREAMS_ROWS(S_, CH_)                                                                                      \
  hipLaunchKernelGGL((streams_update_rows_kernel<TY, TO, S_, CH_>), dim3((unsigned)N), dim3(256), 0, stream(), hp,  \
                     x.data_ptr<float>(), ptr<TY>(y), mx.data_ptr<float>(), wo.data_ptr<float>(), wip, wp, W, (float)eps)
#define STREAMS_CASE(S_)                    \
  case S_:                                  \
    if (W <= 1024) STREAMS_ROWS(S_, 1);     \
    else if (W <= 2048) STREAMS_ROWS(S_, 2); \
    else if (W <= 4096) STREAMS_ROWS(S_, 4); \
    else STREAMS_ROWS(S_, 8);               \
    break
    SERVING_DISPATCH_ACT(y, TY, {
      SERVING_DISPATCH_ACT(like, TO, {
        TO* hp = weight.has_value() ? ptr<TO>(h) : (TO*)nullptr;
        if (rows) {
          switch (S) {
            STREAMS_CASE(1); STREAMS_CASE(2); STREAMS_CASE(3); STREAMS_CASE(4);
            STREAMS_CASE(5); STREAMS_CASE(6); STREAMS_CASE(7); STREAMS_CASE(8);
          }
        } else {
          hipLaunchKernelGGL((streams_update_kernel<TY, TO>), dim3((unsigned)N), dim3(256), 0, stream(), hp,
                             x.data_ptr<float>(), ptr<TY>(y), mx.data_ptr<float>(), wo.data_ptr<float>(), wip, wp, W, S,
                             (float)eps);
        }
      });
    });
#undef STREAMS_CASE
#undef STREAMS_ROWS
    HIP_CHECK_LAST();
  }
  if (!weight.has_value()) return c10::nullopt;
  return h;
}

// One block per token: table row tokens[n] -> all S streams, and rms_norm((sum_s in[s]) * row) * w. V channels per
// thread and step (4: the width is a multiple of 4 and every row 16-byte aligned); the row is read again for the norm.
template <typename TE, int V>
__global__ __launch_bounds__(256) void streams_start_kernel(TE* __restrict__ h, float* __restrict__ x,
                                                            const TE* __restrict__ table, const long* __restrict__ tokens,
                                                            const float* __restrict__ w_in, const float* __restrict__ w,
                                                            int W, int S, float eps, float scale) {
  __shared__ float red[8];
  const long row = blockIdx.x;
  const TE* er = table + tokens[row] * (long)W;
  float* xr = x + row * S * (long)W;
  float ssq = 0.0f, total = 0.0f;
  for (int s = 0; s < S; ++s) total += w_in[s];
#pragma unroll 2
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float e[V];
    if constexpr (V == 4) load4(er + i, e);
    else e[0] = ldf(er + i);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      e[k] *= scale;
      ssq += (total * e[k]) * (total * e[k]);
    }
    for (int s = 0; s < S; ++s) {
      if constexpr (V == 4) store4(xr + (long)s * W + i, e);
      else xr[(long)s * W + i] = e[0];
    }
  }
  ssq = block_reduce_sum(ssq, red);
  const float inv = total / sqrtf(ssq / (float)W + eps);
#pragma unroll 2
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float e[V], wv[V];
    if constexpr (V == 4) {
      load4(er + i, e);
      load4(w + i, wv);
#pragma unroll
      for (int k = 0; k < V; ++k) e[k] = e[k] * scale * inv * wv[k];
      store4(h + row * (long)W + i, e);
    } else {
      stf(h + row * (long)W + i, ldf(er + i) * scale * inv * w[i]);
    }
  }
}

std::vector<at::Tensor> streams_start(at::Tensor table, at::Tensor tokens, int64_t streams, at::Tensor w_in,
                                      at::Tensor weight, double eps, double scale) {
  check_act(table, "table");
  TORCH_CHECK(table.dim() == 2 && table.is_contiguous(), "table must be contiguous [vocab, W]");
  TORCH_CHECK(tokens.is_cuda() && tokens.scalar_type() == at::kLong && tokens.dim() == 1 && tokens.is_contiguous(),
              "tokens must be contiguous int64 [N]");
  const long N = tokens.size(0);
  const int W = (int)table.size(1), S = (int)streams;
  at::Tensor wi = f32c(w_in), w = f32c(weight);
  TORCH_CHECK(S >= 1 && S <= 32 && wi.is_cuda() && wi.numel() == S && w.is_cuda() && w.numel() == W);
  at::Tensor x = at::empty({N, S, W}, table.options().dtype(at::kFloat));
  at::Tensor h = at::empty({N, W}, table.options());
  auto al16 = [](const at::Tensor& t) { return reinterpret_cast<uintptr_t>(t.data_ptr()) % 16 == 0; };
  const bool vec = W % 4 == 0 && al16(table) && al16(w) && al16(x) && al16(h);
  if (N > 0) {
    SERVING_DISPATCH_ACT(table, TE, {
      if (vec)
        hipLaunchKernelGGL((streams_start_kernel<TE, 4>), dim3((unsigned)N), dim3(256), 0, stream(), ptr<TE>(h),
                           x.data_ptr<float>(), ptr<TE>(table), (const long*)tokens.data_ptr<int64_t>(),
                           wi.data_ptr<float>(), w.data_ptr<float>(), W, S, (float)eps, (float)scale);
      else
        hipLaunchKernelGGL((streams_start_kernel<TE, 1>), dim3((unsigned)N), dim3(256), 0, stream(), ptr<TE>(h),
                           x.data_ptr<float>(), ptr<TE>(table), (const long*)tokens.data_ptr<int64_t>(),
                           wi.data_ptr<float>(), w.data_ptr<float>(), W, S, (float)eps, (float)scale);
    });
    HIP_CHECK_LAST();
  }
  return {x, h};
}

}  // namespace serving
}  // namespace cai
