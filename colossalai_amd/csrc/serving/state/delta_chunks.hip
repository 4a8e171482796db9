// Delta rule with one decay per head and token: fused inputs, and the chunked form for prompt portions.
//
// Inputs. One kernel goes from the raw projections to the recurrence's float32 operands: short causal convolution
// (up to four taps, carried tail), SiLU, unit length of every q/k head, write strength beta, decay (or its logarithm).
//
// Chunked form. With b_i the running sum of the log decays inside a chunk of 64 tokens and S0 the state ahead of it,
//   (I + L) U = diag(beta) (V - diag(e^b) K S0),   L_ij = beta_i e^{b_i - b_j} (k_i . k_j), j < i
//   o_i = e^{b_i} S0^T q_i + sum_{j <= i} e^{b_i - b_j} (q_i . k_j) u_j
//   S   = e^{b_C} S0 + sum_j e^{b_C - b_j} k_j u_j^T
// (every exponent is <= 0). delta_chunk_prepare_kernel forms, for all chunks at once, what does not depend on S0:
// A_ij = e^{b_i - b_j} (q_i . k_j), Uv = (I + L)^-1 diag(beta) V, -W = -(I + L)^-1 diag(beta e^b) K and
// (e^{b_C - b} K)^T. delta_chunk_scan_kernel then walks a sequence's chunks: U = Uv - W S0, outputs, next state. Value
// channels are independent, so a block owns 16 of them and keeps its part of the state in registers. All products are
// float32 on the matrix cores (16x16x4), whose results leave the registers in the operand layout of the next product
// when the contraction index of step s and lane group g is taken as 4 g + s.
#include "delta.h"

namespace cai {
namespace serving {

constexpr int CHK = DELTA_CHUNK;
constexpr int FUSED_TAPS = 4;

DEV_INLINE f32x4 mfma4(const float4v& a, const float4v& b, f32x4 c) {
#pragma unroll
  for (int s = 0; s < 4; ++s) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[s], b[s], c, 0, 0, 0);
  return c;
}

// --------------------------------------------------------------------------- inputs
// One wave per (tile of TT tokens, unit): a unit is a q head, a k head, 256 channels of a v head, or (the last one) the
// gates of all heads. Lane channels: 2 * lane + 128 r, two at a time (V2), or lane + 64 r. own_tail: every sequence
// brings one token, so the wave that reads a tail entry is the only one and shifts it in place.
template <typename T, bool V2, int R, int TT>
__global__ __launch_bounds__(256) void delta_inputs_kernel(
    float* __restrict__ qn, float* __restrict__ kn, float* __restrict__ vo, float* __restrict__ gates,
    const T* __restrict__ x, long xs, const float* __restrict__ taps, float* tail, long ts, const T* __restrict__ bl,
    long bls, const T* __restrict__ dt, long dts, const float* __restrict__ A_log, const float* __restrict__ dt_bias,
    const int* __restrict__ cu, const int* __restrict__ start, const int* __restrict__ slots,
    const int* __restrict__ tok_seq, long N, int G, int H, int D, int Dv, int K, int pieces, int own_tail, int log_decay,
    float unit_eps, float q_scale) {
  constexpr int E = V2 ? 2 : 1;
  const int lane = threadIdx.x & 63;
  const int unit = blockIdx.y * (blockDim.x >> 6) + (threadIdx.x >> 6);
  const long n0 = (long)blockIdx.x * TT;
  const int units = 2 * G + H * pieces;
  const int cnt = (int)min((long)TT, N - n0);
  if (unit > units) return;
  if (unit == units) {
    for (int i = lane; i < cnt * H; i += 64) {
      const long n = n0 + i / H;
      const int h = i % H;
      const float lg = -expf(A_log[h]) * softplusf_(ldf(dt + n * dts + h) + dt_bias[h]);
      gates[2 * (n * H + h)] = sigmoidf_(ldf(bl + n * bls + h));
      gates[2 * (n * H + h) + 1] = log_decay ? lg : expf(lg);
    }
    return;
  }
  const bool isv = unit >= 2 * G;
  const int vh = isv ? (unit - 2 * G) / pieces : 0, piece = isv ? (unit - 2 * G) % pieces : 0;
  const int width = isv ? min(256, Dv - piece * 256) : D;         // channels of this unit
  const int C = 2 * G * D + H * Dv;
  const int c0 = isv ? 2 * G * D + vh * Dv + piece * 256 : unit * D;
  float* dst = isv ? vo + (long)vh * Dv + piece * 256 : (unit < G ? qn + (long)unit * D : kn + (long)(unit - G) * D);
  const long drow = isv ? (long)H * Dv : (long)G * D;
  const float post = unit < G ? q_scale : 1.0f;

  int ch[R];
  bool live[R];
  float w[FUSED_TAPS][R][E];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int c = V2 ? 2 * lane + 128 * r : lane + 64 * r;
    live[r] = c < width;
    ch[r] = live[r] ? c : 0;
#pragma unroll
    for (int d = 0; d < FUSED_TAPS; ++d)
#pragma unroll
      for (int e = 0; e < E; ++e) w[d][r][e] = live[r] && d < K ? taps[(long)(c0 + ch[r] + e) * K + K - 1 - d] : 0.0f;
  }
  auto row = [&](const T* p, float (&o)[R][E]) {
#pragma unroll
    for (int r = 0; r < R; ++r) {
      if constexpr (V2) load2(p + c0 + ch[r], o[r][0], o[r][1]);
      else o[r][0] = ldf(p + c0 + ch[r]);
    }
  };
  float cur[TT][R][E];
#pragma unroll
  for (int t = 0; t < TT; ++t) row(x + min(n0 + t, N - 1) * xs, cur[t]);

  float hist[FUSED_TAPS - 1][R][E];   // the inputs 1, 2, 3 tokens back
  int prev = -1;
#pragma unroll
  for (int t = 0; t < TT; ++t) {
    if (t < cnt) {
      const long n = n0 + t;
      const int b = tok_seq[n];
      const int i = (int)(n - cu[b]);
      float* tl = tail + (long)slots[b] * ts;
      if (b != prev) {
        const bool fresh = start[b] == 0;
#pragma unroll
        for (int d = 1; d < FUSED_TAPS; ++d) {
          if (d <= i && d < K) {
            row(x + (n - d) * xs, hist[d - 1]);
          } else {
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
              for (int e = 0; e < E; ++e)
                hist[d - 1][r][e] = d < K && d > i && !fresh ? tl[(long)(K - 1 + i - d) * C + c0 + ch[r] + e] : 0.0f;
          }
        }
        prev = b;
      }
      float y[R][E], ssq = 0.0f;
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < E; ++e) {
          float a = w[0][r][e] * cur[t][r][e];
#pragma unroll
          for (int d = 1; d < FUSED_TAPS; ++d) a += w[d][r][e] * hist[d - 1][r][e];
          a *= sigmoidf_(a);
          y[r][e] = a;
          ssq += live[r] ? a * a : 0.0f;
        }
      float f = 1.0f;
      if (!isv) f = post / sqrtf(wave_reduce_sum(ssq) + unit_eps);
#pragma unroll
      for (int r = 0; r < R; ++r) {
        if (!live[r]) continue;
        if constexpr (V2) *reinterpret_cast<float2v*>(dst + n * drow + ch[r]) = float2v{y[r][0] * f, y[r][1] * f};
        else dst[n * drow + ch[r]] = y[r][0] * f;
      }
      if (own_tail) {
#pragma unroll
        for (int d = FUSED_TAPS - 2; d >= 0; --d)   // entry K - 2 - d of the new tail is the input d tokens back
          if (d <= K - 2) {
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
              for (int e = 0; e < E; ++e)
                if (live[r]) tl[(long)(K - 2 - d) * C + c0 + ch[r] + e] = d == 0 ? cur[t][r][e] : hist[d > 0 ? d - 1 : 0][r][e];
          }
      }
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int e = 0; e < E; ++e) {
#pragma unroll
          for (int d = FUSED_TAPS - 2; d > 0; --d) hist[d][r][e] = hist[d - 1][r][e];
          hist[0][r][e] = cur[t][r][e];
        }
    }
  }
}

// -------------------------------------------------------------------- chunk preparation
// Row-major scratch per (chunk, head): negw [64, Dp], kdt [Dp, 64], amat [64, 64] (lower tiles only are written and
// read), eb [64] = e^{b_i}; uv [VT tiles of 16 columns][4 tiles of 16 tokens][64 lanes][4] in the products' result layout.
struct ChunkScratch {
  float *negw, *kdt, *amat, *eb, *uv;
};

// grid (chunks, H), 256 threads. NT = Dp / 64.
template <int NT>
__global__ __launch_bounds__(256) void delta_chunk_prepare_kernel(
    ChunkScratch o, const float* __restrict__ q, const float* __restrict__ k, const float* __restrict__ gates,
    const float* __restrict__ v, long vs, const int* __restrict__ chunks, int H, int G, int D, int Dv) {
  constexpr int Dp = 64 * NT, KP = Dp + 4, LP = CHK + 4, TP = 20;
  extern __shared__ __align__(16) float lds[];
  float* Ks = lds;                       // [64][KP]
  float* Qs = Ks + CHK * KP;             // [64][KP], then -L [64][LP]
  float* Lm = Qs;
  float* Ti = Qs + CHK * KP;             // [4][16][TP] inverses of the diagonal blocks of I + L
  double* bs = reinterpret_cast<double*>(Ti + 4 * 16 * TP);   // [64] running log decay: only differences of it are used,
                                                              // and one strong decay must not cost them their digits
  float* bt = reinterpret_cast<float*>(bs + CHK);             // [64] beta
  static_assert(KP >= LP, "L must fit where the queries were");
  const int tid = threadIdx.x, wid = tid >> 6, lane = tid & 63;
  const int col = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, hq = h / (H / G);
  const int* cd = chunks + 4 * (long)blockIdx.x;
  const int n0 = cd[1], cnt = min(cd[2] - n0, CHK);
  const long unit = (long)blockIdx.x * H + h;
  const int VT = (Dv + 15) >> 4;

  const bool vec = (D & 3) == 0;
  for (int i = tid; i < 2 * CHK * (Dp / 4); i += 256) {
    const bool isq = i >= CHK * (Dp / 4);
    const int r = (i / (Dp / 4)) % CHK, d = 4 * (i % (Dp / 4));
    float4v val = {0.0f, 0.0f, 0.0f, 0.0f};
    if (r < cnt && d < D) {
      const float* src = (isq ? q : k) + ((long)(n0 + r) * G + hq) * D + d;
      if (vec) {
        val = *reinterpret_cast<const float4v*>(src);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < D) val[e] = src[e];
      }
    }
    *reinterpret_cast<float4v*>((isq ? Qs : Ks) + r * KP + d) = val;
  }
  if (wid == 0) {
    const bool ok = lane < cnt;
    const long at = 2 * ((long)(n0 + (ok ? lane : 0)) * H + h);
    double b = ok ? gates[at + 1] : 0.0f;
    bt[lane] = ok ? gates[at] : 0.0f;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const double up = __shfl_up(b, off);
      if (lane >= off) b += up;
    }
    bs[lane] = b;
    o.eb[unit * CHK + lane] = expf((float)b);
  }
  __syncthreads();

  // the ten lower tiles of K K^T and of Q K^T, five to each wave
  f32x4 res[5];
#pragma unroll
  for (int u = 0; u < 5; ++u) {
    const int id = wid + 4 * u, low = id % 10;
    const int ti = low < 1 ? 0 : low < 3 ? 1 : low < 6 ? 2 : 3, tj = low - ti * (ti + 1) / 2;
    const float* arow = (id < 10 ? Ks : Qs) + (16 * ti + col) * KP + 4 * g;
    const float* brow = Ks + (16 * tj + col) * KP + 4 * g;
    f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int t = 0; t < Dp / 16; ++t)
      acc = mfma4(*reinterpret_cast<const float4v*>(arow + 16 * t), *reinterpret_cast<const float4v*>(brow + 16 * t), acc);
    res[u] = acc;
  }
  __syncthreads();  // the queries have been read: L takes their place
#pragma unroll
  for (int u = 0; u < 5; ++u) {
    const int id = wid + 4 * u, low = id % 10;
    const int ti = low < 1 ? 0 : low < 3 ? 1 : low < 6 ? 2 : 3, tj = low - ti * (ti + 1) / 2;
    const int j = 16 * tj + col;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 16 * ti + 4 * g + r;
      const float e = j <= i ? expf((float)(bs[i] - bs[j])) : 0.0f;
      if (id < 10) Lm[i * LP + j] = j < i ? -bt[i] * e * res[u][r] : 0.0f;
      else o.amat[unit * CHK * CHK + i * CHK + j] = e * res[u][r];
    }
  }
  __syncthreads();
  {  // wave w inverts diagonal block w, a column per lane (the four lane groups hold the same)
    float t[16];
    const float* L = Lm + 16 * wid * LP + 16 * wid;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float a = i == col ? 1.0f : 0.0f;
#pragma unroll
      for (int m = 0; m < i; ++m) a += L[i * LP + m] * t[m];
      t[i] = a;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (g == (i & 3)) Ti[(wid * 16 + i) * TP + col] = t[i];
  }
  __syncthreads();

  // (I + L) X = diag(beta) [V | diag(e^b) K], 16 columns at a time, block rows from the top
  const double btot = bs[CHK - 1];
  for (int ct = wid; ct < VT + Dp / 16; ct += 4) {
    const bool isk = ct >= VT;
    const int c = 16 * (isk ? ct - VT : ct) + col;
    f32x4 X[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      f32x4 acc;
      float4v kd;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * i + 4 * g + r;
        if (isk) {
          const float kv = Ks[t * KP + c];
          acc[r] = bt[t] * expf((float)bs[t]) * kv;
          kd[r] = expf((float)(btot - bs[t])) * kv;
        } else {
          acc[r] = t < cnt && c < Dv ? bt[t] * v[(long)(n0 + t) * vs + (long)h * Dv + c] : 0.0f;
        }
      }
      if (isk) *reinterpret_cast<float4v*>(o.kdt + (unit * Dp + c) * CHK + 16 * i + 4 * g) = kd;
#pragma unroll
      for (int m = 0; m < i; ++m)
        acc = mfma4(*reinterpret_cast<const float4v*>(Lm + (16 * i + col) * LP + 16 * m + 4 * g), X[m], acc);
      const f32x4 none = {0.0f, 0.0f, 0.0f, 0.0f};
      X[i] = mfma4(*reinterpret_cast<const float4v*>(Ti + (i * 16 + col) * TP + 4 * g), acc, none);
      if (isk) {
#pragma unroll
        for (int r = 0; r < 4; ++r) o.negw[(unit * CHK + 16 * i + 4 * g + r) * Dp + c] = -X[i][r];
      } else {
        *reinterpret_cast<f32x4*>(o.uv + ((unit * VT + ct) * 4 + i) * 256 + lane * 4) = X[i];
      }
    }
  }
}

// ------------------------------------------------------------------------ chunk scan
// grid (H, ceil(Dv / 16), B), four waves. Wave w owns tokens 16 w .. 16 w + 15 of a chunk and NT tiles of 16 state rows.
// The loads of the next chunk are issued as soon as this chunk's values have been used, without branches, so that they
// are in flight over the products in between. VEC: D is a multiple of 4.
template <int NT, bool VEC>
__global__ __launch_bounds__(256) void delta_chunk_scan_kernel(
    float* __restrict__ out, ChunkScratch s, const float* __restrict__ q, float* __restrict__ state, long ss,
    const int* __restrict__ start, const int* __restrict__ slots, const int* __restrict__ chunks,
    const int* __restrict__ seq_chunks, int H, int G, int D, int Dv) {
  constexpr int Dp = 64 * NT, SP = Dp + 4, UP = CHK + 4, KT = Dp / 16;
  __shared__ __align__(16) float St[16 * SP];   // [column][state row]
  __shared__ __align__(16) float Ut[16 * UP];   // [column][token]
  const int tid = threadIdx.x, wid = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int col = lane & 15, g = lane >> 4;
  const int h = blockIdx.x, hq = h / (H / G), slice = blockIdx.y, b = blockIdx.z;
  const int VT = (Dv + 15) >> 4;
  const int c = 16 * slice + col;
  float* Sg = state + (long)slots[b] * ss + (long)h * D * Dv;
  const bool fresh = start[b] == 0;
  const int k0 = seq_chunks[b], k1 = seq_chunks[b + 1];

  f32x4 S[NT];
#pragma unroll
  for (int j = 0; j < NT; ++j)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * (wid * NT + j) + 4 * g + r;
      S[j][r] = !fresh && d < D && c < Dv ? Sg[(long)d * Dv + c] : 0.0f;
    }
  float4v wA[KT], qA[KT], aA[4], kA[NT][4];
  float4v ebr;
  f32x4 uv;
  float etot;
  auto load_state_side = [&](int ck) {   // what multiplies the state: -W rows and query rows of this wave's tokens
    const long unit = (long)ck * H + h;
    const int t = 16 * wid + col, n0 = chunks[4 * (long)ck + 1], cnt = chunks[4 * (long)ck + 2] - n0;
    const float* wr = s.negw + (unit * CHK + t) * Dp + 4 * g;
    const float* qr = q + ((long)(n0 + min(t, cnt - 1)) * G + hq) * D;   // a row past the end is not stored
#pragma unroll
    for (int i = 0; i < KT; ++i) {
      wA[i] = *reinterpret_cast<const float4v*>(wr + 16 * i);
      const int d = 16 * i + 4 * g;   // state rows past D are zero: what they are multiplied with only has to exist
      if constexpr (VEC) {
        qA[i] = *reinterpret_cast<const float4v*>(qr + min(d, D - 4));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) qA[i][e] = qr[min(d + e, D - 1)];
      }
    }
    uv = *reinterpret_cast<const f32x4*>(s.uv + ((unit * VT + slice) * 4 + wid) * 256 + lane * 4);
  };
  auto load_token_side = [&](int ck) {   // what multiplies U: A rows of this wave's tokens, its rows of (e^{b_C - b} K)^T
    const long unit = (long)ck * H + h;
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      aA[m] = *reinterpret_cast<const float4v*>(s.amat + unit * CHK * CHK + (16 * wid + col) * CHK + 16 * min(m, wid) + 4 * g);
#pragma unroll
      for (int j = 0; j < NT; ++j)
        kA[j][m] = *reinterpret_cast<const float4v*>(s.kdt + (unit * Dp + 16 * (wid * NT + j) + col) * CHK + 16 * m + 4 * g);
    }
    ebr = *reinterpret_cast<const float4v*>(s.eb + unit * CHK + 16 * wid + 4 * g);
    etot = s.eb[unit * CHK + CHK - 1];
  };
  if (k0 < k1) {
    load_state_side(k0);
    load_token_side(k0);
  }
  for (int ck = k0; ck < k1; ++ck) {
    const int n0 = chunks[4 * (long)ck + 1], cnt = chunks[4 * (long)ck + 2] - n0;
#pragma unroll
    for (int j = 0; j < NT; ++j) *reinterpret_cast<f32x4*>(St + col * SP + 16 * (wid * NT + j) + 4 * g) = S[j];
    __syncthreads();
    f32x4 u = uv, oa = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int i = 0; i < KT; ++i) {
      const float4v sb = *reinterpret_cast<const float4v*>(St + col * SP + 16 * i + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        u = __builtin_amdgcn_mfma_f32_16x16x4f32(wA[i][e], sb[e], u, 0, 0, 0);
        oa = __builtin_amdgcn_mfma_f32_16x16x4f32(qA[i][e], sb[e], oa, 0, 0, 0);
      }
    }
    *reinterpret_cast<f32x4*>(Ut + col * UP + 16 * wid + 4 * g) = u;
    load_state_side(min(ck + 1, k1 - 1));
    __syncthreads();
#pragma unroll
    for (int r = 0; r < 4; ++r) oa[r] *= ebr[r];
#pragma unroll
    for (int j = 0; j < NT; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[j][r] *= etot;
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const float4v ub = *reinterpret_cast<const float4v*>(Ut + col * UP + 16 * m + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
#pragma unroll
        for (int j = 0; j < NT; ++j) S[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(kA[j][m][e], ub[e], S[j], 0, 0, 0);
      }
      if (m <= wid) oa = mfma4(aA[m], ub, oa);
    }
    load_token_side(min(ck + 1, k1 - 1));
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 16 * wid + 4 * g + r;
      if (t < cnt && c < Dv) out[((long)(n0 + t) * H + h) * Dv + c] = oa[r];
    }
  }
#pragma unroll
  for (int j = 0; j < NT; ++j)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int d = 16 * (wid * NT + j) + 4 * g + r;
      if (d < D && c < Dv) Sg[(long)d * Dv + c] = S[j][r];
    }
}

template <int NT>
static void launch_chunks(at::Tensor& out, const at::Tensor& q, const at::Tensor& k, const at::Tensor& gates,
                          const at::Tensor& v, at::Tensor& state, const at::Tensor& start, const at::Tensor& slots,
                          const at::Tensor& chunks, const at::Tensor& seq_chunks) {
  constexpr int Dp = 64 * NT;
  const int G = (int)q.size(1), D = (int)q.size(2), H = (int)v.size(1), Dv = (int)v.size(2), VT = (Dv + 15) / 16;
  const long units = chunks.size(0) * H;
  const int B = (int)start.numel();
  at::Tensor buf = at::empty({units * (2L * CHK * Dp + CHK * CHK + CHK + VT * 1024L)}, q.options());
  ChunkScratch s;
  s.negw = buf.data_ptr<float>();
  s.kdt = s.negw + units * CHK * Dp;
  s.amat = s.kdt + units * CHK * Dp;
  s.eb = s.amat + units * CHK * CHK;
  s.uv = s.eb + units * CHK;
  const size_t smem = (size_t)(2 * CHK * (Dp + 4) + 4 * 16 * 20 + 3 * CHK) * sizeof(float);
  auto prep = delta_chunk_prepare_kernel<NT>;
  if (smem > 65536)  // more dynamic LDS than a kernel gets without asking
    (void)hipFuncSetAttribute((const void*)prep, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem);
  hipLaunchKernelGGL(prep, dim3((unsigned)chunks.size(0), (unsigned)H), dim3(256), smem, stream(), s, q.data_ptr<float>(),
                     k.data_ptr<float>(), gates.data_ptr<float>(), v.data_ptr<float>(), (long)v.stride(0),
                     chunks.data_ptr<int>(), H, G, D, Dv);
  auto scan = D % 4 == 0 ? delta_chunk_scan_kernel<NT, true> : delta_chunk_scan_kernel<NT, false>;
  hipLaunchKernelGGL(scan, dim3((unsigned)H, (unsigned)VT, (unsigned)B), dim3(256), 0, stream(),
                     out.data_ptr<float>(), s, q.data_ptr<float>(), state.data_ptr<float>(), (long)state.stride(0),
                     start.data_ptr<int>(), slots.data_ptr<int>(), chunks.data_ptr<int>(), seq_chunks.data_ptr<int>(), H, G,
                     D, Dv);
  HIP_CHECK_LAST();
}

void delta_head_chunks(at::Tensor& out, const at::Tensor& q, const at::Tensor& k, const at::Tensor& gates,
                       const at::Tensor& v, at::Tensor& state, const at::Tensor& start, const at::Tensor& slots,
                       const at::Tensor& chunks, const at::Tensor& seq_chunks) {
  check_i32(chunks, "chunks"); check_i32(seq_chunks, "seq_chunks");
  TORCH_CHECK(chunks.dim() == 2 && chunks.size(1) == 4 && chunks.size(0) > 0 && seq_chunks.numel() == start.numel() + 1);
  TORCH_CHECK(q.size(2) <= DELTA_CHUNK_MAX_D && is_f32(v) && v.stride(2) == 1 && v.stride(1) == v.size(2));
  if (q.size(2) <= 64) launch_chunks<1>(out, q, k, gates, v, state, start, slots, chunks, seq_chunks);
  else launch_chunks<2>(out, q, k, gates, v, state, start, slots, chunks, seq_chunks);
}

// x [N, 2 G D + H Dv] raw projections (q heads, k heads, v heads), taps [C, K], tail [slots, K - 1, C] float32 or none
// (K = 1), beta_logit and dt [N, H]. Convolution with SiLU, unit length, gates, then the recurrence: in chunks when
// their tables are given, token by token otherwise. Returns o [N, H, Dv] float32.
at::Tensor conv_delta_rule(at::Tensor x, at::Tensor taps, c10::optional<at::Tensor> tail, at::Tensor beta_logit, at::Tensor dt,
                           at::Tensor A_log, at::Tensor dt_bias, at::Tensor state, at::Tensor cu, at::Tensor start,
                           at::Tensor slots, at::Tensor tok_seq, int64_t groups, int64_t dim, double unit_eps, double q_scale,
                           c10::optional<at::Tensor> chunks, c10::optional<at::Tensor> seq_chunks) {
  check_act(x, "x"); check_act(beta_logit, "beta_logit"); check_act(dt, "dt");
  TORCH_CHECK(x.dim() == 2 && x.stride(1) == 1, "x must be [N, C] with unit inner stride");
  TORCH_CHECK(state.is_cuda() && is_f32(state) && state.dim() == 4, "state must be float32 [slots, H, D, Dv]");
  const long N = x.size(0);
  const int C = (int)x.size(1), K = (int)taps.size(1), G = (int)groups, D = (int)dim;
  const int H = (int)state.size(1), Dv = (int)state.size(3);
  TORCH_CHECK(G > 0 && H % G == 0 && D > 0 && D <= 256 && state.size(2) == D && C == 2 * G * D + H * Dv,
              "x must hold G query heads, G key heads and H value heads");
  TORCH_CHECK(state.stride(3) == 1 && state.stride(2) == Dv && state.stride(1) == (long)D * Dv, "state must be dense inside a slot");
  TORCH_CHECK(taps.dim() == 2 && taps.size(0) == C && K >= 1 && K <= FUSED_TAPS, "taps must be [C, K], K <= 4");
  auto logits_ok = [&](const at::Tensor& t) {
    return t.dim() == 2 && t.size(0) == N && t.size(1) == H && t.stride(1) == 1 && t.scalar_type() == x.scalar_type();
  };
  TORCH_CHECK(logits_ok(beta_logit) && logits_ok(dt), "beta_logit and dt must be [N, H] of x's type");
  check_i32(cu, "cu"); check_i32(start, "start"); check_i32(slots, "slots"); check_i32(tok_seq, "tok_seq");
  const int B = (int)start.numel();
  TORCH_CHECK(tok_seq.numel() == N && cu.numel() == B + 1 && slots.numel() == B);
  at::Tensor tp = f32c(taps), Af = f32c(A_log), bf = f32c(dt_bias);
  TORCH_CHECK(Af.numel() == H && bf.numel() == H && Af.is_cuda() && bf.is_cuda() && tp.is_cuda());
  auto fo = x.options().dtype(at::kFloat);
  at::Tensor out = at::empty({N, H, Dv}, fo);
  if (N == 0) return out;
  float* tlp = nullptr;
  long ts = 0;
  if (K > 1) {
    TORCH_CHECK(tail.has_value(), "a convolution with more than one tap carries a tail");
    TORCH_CHECK(tail->is_cuda() && is_f32(*tail) && tail->dim() == 3 && tail->size(1) == K - 1 && tail->size(2) == C &&
                tail->stride(2) == 1 && tail->stride(1) == C, "tail must be float32 [slots, K-1, C]");
    tlp = tail->data_ptr<float>();
    ts = tail->stride(0);
  }
  const bool chunked = chunks.has_value() && D <= DELTA_CHUNK_MAX_D;
  at::Tensor qn = at::empty({N, G, D}, fo), kn = at::empty({N, G, D}, fo), v = at::empty({N, H, Dv}, fo),
             gates = at::empty({N, H, 2}, fo);
  const int own_tail = K > 1 && N == B ? 1 : 0, pieces = (Dv + 255) / 256;
  const int widest = std::max(D, std::min(Dv, 256));
  const int units = 2 * G + H * pieces + 1;
#define INPUTS_LAUNCH(V2_, R_, TT_)                                                                                      \
  hipLaunchKernelGGL((delta_inputs_kernel<T, V2_, R_, TT_>), dim3((unsigned)((N + TT_ - 1) / TT_), (unsigned)((units + 3) / 4)), \
                     dim3(256), 0, stream(), qn.data_ptr<float>(), kn.data_ptr<float>(), v.data_ptr<float>(),            \
                     gates.data_ptr<float>(), ptr<T>(x), (long)x.stride(0), tp.data_ptr<float>(), tlp, ts,               \
                     ptr<T>(beta_logit), (long)beta_logit.stride(0), ptr<T>(dt), (long)dt.stride(0),                     \
                     Af.data_ptr<float>(), bf.data_ptr<float>(), cu.data_ptr<int>(), start.data_ptr<int>(),              \
                     slots.data_ptr<int>(), tok_seq.data_ptr<int>(), N, G, H, D, Dv, K, pieces, own_tail,                \
                     chunked ? 1 : 0, (float)unit_eps, (float)q_scale)
#define INPUTS_ROWS(V2_, R_)                 \
  do {                                       \
    if (tt == 8) INPUTS_LAUNCH(V2_, R_, 8);  \
    else INPUTS_LAUNCH(V2_, R_, 1);          \
  } while (0)
  SERVING_DISPATCH_ACT(x, T, {
    const bool v2 = D % 2 == 0 && Dv % 2 == 0 && x.stride(0) % 2 == 0 && reinterpret_cast<uintptr_t>(x.data_ptr()) % (2 * sizeof(T)) == 0;
    const int tt = N >= 512 ? 8 : 1;
    if (v2 && widest <= 128) INPUTS_ROWS(true, 1);
    else if (v2) INPUTS_ROWS(true, 2);
    else if (widest <= 64) INPUTS_ROWS(false, 1);
    else INPUTS_ROWS(false, 4);
  });
#undef INPUTS_ROWS
#undef INPUTS_LAUNCH
  HIP_CHECK_LAST();
  if (K > 1 && !own_tail) refresh_conv_tail(x, *tail, cu, start, slots, K);
  if (chunked) {
    TORCH_CHECK(seq_chunks.has_value(), "the chunked form needs each sequence's range of chunks");
    delta_head_chunks(out, qn, kn, gates, v, state, start, slots, *chunks, *seq_chunks);
  } else {
    delta_head_scan(out, qn, kn, gates, v, state, cu, start, slots);
  }
  return out;
}

}  // namespace serving
}  // namespace cai
