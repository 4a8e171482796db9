// Split-key paged attention with a key block's rows in registers (decode tokens, float32 serving).
//
// One block per (token, kv head, group of up to RC query heads of that kv head); its waves take every nw-th key block.
// A row is covered by L lanes (a power of two) of 32 bytes each, so a wave's load instruction reads 64 / L whole rows,
// and a key block is NS such steps. All page lookups and then all row loads of a block are issued before the first
// product. Lane group g holds key g of every step, for the scores and for the weighted sum alike:
//   * the scores of a step meet across the L lanes of a row (DPP);
//   * every lane group runs an online softmax of its own over its keys — nothing crosses lane groups in the loop;
//   * the weighted sum uses the values in the same lanes. Where the values are the keys (or their leading channels)
//     they are the registers the scores were formed from: each cached row is read once.
// The lane groups' states meet in a butterfly, the waves' states in LDS, at the end.
#include "paged_attention.h"

namespace cai {
namespace serving {

typedef int int4v_ __attribute__((ext_vector_type(4)));

constexpr int ROW_WAVES = 8;

template <typename T> struct RowLane;   // CH channels = 32 bytes per lane, as two 16-byte pieces
template <> struct RowLane<bf16s> {
  static constexpr int CH = 16;
  DEV_INLINE static void unpack(const int4v_& p, float* o) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      o[2 * e] = __builtin_bit_cast(float, p[e] << 16);
      o[2 * e + 1] = __builtin_bit_cast(float, p[e] & (int)0xffff0000);
    }
  }
};
template <> struct RowLane<float> {
  static constexpr int CH = 8;
  DEV_INLINE static void unpack(const int4v_& p, float* o) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int bits = p[e];  // a bit cast of the vector element itself takes element 0
      o[e] = __builtin_bit_cast(float, bits);
    }
  }
};

template <typename T, int RC, int NS, bool SEP>
__global__ __launch_bounds__(64 * ROW_WAVES) void row_attention_kernel(
    T* __restrict__ out, float* __restrict__ out32, const T* __restrict__ q, long q_stride, const T* __restrict__ kpool,
    const T* __restrict__ vpool, const int* __restrict__ block_tables, int bt_stride, const int* __restrict__ tok_seq,
    const int* __restrict__ positions, const float* __restrict__ slopes, const T* __restrict__ gate, long gate_stride,
    const float* __restrict__ sink_logits, const float* __restrict__ key_fac, int H, int G, int D, int Dv, int page_shift,
    float scale, int window, int keep_first, int chunk, float softcap, int sink, int vrep, long vrow, long vhead,
    int lane_shift, int qvec) {
  constexpr int CH = RowLane<T>::CH, HC = CH / 2;
  extern __shared__ __align__(16) float lds[];
  const int wid = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = blockDim.x >> 6;
  const int R = H / G, chunks = (R + RC - 1) / RC;
  const long n = blockIdx.x / (G * chunks);
  const int g = (int)(blockIdx.x / chunks) % G;
  const int h0 = g * R + (int)(blockIdx.x % chunks) * RC;
  const int nh = min(RC, g * R + R - h0);
  const int L = 1 << lane_shift;
  const int ch = (lane & (L - 1)) * CH;             // this lane's first channel
  const int group = lane >> lane_shift, KPS = 64 >> lane_shift, KB = NS * KPS;
  const int pos = positions[n];
  const int* bt = block_tables + (long)tok_seq[n] * bt_stride;
  const int page_mask = (1 << page_shift) - 1;
  float* coef = lds;                                // [RC][ROW_WAVES]
  float* part = lds + RC * ROW_WAVES;               // [nw][RC][2 + Dv]

  float qf[RC][CH], slope[RC];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    slope[r] = (slopes != nullptr && r < nh) ? slopes[h0 + r] : 0.0f;
    const T* qp = q + n * q_stride + (long)(h0 + r) * D + ch;
    if (qvec) {
      const int4v_ none = {0, 0, 0, 0};
      RowLane<T>::unpack(r < nh && ch < D ? *reinterpret_cast<const int4v_*>(qp) : none, qf[r]);
      RowLane<T>::unpack(r < nh && ch + HC < D ? *reinterpret_cast<const int4v_*>(qp + HC) : none, qf[r] + HC);
    } else {
#pragma unroll
      for (int c = 0; c < CH; ++c) qf[r][c] = r < nh && ch + c < D ? ldf(qp + c) : 0.0f;
    }
#pragma unroll
    for (int c = 0; c < CH; ++c) qf[r][c] *= scale;
  }
  const int lo = first_visible(pos, window, chunk);
  const int n_keep = window > 0 ? min(keep_first, lo) : 0;
  const int total = n_keep + (pos - lo + 1);
  const float inv_cap = softcap > 0.0f ? 1.0f / softcap : 0.0f;
  const T* vbase = SEP ? vpool + (long)(g / vrep) * vhead : nullptr;

  float m[RC], l[RC], acc[RC][CH];
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    m[r] = -INFINITY;
    l[r] = 0.0f;
#pragma unroll
    for (int c = 0; c < CH; ++c) acc[r][c] = 0.0f;
  }
  const int4v_ zero = {0, 0, 0, 0};
  for (int base = wid * KB; base < total; base += nw * KB) {
    int j[NS];
    long row[NS];
    float fac[NS];
    int4v_ kr[NS][2], vr[SEP ? NS : 1][2];
#pragma unroll
    for (int s = 0; s < NS; ++s) {                  // a key past the end reads the query's own row and is masked
      const int idx = base + s * KPS + group;
      j[s] = idx < total ? (idx < n_keep ? idx : lo + (idx - n_keep)) : pos;
      row[s] = ((long)bt[j[s] >> page_shift] << page_shift) + (j[s] & page_mask);
    }
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const bool some = base + s * KPS < total;     // the wave's step holds a key
      const T* kp = kpool + (row[s] * G + g) * D + ch;
      kr[s][0] = some && ch < D ? *reinterpret_cast<const int4v_*>(kp) : zero;
      kr[s][1] = some && ch + HC < D ? *reinterpret_cast<const int4v_*>(kp + HC) : zero;
      fac[s] = key_fac != nullptr && some ? key_fac[row[s] * G + g] : 1.0f;
      if constexpr (SEP) {
        const T* vp = vbase + row[s] * vrow + ch;
        vr[s][0] = some && ch < Dv ? *reinterpret_cast<const int4v_*>(vp) : zero;
        vr[s][1] = some && ch + HC < Dv ? *reinterpret_cast<const int4v_*>(vp + HC) : zero;
      }
    }
    float sc[RC][NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      float kf[CH];
      RowLane<T>::unpack(kr[s][0], kf);
      RowLane<T>::unpack(kr[s][1], kf + HC);
#pragma unroll
      for (int r = 0; r < RC; ++r) {
        float d = 0.0f;
#pragma unroll
        for (int c = 0; c < CH; ++c) d += qf[r][c] * kf[c];
        sc[r][s] = d;
      }
    }
#define ROW_REDUCE(STAGE, EXPR)                        \
  if (lane_shift > STAGE) {                            \
    _Pragma("unroll") for (int r = 0; r < RC; ++r)     \
        _Pragma("unroll") for (int s = 0; s < NS; ++s) { const float v = sc[r][s]; sc[r][s] = EXPR; } \
  }
    ROW_REDUCE(0, dpp_add<0xB1>(v))           // lane xor 1
    ROW_REDUCE(1, dpp_add<0x4E>(v))           // lane xor 2
    ROW_REDUCE(2, dpp_add<0x141>(v))          // the other half of 8 lanes
    ROW_REDUCE(3, dpp_add<0x140>(v))          // the other half of 16 lanes
    ROW_REDUCE(4, v + __shfl_xor(v, 16))
    ROW_REDUCE(5, v + __shfl_xor(v, 32))
#undef ROW_REDUCE
#pragma unroll
    for (int r = 0; r < RC; ++r) {
      float top = m[r];
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        float v = sc[r][s] * fac[s];
        if (softcap > 0.0f) v = softcap * tanhf(v * inv_cap);
        v -= slope[r] * (float)(pos - j[s]);
        sc[r][s] = base + s * KPS + group < total ? v : -INFINITY;
        top = fmaxf(top, sc[r][s]);
      }
      const float ref = top == -INFINITY ? 0.0f : top;   // no key in this lane group yet
      const float corr = expf(m[r] - ref);
      m[r] = top;
      float sum = 0.0f;
#pragma unroll
      for (int s = 0; s < NS; ++s) {
        sc[r][s] = expf(sc[r][s] - ref);
        sum += sc[r][s];
      }
      l[r] = l[r] * corr + sum;
#pragma unroll
      for (int c = 0; c < CH; ++c) acc[r][c] *= corr;
    }
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      // keep the packed registers, not 2 CH floats per step, alive since the scores: unpack anew
      if constexpr (!SEP) asm volatile("" : "+v"(kr[s][0]), "+v"(kr[s][1]));
      float vf[CH];
      RowLane<T>::unpack(SEP ? vr[SEP ? s : 0][0] : kr[s][0], vf);
      RowLane<T>::unpack(SEP ? vr[SEP ? s : 0][1] : kr[s][1], vf + HC);
#pragma unroll
      for (int r = 0; r < RC; ++r)
#pragma unroll
        for (int c = 0; c < CH; ++c) acc[r][c] += sc[r][s] * vf[c];
    }
  }
  const int PS = 2 + Dv;
#pragma unroll
  for (int r = 0; r < RC; ++r) {
    float top = m[r];
    for (int off = L; off < 64; off <<= 1) top = fmaxf(top, __shfl_xor(top, off));
    const float f = m[r] == -INFINITY ? 0.0f : expf(m[r] - top);
    float ll = l[r] * f;
    for (int off = L; off < 64; off <<= 1) ll += __shfl_xor(ll, off);
#pragma unroll
    for (int c = 0; c < CH; ++c) acc[r][c] *= f;
    for (int off = L; off < 64; off <<= 1) {
#pragma unroll
      for (int c = 0; c < CH; ++c) acc[r][c] += __shfl_xor(acc[r][c], off);
    }
    float* mine = part + (wid * RC + r) * PS;
    if (lane == 0) { mine[0] = top; mine[1] = ll; }
    if (group == 0) {
#pragma unroll
      for (int c = 0; c < CH; ++c)
        if (ch + c < Dv) mine[2 + ch + c] = acc[r][c];
    }
  }
  __syncthreads();
  if (wid < nh) {  // wave r: what each wave's partial state counts in head r
    const int r = wid;
    const float mw = lane < nw ? part[(lane * RC + r) * PS] : -INFINITY;
    const float lw = lane < nw ? part[(lane * RC + r) * PS + 1] : 0.0f;
    float top = wave_reduce_max(mw);
    if (sink_logits != nullptr) top = fmaxf(top, sink_logits[h0 + r]);
    const float f = mw == -INFINITY ? 0.0f : expf(mw - top);
    float ll = wave_reduce_sum(lw * f);
    if (sink_logits != nullptr) ll += expf(sink_logits[h0 + r] - top);
    else if (sink) ll += expf(-top);   // the sink's score is 0
    float c = f / ll;
    if (gate != nullptr) c *= sigmoidf_(ldf(gate + n * gate_stride + h0 + r));
    if (lane < nw) coef[r * ROW_WAVES + lane] = c;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < nh * Dv; i += blockDim.x) {
    const int r = i / Dv, dv = i % Dv;
    float o = 0.0f;
#pragma unroll 4
    for (int w = 0; w < nw; ++w) o += coef[r * ROW_WAVES + w] * part[(w * RC + r) * PS + 2 + dv];
    const long at = (n * H + h0 + r) * (long)Dv + dv;
    if (out32 != nullptr) out32[at] = o;
    else stf(out + at, o);
  }
}

bool launch_row_attention(at::Tensor& out, const at::Tensor& q, const at::Tensor& kpool, const at::Tensor& vpool,
                          const at::Tensor& block_tables, const at::Tensor& tok_seq, const at::Tensor& positions,
                          const float* slopes, const c10::optional<at::Tensor>& gate, long gate_stride, double scale,
                          int64_t window, int64_t keep_first, double softcap, bool sink, int page_shift, long vrow,
                          long vhead, const ScalarExtras& x) {
  const long N = q.size(0);
  const int H = (int)q.size(1), D = (int)q.size(2), G = (int)kpool.size(2), Dv = (int)vpool.size(3);
  if (x.dist_bias != nullptr || x.ksum != nullptr || x.cross_out != nullptr) return false;
  const int elem = is_bf16(q) ? 2 : 4, piece = 16 / elem, CH = 2 * piece;
  auto al16 = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  if (D % piece != 0 || !al16(kpool.data_ptr()) || D > 64 * CH || Dv > 64 * CH) return false;
  const bool shared = vpool.data_ptr() == kpool.data_ptr() && vrow == (long)G * D && (G == 1 || vhead == D) && Dv <= D &&
                      x.vrep == 1;
  if (!shared && (Dv % piece != 0 || vrow % piece != 0 || vhead % piece != 0 || !al16(vpool.data_ptr()))) return false;
  int lane_shift = 0;
  while ((CH << lane_shift) < (D > Dv ? D : Dv)) ++lane_shift;
  const int R = H / G;
  int rc = R > 1 && N * G * ((R + 1) / 2) >= 256 ? 2 : 1;   // two heads share a block's rows when enough blocks cover the CUs
  auto lds_bytes = [&](int nw) { return (size_t)(rc * ROW_WAVES + nw * rc * (2 + Dv)) * sizeof(float); };
  int nwaves = ROW_WAVES;
  while (lds_bytes(nwaves) > 64 * 1024 && nwaves > 4) nwaves >>= 1;
  while (lds_bytes(nwaves) > 64 * 1024 && rc > 1) rc >>= 1;
  if (lds_bytes(nwaves) > 64 * 1024) return false;
  const int chunks = (R + rc - 1) / rc;
  const int qvec = al16(q.data_ptr()) && q.stride(0) % piece == 0 ? 1 : 0;
#define ROW_LAUNCH(RC_, NS_, SEP_)                                                                                     \
  hipLaunchKernelGGL((row_attention_kernel<T, RC_, NS_, SEP_>), dim3((unsigned)(N * G * chunks)), dim3(64 * nwaves),    \
                     lds_bytes(nwaves), stream(), x.out32 != nullptr ? (T*)nullptr : ptr<T>(out), x.out32, ptr<T>(q),   \
                     (long)q.stride(0), ptr<T>(kpool), ptr<T>(vpool), block_tables.data_ptr<int>(),                     \
                     (int)block_tables.stride(0), tok_seq.data_ptr<int>(), positions.data_ptr<int>(), slopes,           \
                     gate.has_value() ? ptr<T>(*gate) : (const T*)nullptr, gate_stride, x.sink_logits, x.key_fac, H, G, \
                     D, Dv, page_shift, (float)scale, (int)window, (int)keep_first, x.chunk, (float)softcap,            \
                     sink ? 1 : 0, x.vrep, vrow, vhead, lane_shift, qvec)
  SERVING_DISPATCH_ACT(q, T, {
    if (shared) {
      if (rc == 1) ROW_LAUNCH(1, 8, false);
      else ROW_LAUNCH(2, 8, false);
    } else {
      if (rc == 1) ROW_LAUNCH(1, 8, true);
      else ROW_LAUNCH(2, 4, true);
    }
  });
#undef ROW_LAUNCH
  HIP_CHECK_LAST();
  return true;
}

}  // namespace serving
}  // namespace cai
