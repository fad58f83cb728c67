// Update of S residual streams between two sublayers, the next sublayer's input and its norm, one
// workgroup per token row (fp32 streams [T, S, H]; or all S streams equal one row, src [T, H] or the embedding
// scale * table[ids[t]], so the first layer needs no embedding pass of its own):
//   x_t = sum_s M[s, t] src_s + p1[t] y1 + p2[t] y2
//   u = sum_t c[t] x_t,   out = u / sqrt(mean(u^2) + eps) * w,   dst_t = x_t (dst null: not written)
// y2 = a sublayer's row, or a mixture's output
//   sum_j wts[t, j] * ye[pair_slot[t * top + j]] + sigmoid(gate[t]) * shared     (wts null: ones; gate null: one)
// The coefficients [M (S x S) | p1 | p2 | c] are the same for every token (uniform loads). Every thread owns
// whole channels of all streams, so dst may be src. u waits in LDS for the row's mean square.
#include "seq_common.h"
#include "hipserve/seq_kernels.h"

namespace hipserve {
namespace {

constexpr int kNT = 256;
constexpr int kMaxStreams = 32;   // of the run-time sized instantiation

// SS streams (0: n_streams, at most kMaxStreams); V channels per thread and step (H % V == 0).
template <typename T, int SS, int V>
__global__ __launch_bounds__(kNT) void stream_update_kernel(
    T* __restrict__ out, float* dst, const float* src, bool one_row, const T* __restrict__ table,
    const long* __restrict__ ids, long vocab, float table_scale, const float* __restrict__ coef, int n_streams,
    const float* __restrict__ w, int H, float eps, const T* __restrict__ y1, const T* __restrict__ y2,
    const T* __restrict__ ye, const int* __restrict__ pair_slot, const float* __restrict__ wts, int top,
    const T* __restrict__ shared, const float* __restrict__ gate, long gate_ld) {
  extern __shared__ float us[];   // [H]
  __shared__ float red[16];
  constexpr int N = SS > 0 ? SS : kMaxStreams;
  constexpr int kUn = SS > 0 ? SS : 1;   // known stream counts stay in registers
  const int S = SS > 0 ? SS : n_streams;
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const float* M = coef;
  const float* p1 = coef + S * S;
  const float* p2 = p1 + S;
  const float* c = p2 + S;
  const float* xrow = src + t * (one_row ? 1L : (long)S) * H;
  const T* erow = table != nullptr ? table + min(max(ids[t], 0L), vocab - 1) * H : nullptr;
  const float sg = gate != nullptr ? sigmoid_f(gate[t * gate_ld]) : 1.f;
  float sq = 0.f;
  for (int e = V * tid; e < H; e += V * kNT) {
    float x[N][V];
#pragma unroll kUn
    for (int s = 0; s < S; ++s) {
      if (table == nullptr && (s == 0 || !one_row)) Row<float, V>::ld(xrow + (long)s * H + e, x[s]);
    }
    if (table != nullptr) {
      Row<T, V>::ld(erow + e, x[0]);
#pragma unroll
      for (int i = 0; i < V; ++i) x[0][i] *= table_scale;
    }
    float a[V], b[V];
#pragma unroll
    for (int i = 0; i < V; ++i) a[i] = b[i] = 0.f;
    if (y1 != nullptr) Row<T, V>::ld(y1 + t * H + e, a);
    if (y2 != nullptr) {
      Row<T, V>::ld(y2 + t * H + e, b);
    } else if (ye != nullptr) {
      float v[V];
      if (shared != nullptr) {
        Row<T, V>::ld(shared + t * H + e, v);
#pragma unroll
        for (int i = 0; i < V; ++i) b[i] = sg * v[i];
      }
      for (int j = 0; j < top; ++j) {
        const float f = wts != nullptr ? wts[t * top + j] : 1.f;
        Row<T, V>::ld(ye + (long)pair_slot[t * top + j] * H + e, v);
#pragma unroll
        for (int i = 0; i < V; ++i) b[i] = __builtin_fmaf(f, v[i], b[i]);
      }
    }
    float u[V];
#pragma unroll
    for (int i = 0; i < V; ++i) u[i] = 0.f;
#pragma unroll kUn
    for (int tt = 0; tt < S; ++tt) {
      float z[V];
      const float q1 = p1[tt], q2 = p2[tt], ct = c[tt];
#pragma unroll
      for (int i = 0; i < V; ++i) z[i] = q1 * a[i] + q2 * b[i];
#pragma unroll kUn
      for (int s = 0; s < S; ++s) {
        const float m = M[s * S + tt];
#pragma unroll
        for (int i = 0; i < V; ++i) z[i] = __builtin_fmaf(m, one_row ? x[0][i] : x[s][i], z[i]);
      }
#pragma unroll
      for (int i = 0; i < V; ++i) u[i] = __builtin_fmaf(ct, z[i], u[i]);
      if (dst != nullptr) Row<float, V>::st(dst + (t * S + tt) * H + e, z);
    }
    Row<float, V>::st(us + e, u);
#pragma unroll
    for (int i = 0; i < V; ++i) sq = __builtin_fmaf(u[i], u[i], sq);
  }
  sq = block_sum(sq, red);
  const float inv = 1.f / sqrtf(sq / (float)H + eps);
  for (int e = V * tid; e < H; e += V * kNT) {   // the thread re-reads what it wrote itself
    float u[V], wv[V];
    Row<float, V>::ld(us + e, u);
    Row<float, V>::ld(w + e, wv);
#pragma unroll
    for (int i = 0; i < V; ++i) u[i] *= inv * wv[i];
    Row<T, V>::st(out + t * H + e, u);
  }
}

}  // namespace

int stream_update_max_streams() { return kMaxStreams; }
int stream_update_max_width() { return 15000; }   // u waits in 60 KB of LDS

void launch_stream_update(void* out, float* dst, const float* src, bool one_row, const void* table, const long* ids,
                          long vocab, float table_scale, const float* coef, int S,
                          const float* w, int T, int H, float eps, const void* y1, const void* y2, const void* ye,
                          const int* pair_slot, const float* wts, int top, const void* shared, const float* gate,
                          long gate_ld, bool f32, hipStream_t s) {
  if (T <= 0) return;
  const size_t smem = (size_t)H * sizeof(float);
  const bool v4 = H % 4 == 0;
#define HS_SU(TT, SS, V)                                                                                             \
  stream_update_kernel<TT, SS, V><<<T, kNT, smem, s>>>((TT*)out, dst, src, one_row, (const TT*)table, ids, vocab,       \
                                                       table_scale, coef, S, w, H, eps, (const TT*)y1, (const TT*)y2, (const TT*)ye, pair_slot, wts, top,            \
                                                       (const TT*)shared, gate, gate_ld)
#define HS_SS(TT, V)                          \
  switch (S) {                                \
    case 1: HS_SU(TT, 1, V); break;           \
    case 2: HS_SU(TT, 2, V); break;           \
    case 3: HS_SU(TT, 3, V); break;           \
    case 4: HS_SU(TT, 4, V); break;           \
    case 5: HS_SU(TT, 5, V); break;           \
    case 6: HS_SU(TT, 6, V); break;           \
    case 7: HS_SU(TT, 7, V); break;           \
    case 8: HS_SU(TT, 8, V); break;           \
    default: HS_SU(TT, 0, 1); break;          \
  }
  if (f32) { if (v4) HS_SS(float, 4) else HS_SS(float, 1) }
  else { if (v4) HS_SS(unsigned short, 4) else HS_SS(unsigned short, 1) }
#undef HS_SS
#undef HS_SU
}

}  // namespace hipserve
