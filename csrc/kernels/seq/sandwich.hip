// Residual update between two sublayers of a design that norms every sublayer's input AND its result, one
// workgroup per token row (fp32 stream):
//   residual += mult * y / rms(y) * w_post;   out = residual / rms(residual) * w_next
// y is a sublayer's row; the two results of a parallel mixer, each normed first,
//   a_scale * a / rms(a) * a_w + b_scale * b / rms(b) * b_w;
// or a mixture's output
//   sum_j wts[t, j] * ye[pair_slot[t * top + j]] + sigmoid(gate[t]) * shared        (gate null: one)
// or nothing (the first launch: the stream starts as table_scale * table[ids[t]]). The row stays in registers
// from its first load to its last store: every input is read once, the stream read and written once.
#include "seq_common.h"
#include "hipserve/seq_kernels.h"

namespace hipserve {
namespace {

constexpr int kNT = 256;

// Two block sums at once (one barrier pair).
HS_DEVICE void block_sum2(float& x, float& y, float (*scratch)[16]) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  x = wave_sum(x);
  y = wave_sum(y);
  if (lane == 0) { scratch[0][wid] = x; scratch[1][wid] = y; }
  __syncthreads();
  float a = 0.f, b = 0.f;
#pragma unroll
  for (int w = 0; w < kNT / 64; ++w) { a += scratch[0][w]; b += scratch[1][w]; }
  __syncthreads();
  x = a;
  y = b;
}

HS_DEVICE float row_total(float v, float* scratch) {
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  v = wave_sum(v);
  if (lane == 0) scratch[wid] = v;
  __syncthreads();
  float a = 0.f;
#pragma unroll
  for (int w = 0; w < kNT / 64; ++w) a += scratch[w];
  __syncthreads();
  return a;
}

// V elements per thread and step, NS steps (H <= 256 V NS; H % V == 0).
template <typename T, int V, int NS>
__global__ __launch_bounds__(kNT) void sandwich_kernel(const SandwichUpdate p) {
  __shared__ float red[2][16];
  const long t = blockIdx.x;
  const int H = p.H, e0 = V * threadIdx.x;
  float y[NS][V], r[NS][V];
  float* res = p.residual + t * H;
  // the stream's row first: its loads fly under the sublayer's result
  const T* erow = p.table != nullptr ? (const T*)p.table + min(max(p.ids[t], 0L), p.vocab - 1) * H : nullptr;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int e = e0 + i * kNT * V;
    if (e < H) {
      if (erow != nullptr) {
        Row<T, V>::ld(erow + e, r[i]);
#pragma unroll
        for (int k = 0; k < V; ++k) r[i][k] *= p.table_scale;
      } else {
        Row<float, V>::ld(res + e, r[i]);
      }
    }
  }
  const bool has_y = p.a != nullptr || p.ye != nullptr;
  if (has_y) {
    float ss = 0.f;
    if (p.b != nullptr) {
      float z[NS][V];
      float sa = 0.f, sb = 0.f;
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int e = e0 + i * kNT * V;
        if (e < H) {
          Row<T, V>::ld((const T*)p.a + t * H + e, y[i]);
          Row<T, V>::ld((const T*)p.b + t * H + e, z[i]);
#pragma unroll
          for (int k = 0; k < V; ++k) {
            sa = __builtin_fmaf(y[i][k], y[i][k], sa);
            sb = __builtin_fmaf(z[i][k], z[i][k], sb);
          }
        }
      }
      block_sum2(sa, sb, red);
      const float fa = p.a_scale / sqrtf(sa / (float)H + p.eps), fb = p.b_scale / sqrtf(sb / (float)H + p.eps);
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int e = e0 + i * kNT * V;
        if (e < H) {
          float wa[V], wb[V];
          Row<float, V>::ld(p.a_w + e, wa);
          Row<float, V>::ld(p.b_w + e, wb);
#pragma unroll
          for (int k = 0; k < V; ++k) {
            y[i][k] = y[i][k] * fa * wa[k] + z[i][k] * fb * wb[k];
            ss = __builtin_fmaf(y[i][k], y[i][k], ss);
          }
        }
      }
    } else {
      const float sg = p.gate != nullptr ? sigmoid_f(p.gate[t * p.gate_ld]) : 1.f;
#pragma unroll
      for (int i = 0; i < NS; ++i) {
        const int e = e0 + i * kNT * V;
        if (e < H) {
          if (p.a != nullptr) {
            Row<T, V>::ld((const T*)p.a + t * H + e, y[i]);
          } else {
            float v[V];
#pragma unroll
            for (int k = 0; k < V; ++k) y[i][k] = 0.f;
            if (p.shared != nullptr) {
              Row<T, V>::ld((const T*)p.shared + t * H + e, v);
#pragma unroll
              for (int k = 0; k < V; ++k) y[i][k] = sg * v[k];
            }
            for (int j = 0; j < p.top; ++j) {
              const float f = p.wts[t * p.top + j];
              Row<T, V>::ld((const T*)p.ye + (long)p.pair_slot[t * p.top + j] * H + e, v);
#pragma unroll
              for (int k = 0; k < V; ++k) y[i][k] = __builtin_fmaf(f, v[k], y[i][k]);
            }
          }
#pragma unroll
          for (int k = 0; k < V; ++k) ss = __builtin_fmaf(y[i][k], y[i][k], ss);
        }
      }
    }
    const float f = p.mult / sqrtf(row_total(ss, red[0]) / (float)H + p.eps);
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const int e = e0 + i * kNT * V;
      if (e < H) {
        float w[V];
        Row<float, V>::ld(p.w_post + e, w);
#pragma unroll
        for (int k = 0; k < V; ++k) r[i][k] = __builtin_fmaf(y[i][k] * f, w[k], r[i][k]);
      }
    }
  }
  float sr = 0.f;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int e = e0 + i * kNT * V;
    if (e < H) {
      Row<float, V>::st(res + e, r[i]);
#pragma unroll
      for (int k = 0; k < V; ++k) sr = __builtin_fmaf(r[i][k], r[i][k], sr);
    }
  }
  const float inv = 1.f / sqrtf(row_total(sr, red[1]) / (float)H + p.eps);
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    const int e = e0 + i * kNT * V;
    if (e < H) {
      float w[V];
      Row<float, V>::ld(p.w_next + e, w);
#pragma unroll
      for (int k = 0; k < V; ++k) r[i][k] *= inv * w[k];
      Row<T, V>::st((T*)p.out + t * H + e, r[i]);
    }
  }
}

template <typename T>
void launch(const SandwichUpdate& p, hipStream_t s) {
  auto aligned = [](const void* q) { return reinterpret_cast<uintptr_t>(q) % 16 == 0; };
  const bool vec = p.H % 8 == 0 && p.H <= 8192 && aligned(p.out) && aligned(p.residual) && aligned(p.w_next) &&
                   aligned(p.w_post) && aligned(p.table) && aligned(p.a) && aligned(p.b) && aligned(p.a_w) &&
                   aligned(p.b_w) && aligned(p.ye) && aligned(p.shared);
#define HS_SW(V, NS) sandwich_kernel<T, V, NS><<<p.T, kNT, 0, s>>>(p)
  if (vec) { if (p.H <= 2048) HS_SW(8, 1); else if (p.H <= 4096) HS_SW(8, 2); else HS_SW(8, 4); }
  else if (p.H <= 1024) HS_SW(1, 4);
  else if (p.H <= 4096) HS_SW(1, 16);
  else HS_SW(1, 64);
#undef HS_SW
}

}  // namespace

int sandwich_update_max_width() { return 64 * kNT; }

void launch_sandwich_update(const SandwichUpdate& p, bool f32, hipStream_t s) {
  if (p.T <= 0) return;
  if (f32) launch<float>(p, s);
  else launch<unsigned short>(p, s);
}

}  // namespace hipserve
