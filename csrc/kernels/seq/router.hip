// Router with a selection correction: per token, s = softmax(logits) over all n router outputs, or the sigmoid
// of each (fp32); the `top` outputs with the largest s + correction are chosen (ties: the lower
// index); wts = s * scale of the chosen ones, ids = their index, where every index >= E (an
// expert without weights) is written as E, so the expert alignment sees them as one bucket that
// no GEMM tile serves. One wave per token, output e on lane e % 64, slot e / 64 (n <= 256).
// groups > 1 (at most 64): the outputs form equal groups of neighbours; a group scores the largest
// corrected score in it, or with top2 the sum of its two largest (of the scores s alone without a correction;
// group g's on lane g), and the outputs outside the `keep` best groups (ties:
// the lower group) cannot be chosen. Without a correction the choice is made by the logits, which have the order of
// s but do not saturate. renorm: the chosen scores are divided by their sum + 1e-20.
#include "seq_common.h"
#include "hipserve/seq_kernels.h"

namespace hipserve {
namespace {

constexpr int kSlots = 4;

// One wave routes token t; ids_row / wts_row take its `top` choices, lds_ids (may be null) the ids once more.
HS_DEVICE void route_token(int* __restrict__ ids_row, float* __restrict__ wts_row, int* lds_ids,
                           const float* __restrict__ row, const float* __restrict__ correction, int n, int top,
                           float scale, int E, int groups, int keep, bool renorm, bool sigmoid, bool top2) {
  const int lane = threadIdx.x & 63;
  float p[kSlots], c[kSlots];
  float z[kSlots];
  float mx = -INFINITY;
#pragma unroll
  for (int s = 0; s < kSlots; ++s) {
    const int e = lane + 64 * s;
    z[s] = e < n ? row[e] : -INFINITY;
    mx = fmaxf(mx, z[s]);
  }
  mx = wave_max(mx);
  float sum = 0.f;
#pragma unroll
  for (int s = 0; s < kSlots; ++s) {
    p[s] = lane + 64 * s < n ? (sigmoid ? sigmoid_f(z[s]) : expf(z[s] - mx)) : 0.f;
    sum += p[s];
  }
  sum = sigmoid ? 1.f : wave_sum(sum);
#pragma unroll
  for (int s = 0; s < kSlots; ++s) {
    const int e = lane + 64 * s;
    p[s] = p[s] / sum;
    c[s] = e < n ? (correction != nullptr ? p[s] + correction[e] : z[s]) : -INFINITY;
  }
  if (groups > 1) {
    const int per = n / groups;
    float gbest = -INFINITY;   // lane g: group g's score
    for (int g = 0; g < groups; ++g) {
      float v = -INFINITY;
      if (!top2) {
#pragma unroll
        for (int s = 0; s < kSlots; ++s)
          if ((lane + 64 * s) / per == g) v = fmaxf(v, c[s]);
        v = wave_max(v);
      } else {
        // the largest and the second largest (ties count as two) of the lanes' own largest pairs
        float a = -INFINITY, b = -INFINITY;
#pragma unroll
        for (int s = 0; s < kSlots; ++s) {
          const int e = lane + 64 * s;
          if (e / per == g && e < n) {
            const float x = correction != nullptr ? c[s] : p[s];
            b = fmaxf(b, fminf(a, x));
            a = fmaxf(a, x);
          }
        }
        v = wave_max(a);
        if (per > 1) {
          const int who = __builtin_ctzll(__ballot(a == v));
          v += wave_max(lane == who ? b : a);
        }
      }
      if (lane == g) gbest = v;
    }
    unsigned long long allowed = 0;
    for (int j = 0; j < keep; ++j) {
      const float best = wave_max(gbest);
      const unsigned long long b = __ballot(gbest == best && lane < groups);
      if (!b) break;
      const int who = __builtin_ctzll(b);
      allowed |= 1ull << who;
      if (lane == who) gbest = -INFINITY;
    }
#pragma unroll
    for (int s = 0; s < kSlots; ++s) {
      const int e = lane + 64 * s;
      if (e < n && !((allowed >> (e / per)) & 1ull)) c[s] = -INFINITY;
    }
  }
  int mine[kSlots];
#pragma unroll
  for (int s = 0; s < kSlots; ++s) mine[s] = -1;
  float chosen = 0.f;
  for (int j = 0; j < top; ++j) {
    float best = -INFINITY;
#pragma unroll
    for (int s = 0; s < kSlots; ++s) best = fmaxf(best, c[s]);
    best = wave_max(best);
    // the lowest index holding the best value: slot 0 holds outputs 0..63, slot 1 the next 64, ...
    int who = -1;
#pragma unroll
    for (int s = 0; s < kSlots; ++s) {
      const unsigned long long b = __ballot(c[s] == best);
      if (who < 0 && b) who = 64 * s + __builtin_ctzll(b);
    }
#pragma unroll
    for (int s = 0; s < kSlots; ++s) {
      if (who == lane + 64 * s) {
        ids_row[j] = min(who, E);
        if (lds_ids != nullptr) lds_ids[j] = min(who, E);
        mine[s] = j;
        chosen += p[s];
        c[s] = -INFINITY;
      }
    }
  }
  const float f = renorm ? scale / (wave_sum(chosen) + 1e-20f) : scale;
#pragma unroll
  for (int s = 0; s < kSlots; ++s)
    if (mine[s] >= 0) wts_row[mine[s]] = p[s] * f;
}

__global__ __launch_bounds__(256) void route_topk_kernel(int* __restrict__ ids, float* __restrict__ wts,
                                                         const float* __restrict__ logits, long ld,
                                                         const float* __restrict__ correction, int T, int n, int top,
                                                         float scale, int E, int groups, int keep, bool renorm,
                                                         bool sigmoid, bool top2) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= T) return;
  route_token(ids + (long)t * top, wts + (long)t * top, nullptr, logits + (long)t * ld, correction, n, top, scale, E,
              groups, keep, renorm, sigmoid, top2);
}

// ---- router and alignment of a small batch in one workgroup: the choices go to LDS, pair p's place among the
// pairs of its bucket is the number of earlier pairs there (as many LDS reads as there are pairs), and the
// tables are put together in LDS and written once.
constexpr int kAlignThreads = 1024, kMaxPairs = 256, kMaxBuckets = 128, kMaxSlots = 8192;

__global__ __launch_bounds__(kAlignThreads) void route_align_kernel(
    int* __restrict__ ids, float* __restrict__ wts, int* __restrict__ slots, int cap, int* __restrict__ tile_expert,
    int tile, int* __restrict__ pair_slot, const float* __restrict__ logits, long ld,
    const float* __restrict__ correction, int T, int n, int top, float scale, int E, int nb, int groups, int keep,
    bool renorm, bool sigmoid, bool top2) {
  __shared__ int sid[kMaxPairs], cnt[kMaxBuckets], off[kMaxBuckets];
  extern __shared__ int tab[];   // [cap] slots, [cap / tile] experts
  const int tid = threadIdx.x, P = T * top, nt = cap / tile;
  for (int t = tid >> 6; t < T; t += kAlignThreads / 64)
    route_token(ids + (long)t * top, wts + (long)t * top, sid + t * top, logits + (long)t * ld, correction, n, top, scale,
                E, groups, keep, renorm, sigmoid, top2);
  for (int i = tid; i < cap + nt; i += kAlignThreads) tab[i] = -1;
  __syncthreads();
  int rank = 0;
  if (tid < P) {
    const int e = sid[tid];
    for (int p = 0; p < tid; ++p) rank += sid[p] == e;
  } else if (tid >= 512 && tid < 512 + nb) {
    int c = 0;
    for (int p = 0; p < P; ++p) c += sid[p] == tid - 512;
    cnt[tid - 512] = (c + tile - 1) / tile;   // tiles of the bucket
  }
  __syncthreads();
  if (tid < nb) {
    int at = 0;
    for (int e = 0; e < tid; ++e) at += cnt[e];
    off[tid] = at;
    for (int k = 0; k < cnt[tid]; ++k) tab[cap + at + k] = tid;
  }
  __syncthreads();
  if (tid < P) {
    const int slot = off[sid[tid]] * tile + rank;
    tab[slot] = tid;
    pair_slot[tid] = slot;
  }
  __syncthreads();
  for (int i = tid; i < cap; i += kAlignThreads) slots[i] = tab[i];
  for (int i = tid; i < nt; i += kAlignThreads) tile_expert[i] = tab[cap + i];
}

}  // namespace

int route_align_max_pairs() { return kMaxPairs; }
int route_align_max_slots() { return kMaxSlots; }

void launch_route_align(int* ids, float* wts, int* slots, int cap, int* tile_expert, int tile, int* pair_slot,
                        const float* logits, long ld, const float* correction, int T, int n, int top, float scale, int E,
                        int nb, int groups, int keep, bool renorm, bool sigmoid, bool top2, hipStream_t s) {
  if (T <= 0) return;
  route_align_kernel<<<1, kAlignThreads, (size_t)(cap + cap / tile) * sizeof(int), s>>>(
      ids, wts, slots, cap, tile_expert, tile, pair_slot, logits, ld, correction, T, n, top, scale, E, nb, groups, keep,
      renorm, sigmoid, top2);
}

int route_topk_max_outputs() { return 64 * kSlots; }

void launch_route_topk(int* ids, float* wts, const float* logits, long ld, const float* correction, int T, int n,
                       int top, float scale, int E, int groups, int keep, bool renorm, bool sigmoid, bool top2,
                       hipStream_t s) {
  if (T <= 0) return;
  route_topk_kernel<<<(T + 3) / 4, 256, 0, s>>>(ids, wts, logits, ld, correction, T, n, top, scale, E, groups, keep, renorm,
                                               sigmoid, top2);
}

}  // namespace hipserve
