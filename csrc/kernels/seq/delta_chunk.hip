// The gated delta rule of prompt portions in chunks of 16 tokens, fp32 throughout (fp32 matrix cores):
//   S_t = diag(g_t) S_{t-1} + k_t u_t^T,  u_t = beta_t (v_t - (diag(g_t) S_{t-1})^T k_t),  o_t = S_t^T q_t
// with a decay g per key channel or per head. With G_i the product of a chunk's decays up to token i and S the
// state before the chunk,
//   u_i + beta_i sum_{j<i} A_ij u_j = beta_i (v_i - S^T (G_i k_i)),   A_ij = k_i^T diag(G_i / G_j) k_j
//   o_i = S^T (G_i q_i) + sum_{j<=i} P_ij u_j,                         P_ij = q_i^T diag(G_i / G_j) k_j
//   S' = diag(G_15) S + sum_j (G_15 / G_j k_j) u_j^T
// so a chunk costs a few small matrix products instead of 16 dependent passes over the state. The ratios G_i / G_j are
// formed as products of the decays between the two tokens (never as a quotient), so strong decays only underflow.
//
// delta_chunk_prepare: everything that does not need the state, one workgroup per (head, chunk): A, P, the inverse
// M = (1 + diag(beta) A)^-1 diag(beta) by forward substitution, and W = M (G k), U0 = M v, G q, G_15 / G k, G_15.
// delta_chunk_scan: one workgroup per (sequence, head, 16 value channels) walks the chunks: U = U0 - W S,
// o = (G q) S + P U, S = G_15 S + (G_15 / G k)^T U on mfma_f32_16x16x4f32. The state stays in registers in the
// accumulators' layout, which is also the second operand's: lane (n, g) of a 16-row tile holds rows 4 g + r of column n,
// and k step r of a product takes rows {4 g + r}.
#include "seq_common.h"
#include "hipserve/seq_kernels.h"

namespace hipserve {
namespace {

constexpr int kC = 16;   // tokens per chunk

// Chunk `id` of the step: its sequence and first token there; false past the last one.
HS_DEVICE bool find_chunk(const int* __restrict__ seq_cu, int nseq, int id, int& s, int& t0) {
  for (s = 0; s < nseq; ++s) {
    const int nc = (seq_cu[s + 1] - seq_cu[s] + kC - 1) / kC;
    if (id < nc) {
      t0 = id * kC;
      return true;
    }
    id -= nc;
  }
  return false;
}

// Buffers per (chunk, head): W, GQ [16][DP], KT [DP][16], GE [DP], UT [VP][16], P [16][16]
struct ChunkBuf {
  float *W, *GQ, *KT, *GE, *UT, *P;
};
HS_DEVICE ChunkBuf chunk_buf(float* base, long item, int DP, int VP) {
  float* p = base + item * (3L * kC * DP + DP + (long)kC * VP + kC * kC);
  ChunkBuf b;
  b.W = p;
  b.GQ = b.W + kC * DP;
  b.KT = b.GQ + kC * DP;
  b.GE = b.KT + kC * DP;
  b.UT = b.GE + DP;
  b.P = b.UT + kC * VP;
  return b;
}

// 16 DPP rows of 16 lanes: row i is token i; lane `seg` of a row owns channels 16 VD j + VD seg + e (DS in all).
template <int DS, bool CH>
__global__ __launch_bounds__(256) void delta_chunk_prepare_kernel(
    float* __restrict__ base, const float* __restrict__ qk, const float* __restrict__ vv, const float* __restrict__ gg,
    const float* __restrict__ bb, const int* __restrict__ seq_cu, int nseq, int heads, int kv_heads, int dim, int vdim,
    int VP) {
  constexpr int DP = 16 * DS, VD = DS < 4 ? DS : 4, NJ = DS / VD;
  __shared__ __attribute__((aligned(16))) float sk[kC][DP], sg[kC][DP];
  __shared__ __attribute__((aligned(16))) float sMt[kC][kC];   // [j][i]
  __shared__ float sA[kC][kC + 1], sP[kC][kC + 1], sb[kC];
  int s, t0;
  if (!find_chunk(seq_cu, nseq, blockIdx.y, s, t0)) return;
  const int h = blockIdx.x, tid = threadIdx.x, row = tid >> 4, seg = tid & 15;
  const int r0 = seq_cu[s] + t0, nt = min(kC, seq_cu[s + 1] - r0);
  const int nqk = kv_heads * dim, nv = heads * vdim, kh = h / (heads / kv_heads);
  const ChunkBuf out = chunk_buf(base, (long)blockIdx.y * heads + h, DP, VP);
  float vcol[kC];   // this thread's value channel (tid < vdim), all tokens: loaded early, used at the end
#pragma unroll
  for (int j = 0; j < kC; ++j) vcol[j] = (tid < vdim && j < nt) ? vv[(long)(r0 + j) * nv + h * vdim + tid] : 0.f;
  float xk[NJ][VD], xq[NJ][VD], g0[NJ][VD];
  const bool in = row < nt;
  const long t = r0 + (in ? row : 0);
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int c = 16 * VD * j + VD * seg;
    const float* pq = qk + t * 2 * nqk + kh * dim + c;
    const float* pg = CH ? gg + (t * heads + h) * dim + c : gg + t * heads + h;
    if (VD == 4 && dim % 4 == 0) {   // four channels are inside together, rows are 16-byte aligned
      f32x4 a = {0.f, 0.f, 0.f, 0.f}, b = a, g = {1.f, 1.f, 1.f, 1.f};
      if (in && c < dim) {
        a = *reinterpret_cast<const f32x4*>(pq + nqk);
        b = *reinterpret_cast<const f32x4*>(pq);
        if constexpr (CH) g = *reinterpret_cast<const f32x4*>(pg);
        else g = f32x4{*pg, *pg, *pg, *pg};
      }
#pragma unroll
      for (int e = 0; e < VD; ++e) { xk[j][e] = a[e]; xq[j][e] = b[e]; g0[j][e] = g[e]; }
    } else {
#pragma unroll
      for (int e = 0; e < VD; ++e) {
        const bool ok = in && c + e < dim;
        xk[j][e] = ok ? pq[nqk + e] : 0.f;
        xq[j][e] = ok ? pq[e] : 0.f;
        g0[j][e] = ok ? pg[CH ? e : 0] : 1.f;
      }
    }
    Row<float, VD>::st(&sk[row][c], xk[j]);
    Row<float, VD>::st(&sg[row][c], g0[j]);
  }
  if (seg == 0) sb[row] = in ? bb[t * heads + h] : 0.f;
  for (int i = tid; i < kC * (kC + 1); i += 256) { (&sA[0][0])[i] = 0.f; (&sP[0][0])[i] = 0.f; }
  __syncthreads();
  float yk[NJ][VD], ge[NJ][VD];
  float p = 0.f;
#pragma unroll
  for (int j = 0; j < NJ; ++j)
#pragma unroll
    for (int e = 0; e < VD; ++e) {
      yk[j][e] = xk[j][e];
      ge[j][e] = g0[j][e];
      p = __builtin_fmaf(xq[j][e], xk[j][e], p);
    }
  p = row_sum(p);
  if (seg == 0) sP[row][row] = p;
  // back through the earlier tokens: xk, xq = k_i, q_i times the decays of tokens m + 1 .. i
  for (int m = row - 1; m >= 0; --m) {
    float a = 0.f;
    p = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      float g[VD], k[VD];
      Row<float, VD>::ld(&sg[m + 1][16 * VD * j + VD * seg], g);
      Row<float, VD>::ld(&sk[m][16 * VD * j + VD * seg], k);
#pragma unroll
      for (int e = 0; e < VD; ++e) {
        xk[j][e] *= g[e];
        xq[j][e] *= g[e];
        a = __builtin_fmaf(xk[j][e], k[e], a);
        p = __builtin_fmaf(xq[j][e], k[e], p);
      }
    }
    a = row_sum(a);   // the 16 lanes of a row take the same trips
    p = row_sum(p);
    if (seg == 0) { sA[row][m] = a; sP[row][m] = p; }
  }
  // forward: yk = k_i times the decays of the later tokens; row 0 also forms the product of all of them
  for (int m = row + 1; m < kC; ++m) {
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      float g[VD];
      Row<float, VD>::ld(&sg[m][16 * VD * j + VD * seg], g);
#pragma unroll
      for (int e = 0; e < VD; ++e) { yk[j][e] *= g[e]; ge[j][e] *= g[e]; }
    }
  }
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    const int c = 16 * VD * j + VD * seg;
    float g[VD];
    Row<float, VD>::ld(&sg[0][c], g);
#pragma unroll
    for (int e = 0; e < VD; ++e) { xk[j][e] *= g[e]; xq[j][e] *= g[e]; }   // G_i k_i, G_i q_i
    Row<float, VD>::st(out.GQ + row * DP + c, xq[j]);
    if (row == 0) Row<float, VD>::st(out.GE + c, ge[j]);
  }
  __syncthreads();   // sk, sg are read, sA is written
#pragma unroll
  for (int j = 0; j < NJ; ++j) {
    Row<float, VD>::st(&sg[row][16 * VD * j + VD * seg], xk[j]);
    Row<float, VD>::st(&sk[row][16 * VD * j + VD * seg], yk[j]);
  }
  if (tid < kC) {   // column tid of M: (1 + diag(beta) A) x = beta e
    float x[kC];
#pragma unroll
    for (int i = 0; i < kC; ++i) {
      float r = 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) r = __builtin_fmaf(sA[i][j], x[j], r);
      x[i] = sb[i] * ((i == tid ? 1.f : 0.f) - r);
      sMt[tid][i] = x[i];
    }
  }
  out.P[tid] = sP[row][seg];
  __syncthreads();
  // W = M (G k)
  float w[NJ][VD];
#pragma unroll
  for (int j = 0; j < NJ; ++j)
#pragma unroll
    for (int e = 0; e < VD; ++e) w[j][e] = 0.f;
  for (int m = 0; m <= row; ++m) {
    const float f = sMt[m][row];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
      float k[VD];
      Row<float, VD>::ld(&sg[m][16 * VD * j + VD * seg], k);
#pragma unroll
      for (int e = 0; e < VD; ++e) w[j][e] = __builtin_fmaf(f, k[e], w[j][e]);
    }
  }
#pragma unroll
  for (int j = 0; j < NJ; ++j) Row<float, VD>::st(out.W + row * DP + 16 * VD * j + VD * seg, w[j]);
  // G_15 / G k, transposed
  for (int i = tid; i < DP * (kC / 4); i += 256) {
    const int c = i >> 2, q = 4 * (i & 3);
    *reinterpret_cast<f32x4*>(out.KT + 4 * i) = f32x4{sk[q][c], sk[q + 1][c], sk[q + 2][c], sk[q + 3][c]};
  }
  // U0 = M v, transposed, a value channel per thread
  for (int v = tid; v < VP; v += 256) {
    float u[kC];
#pragma unroll
    for (int i = 0; i < kC; ++i) u[i] = 0.f;
#pragma unroll
    for (int j = 0; j < kC; ++j) {
      const float x = v == tid ? vcol[j] : (v < vdim && j < nt ? vv[(long)(r0 + j) * nv + h * vdim + v] : 0.f);
#pragma unroll
      for (int i = j; i < kC; ++i) u[i] = __builtin_fmaf(sMt[j][i], x, u[i]);
    }
#pragma unroll
    for (int q = 0; q < kC; q += 4)
      *reinterpret_cast<f32x4*>(out.UT + (long)v * kC + q) = f32x4{u[q], u[q + 1], u[q + 2], u[q + 3]};
  }
}

// TPW 16-row state tiles per wave, NW waves.
template <int TPW, int NW>
__global__ __launch_bounds__(64 * NW) void delta_chunk_scan_kernel(
    float* __restrict__ o, float* __restrict__ S, float* __restrict__ base, const int* __restrict__ seq_cu,
    const int* __restrict__ seq_ctx, const int* __restrict__ seq_state, int heads, int dim, int vdim, int VP, long pad) {
  constexpr int DP = 16 * TPW * NW;
  static_assert(NW == 1 || NW == 2 || NW == 4, "the waves share the four rows of a lane");
  __shared__ __attribute__((aligned(16))) f32x4 part[2][2][NW][64];   // [chunk parity][W S | (G q) S][wave][lane]
  const int s = blockIdx.z, h = blockIdx.x, v0 = 16 * blockIdx.y;
  const int r0 = seq_cu[s], n = seq_cu[s + 1] - r0;
  if (n <= 0) return;
  int first = 0;   // the sequence's first chunk in the step
  for (int i = 0; i < s; ++i) first += (seq_cu[i + 1] - seq_cu[i] + kC - 1) / kC;
  const int nc = (n + kC - 1) / kC;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), c = lane & 15, g = lane >> 4;
  const int col = v0 + c, nv = heads * vdim;
  const bool carried = seq_ctx[s] - n > 0;
  float* Sp = S + ((long)seq_state[s] * heads + h) * dim * vdim + col;
  f32x4 st[TPW];
#pragma unroll
  for (int b = 0; b < TPW; ++b)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int k = 16 * (wave * TPW + b) + 4 * g + r;
      st[b][r] = (carried && k < dim && col < vdim) ? Sp[(long)k * vdim] : 0.f;
    }
  // Two chunks' operands, each loaded two chunks ahead as soon as its registers are free. Loads and stores of the loop are
  // unconditional (past the end the last chunk is loaded again, rows and columns that do not exist are stored behind
  // o), so that the wait for an operand never has to cover the younger loads behind it.
  struct Ops {
    f32x4 W[TPW], Q[TPW], K[TPW], E[TPW], U, P;
  } even, odd;
  auto fetch_products = [&](Ops& x, int ci) {   // what the products with the state take
    const ChunkBuf b = chunk_buf(base, (long)(first + min(ci, nc - 1)) * heads + h, DP, VP);
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      const int at = c * DP + 16 * (wave * TPW + i) + 4 * g;
      x.W[i] = *reinterpret_cast<const f32x4*>(b.W + at);
      x.Q[i] = *reinterpret_cast<const f32x4*>(b.GQ + at);
    }
  };
  auto fetch_update = [&](Ops& x, int ci) {     // what the state's update and the read-out take
    const ChunkBuf b = chunk_buf(base, (long)(first + min(ci, nc - 1)) * heads + h, DP, VP);
#pragma unroll
    for (int i = 0; i < TPW; ++i) {
      const int k0 = 16 * (wave * TPW + i);
      x.K[i] = *reinterpret_cast<const f32x4*>(b.KT + (k0 + c) * kC + 4 * g);
      x.E[i] = *reinterpret_cast<const f32x4*>(b.GE + k0 + 4 * g);
    }
    x.U = *reinterpret_cast<const f32x4*>(b.UT + (long)col * kC + 4 * g);   // col < VP
    x.P = *reinterpret_cast<const f32x4*>(b.P + c * kC + 4 * g);
  };
  auto step = [&](Ops& x, int ci) {
    f32x4 ws = {0.f, 0.f, 0.f, 0.f}, qs = ws;
#pragma unroll
    for (int b = 0; b < TPW; ++b)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        ws = __builtin_amdgcn_mfma_f32_16x16x4f32(x.W[b][r], st[b][r], ws, 0, 0, 0);
        qs = __builtin_amdgcn_mfma_f32_16x16x4f32(x.Q[b][r], st[b][r], qs, 0, 0, 0);
      }
    fetch_products(x, ci + 2);
    f32x4 u = x.U;
#pragma unroll
    for (int b = 0; b < TPW; ++b) st[b] *= x.E[b];
    f32x4 (*pt)[NW][64] = part[ci & 1];
    if constexpr (NW > 1) {
      pt[0][wave][lane] = ws;
      pt[1][wave][lane] = qs;
      __syncthreads();   // the other parity's rows are read before a wave comes here again
#pragma unroll
      for (int i = 0; i < NW; ++i) u -= pt[0][i][lane];
    } else {
      u -= ws;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int b = 0; b < TPW; ++b) st[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.K[b][r], u[r], st[b], 0, 0, 0);
    f32x4 oo = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r) oo = __builtin_amdgcn_mfma_f32_16x16x4f32(x.P[r], u[r], oo, 0, 0, 0);
    fetch_update(x, ci + 2);
#pragma unroll
    for (int k = 0; k < 4 / NW; ++k) {   // wave w reads out the rows 4 g + w (+ NW ..)
      const int r = wave + NW * k, i = ci * kC + 4 * g + r;
      float y = r == 0 ? oo[0] : r == 1 ? oo[1] : r == 2 ? oo[2] : oo[3];
      if constexpr (NW > 1) {
#pragma unroll
        for (int w = 0; w < NW; ++w) y += reinterpret_cast<const float*>(&pt[1][w][lane])[r];
      } else {
        y += r == 0 ? qs[0] : r == 1 ? qs[1] : r == 2 ? qs[2] : qs[3];
      }
      const long at = i < n && col < vdim ? (long)(r0 + i) * nv + h * vdim + col : pad + lane;
      o[at] = y;
    }
  };
  fetch_products(even, 0);
  fetch_update(even, 0);
  fetch_products(odd, 1);
  fetch_update(odd, 1);
  __builtin_amdgcn_s_waitcnt(0x0F70);   // vmcnt(0): the loop's own waits then count the loop's loads only
  for (int ci = 0; ci < nc; ci += 2) {
    step(even, ci);
    if (ci + 1 >= nc) break;
    step(odd, ci + 1);
  }
#pragma unroll
  for (int b = 0; b < TPW; ++b)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int k = 16 * (wave * TPW + b) + 4 * g + r;
      if (k < dim && col < vdim) Sp[(long)k * vdim] = st[b][r];
    }
}

int padded(int dim) { return dim <= 16 ? 16 : dim <= 32 ? 32 : dim <= 64 ? 64 : 128; }

}  // namespace

int delta_chunk_max_dim() { return 128; }
int delta_chunk_bound(int T, int nseq) { return T / kC + nseq; }

long delta_chunk_floats(int T, int nseq, int heads, int dim, int vdim) {
  const long DP = padded(dim), VP = (vdim + 15) / 16 * 16;
  return delta_chunk_bound(T, nseq) * (long)heads * (3 * kC * DP + DP + kC * VP + kC * kC);
}

void launch_delta_chunk(float* o, float* S, float* buf, const float* qk, const float* vv, const float* gg,
                        const float* bb, const int* seq_cu, const int* seq_ctx, const int* seq_state, int nseq, int T,
                        int heads, int kv_heads, int dim, int vdim, bool channel, hipStream_t s) {
  const int VP = (vdim + 15) / 16 * 16;
  dim3 pgrid(heads, delta_chunk_bound(T, nseq)), sgrid(heads, VP / 16, nseq);
#define HS_DC(DS, TPW, NW)                                                                                             \
  do {                                                                                                                 \
    if (channel)                                                                                                       \
      delta_chunk_prepare_kernel<DS, true><<<pgrid, 256, 0, s>>>(buf, qk, vv, gg, bb, seq_cu, nseq, heads, kv_heads, dim,  \
                                                                 vdim, VP);                                            \
    else                                                                                                               \
      delta_chunk_prepare_kernel<DS, false><<<pgrid, 256, 0, s>>>(buf, qk, vv, gg, bb, seq_cu, nseq, heads, kv_heads, dim, \
                                                                  vdim, VP);                                           \
    delta_chunk_scan_kernel<TPW, NW><<<sgrid, 64 * NW, 0, s>>>(o, S, buf, seq_cu, seq_ctx, seq_state, heads, dim, vdim, VP,  \
                                                               (long)T * heads * vdim);                                \
  } while (0)
  switch (padded(dim)) {
    case 16: HS_DC(1, 1, 1); break;
    case 32: HS_DC(2, 1, 2); break;
    case 64: HS_DC(4, 1, 4); break;
    default: HS_DC(8, 2, 4); break;
  }
#undef HS_DC
}

}  // namespace hipserve
