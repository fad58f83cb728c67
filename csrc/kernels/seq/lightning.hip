// Linear attention with one fixed decay per head over per-sequence state slots (S [dim, vdim] per head, fp32):
//   q, k, v <- SiLU of their projections;  S <- lam S + k v^T;  o = S^T q
//   out = o / sqrt(mean(o^2) + eps) * w * sigmoid(gate) * out_scale     (the norm over ALL heads of a token)
// A step that starts at position 0 starts from S = 0. Rows of the projection: [q | k | v | gate], head by head.
// powers[h][n] = lam_h^n, n = 0 .. 64.
//
// Prompt portions, bf16: lightning_chunk, 64 tokens at a time on the matrix cores. For query i and key j of a chunk
//   o_i = lam^(i+1) S^T q_i + sum_{j <= i} lam^(i-j) (q_i . k_j) v_j
//   S' = lam^m S + sum_j lam^(m-1-j) k_j v_j^T                          (m tokens in the chunk)
// Few long sequences would leave most of the chip idle, so they are cut into segments that run side by side:
// lightning_chunk<.., true> sums every segment's own keys and values, lightning_carry turns those sums into the
// state before each segment (one pass over them in order), and the segments then run as sequences of their own.
// The state stays in fp32 accumulator registers from the first chunk to the last. Whatever carries a decay or the
// state enters an MFMA as the sum of two bf16 numbers (the rounding and what it left), so the products see it
// to 16 bits; q, k and v are bf16 like every activation.
// Prompt portions, fp32 (and head sizes the chunk kernel does not take): lightning_stage (SiLU, dense fp32 rows) and
// lightning_scan, token by token: a state column in the registers of the 16 lanes of a DPP row.
// Decode rows (one per sequence): lightning_step, a workgroup per (sequence, head, block of state columns); the
// state is read and written once, coalesced.
// All of them write o as fp32 rows [T, heads * vdim]; lightning_out (one workgroup per token) norms and gates.
#include "seq_common.h"
#include "hipserve/seq_kernels.h"

namespace hipserve {
namespace {

HS_DEVICE float silu_f(float x) { return x * sigmoid_f(x); }
HS_DEVICE float silu_fast(float x) {   // for values that are rounded to bf16 next
  return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.44269504088896341f * x));
}

constexpr int kPowers = 65;   // lam^0 .. lam^64

// ---------------------------------------------------------------- staging + scan
// qk[t, h] = [q (dim) | k (dim)], vv[t, h] = v (vdim)
template <typename T>
__global__ __launch_bounds__(256) void lightning_stage_kernel(float* __restrict__ qk, float* __restrict__ vv,
                                                             const T* __restrict__ proj, long ld, int heads, int dim,
                                                             int vdim) {
  const long t = blockIdx.x;
  const T* row = proj + t * ld;
  const int nqk = heads * dim, nv = heads * vdim;
  for (int e = threadIdx.x; e < nqk; e += 256) {
    const int h = e / dim, i = e - h * dim;
    float* dst = qk + (t * heads + h) * 2 * dim;
    dst[i] = silu_f(ldf<T>(row, e));
    dst[dim + i] = silu_f(ldf<T>(row, nqk + e));
  }
  for (int e = threadIdx.x; e < nv; e += 256) vv[t * nv + e] = silu_f(ldf<T>(row, 2L * nqk + e));
}

constexpr int kTB = 8;     // tokens staged at a time
constexpr int kSeg = 16;   // lanes that share a state column (one DPP row)
constexpr int kScanThreads = 256;
constexpr int kCols = kScanThreads / kSeg;  // state columns per workgroup

HS_DEVICE float row_sum(float v) {
  v = dpp_step<0xB1, 0xf, false>(v);   // quad_perm [1, 0, 3, 2]
  v = dpp_step<0x4E, 0xf, false>(v);   // quad_perm [2, 3, 0, 1]
  v = dpp_step<0x141, 0xf, false>(v);  // row_half_mirror
  return dpp_step<0x140, 0xf, false>(v);  // row_mirror
}

// grid (heads, ceil(vdim / kCols), sequences); dim <= 16 DS.
template <int DS>
__global__ __launch_bounds__(kScanThreads) void lightning_scan_kernel(
    float* __restrict__ o, float* __restrict__ S, const float* __restrict__ qk, const float* __restrict__ vv,
    const float* __restrict__ powers, const int* __restrict__ seq_cu, const int* __restrict__ seq_ctx,
    const int* __restrict__ seq_state, int heads, int dim, int vdim) {
  constexpr int DP = kSeg * DS;
  __shared__ __attribute__((aligned(16))) float sq[kTB][DP], sk[kTB][DP];
  const int s = blockIdx.z, h = blockIdx.x, tid = threadIdx.x;
  const int r0 = seq_cu[s], n = seq_cu[s + 1] - r0;
  if (n <= 0) return;
  const int seg = tid & (kSeg - 1), k0 = seg * DS;
  const int c = blockIdx.y * kCols + tid / kSeg;   // this lane row's column
  const bool has_col = c < vdim;
  float* Sp = S + (((long)seq_state[s] * heads + h) * dim) * vdim;
  const bool carried = seq_ctx[s] - n > 0;
  const float lam = powers[h * kPowers + 1];
  float st[DS];
#pragma unroll
  for (int i = 0; i < DS; ++i) st[i] = (carried && has_col && k0 + i < dim) ? Sp[(long)(k0 + i) * vdim + c] : 0.f;
  constexpr int kLd = (kTB * DP + kScanThreads - 1) / kScanThreads;
  float rq[kLd], rk[kLd], rv[kTB];
  auto fetch = [&](int t0) {
    const int nt = min(kTB, n - t0);
#pragma unroll
    for (int it = 0; it < kLd; ++it) {
      const int i = it * kScanThreads + tid;
      const int tt = i / DP, k = i % DP;
      const float* row = qk + ((long)(r0 + t0 + tt) * heads + h) * 2 * dim;
      const bool in = tt < nt && k < dim;
      rq[it] = in ? row[k] : 0.f;
      rk[it] = in ? row[dim + k] : 0.f;
    }
#pragma unroll
    for (int tt = 0; tt < kTB; ++tt)
      rv[tt] = (tt < nt && has_col) ? vv[((long)(r0 + t0 + tt) * heads + h) * vdim + c] : 0.f;
  };
  float* po = o + ((long)r0 * heads + h) * vdim + c;
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += kTB) {
    const int nt = min(kTB, n - t0);
    __syncthreads();
#pragma unroll
    for (int it = 0; it < kLd; ++it) {
      const int i = it * kScanThreads + tid;
      if (i < kTB * DP) {
        sq[i / DP][i % DP] = rq[it];
        sk[i / DP][i % DP] = rk[it];
      }
    }
    float val[kTB];
#pragma unroll
    for (int tt = 0; tt < kTB; ++tt) val[tt] = rv[tt];
    __syncthreads();
    if (t0 + kTB < n) fetch(t0 + kTB);
#pragma unroll
    for (int tt = 0; tt < kTB; ++tt) {
      if (tt < nt) {
        float out = 0.f, out2 = 0.f;
#pragma unroll
        for (int i = 0; i < DS; ++i) {
          st[i] = __builtin_fmaf(lam, st[i], val[tt] * sk[tt][k0 + i]);
          if (i & 1) out2 = __builtin_fmaf(st[i], sq[tt][k0 + i], out2);
          else out = __builtin_fmaf(st[i], sq[tt][k0 + i], out);
        }
        const float r = row_sum(out + out2);
        if (seg == 0 && has_col) po[(long)(t0 + tt) * heads * vdim] = r;
      }
    }
  }
#pragma unroll
  for (int i = 0; i < DS; ++i)
    if (has_col && k0 + i < dim) Sp[(long)(k0 + i) * vdim + c] = st[i];
}

// ---------------------------------------------------------------- chunks on the matrix cores
constexpr int kC = 64;         // tokens per chunk
constexpr int kTLd = kC + 8;   // row stride of the token-minor tiles (elements; rows stay 16-byte aligned)

// Column of token tt (0 .. 63) in the token-minor tiles: the 32 tokens of a block in the order in which the score
// registers of lane group g hold them (16 a + 4 g + b at 8 g + 4 a + b), so the weights are MFMA operands as
// they are; the state update sums over tokens and takes any order that both its operands share.
HS_DEVICE int tok_col(int tt) { return (tt & 32) + 8 * ((tt >> 2) & 3) + 4 * ((tt >> 4) & 1) + (tt & 3); }

template <int KS, int NT, bool SUM>
constexpr size_t chunk_lds() {
  const size_t both = (2 * 32 * KS + 16 * NT) * kTLd * 2 + (kPowers + 3) * sizeof(float);
  return SUM ? both : both + ((size_t)kC * (32 * KS + 8) + 2 * 16 * NT * (32 * KS + 8)) * 2;
}

// grid (heads, ceil(vdim / (16 NT)), sequences x nseg), 4 waves. dim <= 32 KS; dim % 8 == 0, vdim % 8 == 0. Wave w owns
// the chunk's query rows 16 w .. 16 w + 15 (scores and outputs never leave its registers) and the state rows
// 16 DT w .. (the rest of the update). nseg > 1: segment z % nseg of sequence z / nseg, seg_len tokens (a multiple
// of 64) from the state ws[z, head]; the last segment's last state goes into the slot. SUM: only the state update,
// from zero, for every segment but a sequence's last; the sum goes to ws[z, head].
template <int KS, int NT, bool SUM>
__global__ __launch_bounds__(256) void lightning_chunk_kernel(
    float* __restrict__ o, float* __restrict__ S, const unsigned short* __restrict__ proj, long ld,
    const float* __restrict__ powers, const int* __restrict__ seq_cu, const int* __restrict__ seq_ctx,
    const int* __restrict__ seq_state, int heads, int dim, int vdim, float* __restrict__ ws, int nseg, int seg_len) {
  constexpr int DP = 32 * KS, KLd = DP + 8, VB = 16 * NT;
  constexpr int DT = KS >= 2 ? KS / 2 : 1;   // 16-row state tiles per wave
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  unsigned short* kth = reinterpret_cast<unsigned short*>(smem);   // [dim][token] lam^(m-1-j) k_j, rounded ...
  unsigned short* ktl = kth + DP * kTLd;  // ... and the rest
  unsigned short* vt = ktl + DP * kTLd;   // [vdim][token]
  float* pw = reinterpret_cast<float*>(vt + VB * kTLd);
  unsigned short* kr = reinterpret_cast<unsigned short*>(pw + kPowers + 3);   // [token][dim] k
  unsigned short* sh = kr + kC * KLd;     // [vdim][dim] the state, rounded ...
  unsigned short* sl = sh + VB * KLd;     // ... and the rest
  const int z = blockIdx.z, s = z / nseg, seg = z - s * nseg, h = blockIdx.x, vb0 = blockIdx.y * VB;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int c = lane & 15, g = lane >> 4;
  int r0 = seq_cu[s], n = seq_cu[s + 1] - r0;
  bool carried = seq_ctx[s] - n > 0;
  float* Sp = S + (((long)seq_state[s] * heads + h) * dim) * vdim;
  const float* S0 = Sp;
  bool last = true;
  if (nseg > 1) {
    const int at = seg * seg_len;
    last = at + seg_len >= n;
    if (SUM && last) return;
    n = min(seg_len, n - at);
    r0 += at;
    float* wp = ws + ((long)z * heads + h) * dim * vdim;
    if (SUM) { Sp = wp; carried = false; }
    else { S0 = wp; carried = true; }
  }
  if (n <= 0) return;
  const unsigned short* pq = proj + (long)r0 * ld + (long)h * dim;
  const unsigned short* pk = pq + (long)heads * dim;
  const unsigned short* pv = proj + (long)r0 * ld + 2L * heads * dim + (long)h * vdim + vb0;
  const bool owner = 16 * DT * wave < DP;   // KS == 1: two waves hold the state
  if (tid < kPowers) pw[tid] = powers[h * kPowers + tid];
  // state tiles: lane (c, g) holds rows 16 (DT wave + a) + 4 g + i of column vb0 + 16 b + c
  f32x4 st[DT][NT];
#pragma unroll
  for (int a = 0; a < DT; ++a)
#pragma unroll
    for (int b = 0; b < NT; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * (DT * wave + a) + 4 * g + i, v = vb0 + 16 * b + c;
        st[a][b][i] = (carried && d < dim && v < vdim) ? S0[(long)d * vdim + v] : 0.f;
      }
  // staging items: four neighbouring tokens x 8 channels, so the token-minor tiles take 8-byte stores
  constexpr int kKC = DP / 8, kVC = VB / 8;                         // 16-byte pieces per token row
  constexpr int kKI = 16 * kKC / 256 > 0 ? 16 * kKC / 256 : 1;
  static_assert(16 * kVC <= 256, "one value item per thread");
  u16x8 kf[kKI][4], vf[4], qf[KS];
  const u16x8 zero = {0, 0, 0, 0, 0, 0, 0, 0};
  const int vq = tid / kVC, vch = tid % kVC;
  auto fetch = [&](int t0) {
    const int m = n - t0;
#pragma unroll
    for (int i = 0; i < kKI; ++i) {
      const int kq = (tid + 256 * i) / kKC, ch = (tid + 256 * i) % kKC;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        kf[i][j] = (kq < 16 && 4 * kq + j < m && 8 * ch < dim)
                       ? *reinterpret_cast<const u16x8*>(pk + (long)(t0 + 4 * kq + j) * ld + 8 * ch)
                       : zero;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      vf[j] = (vq < 16 && 4 * vq + j < m && vb0 + 8 * vch < vdim)
                  ? *reinterpret_cast<const u16x8*>(pv + (long)(t0 + 4 * vq + j) * ld + 8 * vch)
                  : zero;
    if constexpr (!SUM) {
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
        qf[ks] = (16 * wave + c < m && 32 * ks + 8 * g < dim)
                     ? *reinterpret_cast<const u16x8*>(pq + (long)(t0 + 16 * wave + c) * ld + 32 * ks + 8 * g)
                     : zero;
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < n; t0 += kC) {
    const int m = min(kC, n - t0);
    __syncthreads();   // the previous chunk's reads are done (and pw is there, the first time)
    if (!SUM && owner) {
#pragma unroll
      for (int a = 0; a < DT; ++a)
#pragma unroll
        for (int b = 0; b < NT; ++b) {
          u16x4 hi, lo;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            hi[i] = f32_to_bf16(st[a][b][i]);
            lo[i] = f32_to_bf16(st[a][b][i] - bf16_to_f32(hi[i]));
          }
          const int at = (16 * b + c) * KLd + 16 * (DT * wave + a) + 4 * g;
          *reinterpret_cast<u16x4*>(sh + at) = hi;
          *reinterpret_cast<u16x4*>(sl + at) = lo;
        }
    }
#pragma unroll
    for (int i = 0; i < kKI; ++i) {
      const int kq = (tid + 256 * i) / kKC, ch = (tid + 256 * i) % kKC;
      if (kq < 16) {
        const int col = tok_col(4 * kq) ^ (((ch >> 1) & 7) << 3);
        float f[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          f[j] = pw[max(m - 1 - (4 * kq + j), 0)];   // rows past the end are zero
#pragma unroll
          for (int e = 0; e < 8; ++e) kf[i][j][e] = f32_to_bf16(silu_fast(bf16_to_f32(kf[i][j][e])));
          if (!SUM) *reinterpret_cast<u16x8*>(kr + (4 * kq + j) * KLd + 8 * ch) = kf[i][j];
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          u16x4 hi, lo;
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float x = f[j] * bf16_to_f32(kf[i][j][e]);
            hi[j] = f32_to_bf16(x);
            lo[j] = f32_to_bf16(x - bf16_to_f32(hi[j]));
          }
          *reinterpret_cast<u16x4*>(kth + (8 * ch + e) * kTLd + col) = hi;
          *reinterpret_cast<u16x4*>(ktl + (8 * ch + e) * kTLd + col) = lo;
        }
      }
    }
    if (vq < 16) {
      const int col = tok_col(4 * vq) ^ (((vch >> 1) & 7) << 3);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        u16x4 x;
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] = f32_to_bf16(silu_fast(bf16_to_f32(vf[j][e])));
        *reinterpret_cast<u16x4*>(vt + (8 * vch + e) * kTLd + col) = x;
      }
    }
    bf16x8 q[KS];
    if constexpr (!SUM) {
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        u16x8 x;
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = f32_to_bf16(silu_fast(bf16_to_f32(qf[ks][e])));
        q[ks] = __builtin_bit_cast(bf16x8, x);
      }
    }
    __syncthreads();
    if (t0 + kC < n) fetch(t0 + kC);   // the next chunk's loads fly during this chunk's math
    auto frag = [&](const unsigned short* p) { return __builtin_bit_cast(bf16x8, *reinterpret_cast<const u16x8*>(p)); };
    if constexpr (!SUM) {
    // what the state before the chunk gives: O^T tiles, lane (c, g) holds columns 16 b + 4 g + i of row 16 wave + c
    f32x4 acc[NT];
#pragma unroll
    for (int b = 0; b < NT; ++b) acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int qi = 16 * wave + c;
    if (carried || t0 > 0) {
#pragma unroll
      for (int ks = 0; ks < KS; ++ks)
#pragma unroll
        for (int b = 0; b < NT; ++b) {
          const int at = (16 * b + c) * KLd + 32 * ks + 8 * g;
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(sh + at), q[ks], acc[b], 0, 0, 0);
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(sl + at), q[ks], acc[b], 0, 0, 0);
        }
      const float f = pw[qi + 1];
#pragma unroll
      for (int b = 0; b < NT; ++b) acc[b] *= f;
    }
    // inside the chunk: lane (c, g) holds the weights of row qi against tokens 16 nt + 4 g + i
    f32x4 sc[4];
#pragma unroll
    for (int nt = 0; nt < 4; ++nt) {
      sc[nt] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (nt <= wave) {
#pragma unroll
        for (int ks = 0; ks < KS; ++ks)
          sc[nt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(frag(kr + (16 * nt + c) * KLd + 32 * ks + 8 * g), q[ks], sc[nt], 0, 0, 0);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int dist = qi - (16 * nt + 4 * g + i);
          sc[nt][i] = dist >= 0 ? sc[nt][i] * pw[dist] : 0.f;
        }
      }
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      if (2 * kk <= wave) {
        u16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float x = sc[2 * kk + (e >> 2)][e & 3];
          hi[e] = f32_to_bf16(x);
          lo[e] = f32_to_bf16(x - bf16_to_f32(hi[e]));
        }
        const bf16x8 ph = __builtin_bit_cast(bf16x8, hi), pl = __builtin_bit_cast(bf16x8, lo);
#pragma unroll
        for (int b = 0; b < NT; ++b) {
          const bf16x8 v = frag(vt + (16 * b + c) * kTLd + 8 * ((4 * kk + g) ^ (b & 7)));
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph, acc[b], 0, 0, 0);
          acc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl, acc[b], 0, 0, 0);
        }
      }
    }
    if (qi < m) {
      float* dst = o + ((long)(r0 + t0 + qi) * heads + h) * vdim + vb0;
#pragma unroll
      for (int b = 0; b < NT; ++b)
        if (vb0 + 16 * b + 4 * g < vdim) *reinterpret_cast<f32x4*>(dst + 16 * b + 4 * g) = acc[b];
    }
    }
    if (owner) {
      const float f = pw[m];
#pragma unroll
      for (int a = 0; a < DT; ++a) {
        const int dt = DT * wave + a;
#pragma unroll
        for (int b = 0; b < NT; ++b) st[a][b] *= f;
#pragma unroll
        for (int kk = 0; kk < 2; ++kk) {
          const int at = (16 * dt + c) * kTLd + 8 * ((4 * kk + g) ^ (dt & 7));
          const bf16x8 kh = frag(kth + at), kl = frag(ktl + at);
#pragma unroll
          for (int b = 0; b < NT; ++b) {
            const bf16x8 v = frag(vt + (16 * b + c) * kTLd + 8 * ((4 * kk + g) ^ (b & 7)));
            st[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, v, st[a][b], 0, 0, 0);
            st[a][b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl, v, st[a][b], 0, 0, 0);
          }
        }
      }
    }
  }
  if (!SUM && !last) return;
#pragma unroll
  for (int a = 0; a < DT; ++a)
#pragma unroll
    for (int b = 0; b < NT; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * (DT * wave + a) + 4 * g + i, v = vb0 + 16 * b + c;
        if (owner && d < dim && v < vdim) Sp[(long)d * vdim + v] = st[a][b][i];
      }
}

// ws[s, seg, head]: a segment's own sum on entry (all but the last segment's), the state before the segment on exit.
// grid (ceil(dim * vdim / 256), heads, sequences)
__global__ __launch_bounds__(256) void lightning_carry_kernel(float* __restrict__ ws, const float* __restrict__ S,
                                                             const float* __restrict__ powers,
                                                             const int* __restrict__ seq_cu,
                                                             const int* __restrict__ seq_ctx,
                                                             const int* __restrict__ seq_state, int heads, int dv,
                                                             int nseg, int seg_len) {
  const int s = blockIdx.z, h = blockIdx.y, e = blockIdx.x * 256 + threadIdx.x;
  if (e >= dv) return;
  const int n = seq_cu[s + 1] - seq_cu[s];
  float f = 1.f;   // decay^seg_len
  for (int i = 0; i < seg_len; i += 64) f *= powers[h * kPowers + 64];
  float cur = seq_ctx[s] - n > 0 ? S[((long)seq_state[s] * heads + h) * dv + e] : 0.f;
  float* p = ws + ((long)s * nseg * heads + h) * dv + e;
  const long step = (long)heads * dv;
  for (int at = 0; at < n; at += seg_len, p += step) {
    const float own = at + seg_len < n ? *p : 0.f;
    *p = cur;
    cur = __builtin_fmaf(f, cur, own);
  }
}

template <int KS, int NT, bool SUM>
void launch_chunk1(float* o, float* S, const unsigned short* proj, long ld, const float* powers, const int* seq_cu,
                   const int* seq_ctx, const int* seq_state, int nseq, int heads, int dim, int vdim, float* ws, int nseg,
                   int seg_len, hipStream_t s) {
  constexpr size_t smem = chunk_lds<KS, NT, SUM>();
  static_assert(smem <= 160 * 1024, "LDS");
  static const bool ok = hipFuncSetAttribute(reinterpret_cast<const void*>(&lightning_chunk_kernel<KS, NT, SUM>),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) == hipSuccess;
  (void)ok;
  lightning_chunk_kernel<KS, NT, SUM><<<dim3(heads, (vdim + 16 * NT - 1) / (16 * NT), nseq * nseg), 256, smem, s>>>(
      o, S, proj, ld, powers, seq_cu, seq_ctx, seq_state, heads, dim, vdim, ws, nseg, seg_len);
}

template <int KS>
void launch_chunk(float* o, float* S, const unsigned short* proj, long ld, const float* powers, const int* seq_cu,
                  const int* seq_ctx, const int* seq_state, int nseq, int heads, int dim, int vdim, float* ws, int nseg,
                  int seg_len, hipStream_t s) {
  // narrow column blocks (two workgroups per CU) while wide ones leave compute units idle
  const bool narrow = vdim <= 32 || (long)nseq * nseg * heads * ((vdim + 63) / 64) < 512;
  if (nseg > 1) {
    launch_chunk1<KS, 4, true>(o, S, proj, ld, powers, seq_cu, seq_ctx, seq_state, nseq, heads, dim, vdim, ws, nseg, seg_len, s);
    lightning_carry_kernel<<<dim3((dim * vdim + 255) / 256, heads, nseq), 256, 0, s>>>(
        ws, S, powers, seq_cu, seq_ctx, seq_state, heads, dim * vdim, nseg, seg_len);
  }
  if (narrow)
    launch_chunk1<KS, 2, false>(o, S, proj, ld, powers, seq_cu, seq_ctx, seq_state, nseq, heads, dim, vdim, ws, nseg, seg_len, s);
  else
    launch_chunk1<KS, 4, false>(o, S, proj, ld, powers, seq_cu, seq_ctx, seq_state, nseq, heads, dim, vdim, ws, nseg, seg_len, s);
}

// ---------------------------------------------------------------- one row per sequence
// grid (heads, column blocks, sequences from seq0 on), 256 threads: G = 256 / (kCW / CV) groups over the key channels,
// thread (g, x) holds CV neighbouring state columns; eight rows' loads in flight before their updates are stored.
constexpr int kCW = 128;   // state columns per workgroup

template <typename T, int CV>
__global__ __launch_bounds__(256) void lightning_step_kernel(float* __restrict__ o, float* __restrict__ S,
                                                            const T* __restrict__ proj, long ld,
                                                            const float* __restrict__ powers,
                                                            const int* __restrict__ seq_cu,
                                                            const int* __restrict__ seq_ctx,
                                                            const int* __restrict__ seq_state, int seq0, int heads,
                                                            int dim, int vdim) {
  extern __shared__ float sm[];   // q, k [dim] each
  constexpr int XT = kCW / CV, G = 256 / XT;
  __shared__ float part[G][kCW];
  float* sq = sm;
  float* sk = sm + dim;
  const int s = seq0 + blockIdx.z, h = blockIdx.x, tid = threadIdx.x;
  const long t = seq_cu[s];
  if (seq_cu[s + 1] - t <= 0) return;
  const int g = tid / XT, x = tid % XT;
  const int c0 = blockIdx.y * kCW + CV * x;
  const bool carried = seq_ctx[s] - 1 > 0;
  float* Sp = S + (((long)seq_state[s] * heads + h) * dim) * vdim;
  const T* row = proj + t * ld;
  for (int i = tid; i < dim; i += 256) {
    sq[i] = silu_f(ldf<T>(row, (long)h * dim + i));
    sk[i] = silu_f(ldf<T>(row, (long)(heads + h) * dim + i));
  }
  const float lam = powers[h * kPowers + 1];
  float v[CV], acc[CV];
#pragma unroll
  for (int j = 0; j < CV; ++j) {
    v[j] = c0 + j < vdim ? silu_f(ldf<T>(row, 2L * heads * dim + (long)h * vdim + c0 + j)) : 0.f;
    acc[j] = 0.f;
  }
  __syncthreads();
  if (c0 < vdim) {   // CV == 4: vdim % 4 == 0, the columns are inside together
    for (int i0 = g; i0 < dim; i0 += 8 * G) {
      float sv[8][CV];
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int i = i0 + u * G;
        if constexpr (CV == 4) {
          f32x4 z = {0.f, 0.f, 0.f, 0.f};
          if (carried && i < dim) z = *reinterpret_cast<const f32x4*>(Sp + (long)i * vdim + c0);
#pragma unroll
          for (int j = 0; j < 4; ++j) sv[u][j] = z[j];
        } else {
          sv[u][0] = (carried && i < dim) ? Sp[(long)i * vdim + c0] : 0.f;
        }
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) {
        const int i = i0 + u * G;
        if (i < dim) {
          const float k = sk[i], q = sq[i];
#pragma unroll
          for (int j = 0; j < CV; ++j) {
            sv[u][j] = __builtin_fmaf(lam, sv[u][j], k * v[j]);
            acc[j] = __builtin_fmaf(sv[u][j], q, acc[j]);
          }
          if constexpr (CV == 4)
            *reinterpret_cast<f32x4*>(Sp + (long)i * vdim + c0) = f32x4{sv[u][0], sv[u][1], sv[u][2], sv[u][3]};
          else
            Sp[(long)i * vdim + c0] = sv[u][0];
        }
      }
    }
  }
#pragma unroll
  for (int j = 0; j < CV; ++j) part[g][CV * x + j] = acc[j];
  __syncthreads();
  if (tid < kCW && blockIdx.y * kCW + tid < vdim) {
    float r = 0.f;
#pragma unroll
    for (int gg = 0; gg < G; ++gg) r += part[gg][tid];
    o[(t * heads + h) * vdim + blockIdx.y * kCW + tid] = r;
  }
}

// ---------------------------------------------------------------- norm over the concatenated heads, gate
template <typename T, int V>
__global__ __launch_bounds__(256) void lightning_out_kernel(T* __restrict__ out, long out_ld, const float* __restrict__ o,
                                                           const T* __restrict__ gate, long ld,
                                                           const float* __restrict__ w, int N, float eps,
                                                           float out_scale) {
  __shared__ float red[16];
  const long t = blockIdx.x;
  const float* src = o + t * N;
  float a = 0.f;
  for (int e = V * threadIdx.x; e < N; e += V * 256) {
    if constexpr (V == 4) {
      const f32x4 x = *reinterpret_cast<const f32x4*>(src + e);
      a += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
    } else {
      a += src[e] * src[e];
    }
  }
  a = block_sum(a, red);
  const float inv = out_scale / sqrtf(a / (float)N + eps);
  for (int e = V * threadIdx.x; e < N; e += V * 256) {
    if constexpr (V == 4) {   // bf16 rows at multiples of 4 elements
      const f32x4 x = *reinterpret_cast<const f32x4*>(src + e), wv = *reinterpret_cast<const f32x4*>(w + e);
      const u16x4 gv = *reinterpret_cast<const u16x4*>(gate + t * ld + e);
      u16x4 r;
#pragma unroll
      for (int i = 0; i < 4; ++i) r[i] = f32_to_bf16(x[i] * inv * wv[i] * sigmoid_f(bf16_to_f32(gv[i])));
      *reinterpret_cast<u16x4*>(out + t * out_ld + e) = r;
    } else {
      stf<T>(out, t * out_ld + e, src[e] * inv * w[e] * sigmoid_f(ldf<T>(gate, t * ld + e)));
    }
  }
}

template <typename T>
void run(void* out, long out_ld, float* S, const void* proj_, long ld, const float* powers, const float* norm_w,
         const int* seq_cu, const int* seq_ctx, const int* seq_state, int nseq, int npf, int T_rows, int pf_rows,
         float* scratch, int heads, int dim, int vdim, float eps, float out_scale, bool mfma, int nseg, int seg_len,
         hipStream_t s) {
  const T* proj = static_cast<const T*>(proj_);
  const int N = heads * vdim;
  float* o = scratch;                              // [T_rows, heads * vdim]
  if (npf > 0 && mfma) {
    if constexpr (sizeof(T) == 2) {
      auto p = reinterpret_cast<const unsigned short*>(proj);
      float* ws = o + (long)T_rows * N;              // nseg > 1: [npf, nseg, heads, dim, vdim]
#define HS_LC(KS) launch_chunk<KS>(o, S, p, ld, powers, seq_cu, seq_ctx, seq_state, npf, heads, dim, vdim, ws, nseg, seg_len, s)
      if (dim <= 32) HS_LC(1);
      else if (dim <= 64) HS_LC(2);
      else HS_LC(4);
#undef HS_LC
    }
  } else if (npf > 0) {
    float* vv = o + (long)T_rows * N;                // [pf_rows, heads, vdim]
    float* qk = vv + (long)pf_rows * N;              // [pf_rows, heads, 2 dim]
    lightning_stage_kernel<T><<<pf_rows, 256, 0, s>>>(qk, vv, proj, ld, heads, dim, vdim);
    dim3 grid(heads, (vdim + kCols - 1) / kCols, npf);
    const int ds = dim <= 16 ? 1 : dim <= 32 ? 2 : dim <= 64 ? 4 : dim <= 128 ? 8 : dim <= 256 ? 16 : 32;
    switch (ds) {
#define HS_LS(D)                                                                                                    \
  case D:                                                                                                           \
    lightning_scan_kernel<D><<<grid, kScanThreads, 0, s>>>(o, S, qk, vv, powers, seq_cu, seq_ctx, seq_state, heads,    \
                                                          dim, vdim);                                               \
    break;
      HS_LS(1) HS_LS(2) HS_LS(4) HS_LS(8) HS_LS(16) HS_LS(32)
#undef HS_LS
    }
  }
  if (nseq > npf) {
    dim3 grid(heads, (vdim + kCW - 1) / kCW, nseq - npf);
    const size_t smem = 2 * (size_t)dim * sizeof(float);
    if (vdim % 4 == 0)
      lightning_step_kernel<T, 4><<<grid, 256, smem, s>>>(o, S, proj, ld, powers, seq_cu, seq_ctx, seq_state, npf, heads,
                                                          dim, vdim);
    else
      lightning_step_kernel<T, 1><<<grid, 256, smem, s>>>(o, S, proj, ld, powers, seq_cu, seq_ctx, seq_state, npf, heads,
                                                          dim, vdim);
  }
  const T* gate = proj + 2L * heads * dim + N;
  bool v4 = false;
  if constexpr (sizeof(T) == 2)
    v4 = N % 4 == 0 && ld % 4 == 0 && out_ld % 4 == 0 && (uintptr_t)gate % 8 == 0 && (uintptr_t)out % 8 == 0;
  if constexpr (sizeof(T) == 2) {
    if (v4) {
      lightning_out_kernel<T, 4><<<T_rows, 256, 0, s>>>((T*)out, out_ld, o, gate, ld, norm_w, N, eps, out_scale);
      return;
    }
  }
  lightning_out_kernel<T, 1><<<T_rows, 256, 0, s>>>((T*)out, out_ld, o, gate, ld, norm_w, N, eps, out_scale);
}

}  // namespace

int lightning_max_dim() { return 512; }
int lightning_powers() { return kPowers; }

bool lightning_mfma_ok(int dim, int vdim, long ld, long offset) {
  return dim % 8 == 0 && vdim % 8 == 0 && dim <= 128 && ld % 8 == 0 && offset % 8 == 0;
}

void launch_lightning(void* out, long out_ld, float* S, const void* proj, long ld, const float* powers,
                      const float* norm_w, const int* seq_cu, const int* seq_ctx, const int* seq_state, int nseq,
                      int npf, int T, int pf_rows, float* scratch, int heads, int dim, int vdim, float eps,
                      float out_scale, bool mfma, int nseg, int seg_len, bool f32, hipStream_t s) {
  if (nseq <= 0 || T <= 0) return;
  if (f32)
    run<float>(out, out_ld, S, proj, ld, powers, norm_w, seq_cu, seq_ctx, seq_state, nseq, npf, T, pf_rows, scratch,
               heads, dim, vdim, eps, out_scale, false, 1, 0, s);
  else
    run<unsigned short>(out, out_ld, S, proj, ld, powers, norm_w, seq_cu, seq_ctx, seq_state, nseq, npf, T, pf_rows,
                        scratch, heads, dim, vdim, eps, out_scale, mfma, nseg, seg_len, s);
}

}  // namespace hipserve
