#pragma once
#include "hipserve/common.h"

namespace hipserve {

template <typename T> HS_DEVICE float ldf(const T* p, long i);
template <> HS_DEVICE float ldf<unsigned short>(const unsigned short* p, long i) { return bf16_to_f32(p[i]); }
template <> HS_DEVICE float ldf<float>(const float* p, long i) { return p[i]; }
template <typename T> HS_DEVICE void stf(T* p, long i, float v);
template <> HS_DEVICE void stf<unsigned short>(unsigned short* p, long i, float v) { p[i] = f32_to_bf16(v); }
template <> HS_DEVICE void stf<float>(float* p, long i, float v) { p[i] = v; }

// V consecutive elements of a row as fp32 (V > 1: the address is aligned to V elements)
template <typename T, int V> struct Row;
template <> struct Row<float, 1> {
  static HS_DEVICE void ld(const float* p, float (&v)[1]) { v[0] = *p; }
  static HS_DEVICE void st(float* p, const float (&v)[1]) { *p = v[0]; }
};
template <> struct Row<float, 2> {
  static HS_DEVICE void ld(const float* p, float (&v)[2]) { const float2 a = *reinterpret_cast<const float2*>(p); v[0] = a.x; v[1] = a.y; }
  static HS_DEVICE void st(float* p, const float (&v)[2]) { *reinterpret_cast<float2*>(p) = float2{v[0], v[1]}; }
};
template <> struct Row<float, 4> {
  static HS_DEVICE void ld(const float* p, float (&v)[4]) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = a[i];
  }
  static HS_DEVICE void st(float* p, const float (&v)[4]) { *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]}; }
};
template <> struct Row<unsigned short, 1> {
  static HS_DEVICE void ld(const unsigned short* p, float (&v)[1]) { v[0] = bf16_to_f32(*p); }
  static HS_DEVICE void st(unsigned short* p, const float (&v)[1]) { *p = f32_to_bf16(v[0]); }
};
template <> struct Row<unsigned short, 4> {
  static HS_DEVICE void ld(const unsigned short* p, float (&v)[4]) {
    const u16x4 a = *reinterpret_cast<const u16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = bf16_to_f32(a[i]);
  }
  static HS_DEVICE void st(unsigned short* p, const float (&v)[4]) {
    u16x4 a;
#pragma unroll
    for (int i = 0; i < 4; ++i) a[i] = f32_to_bf16(v[i]);
    *reinterpret_cast<u16x4*>(p) = a;
  }
};
template <> struct Row<float, 8> {
  static HS_DEVICE void ld(const float* p, float (&v)[8]) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) { v[i] = a[i]; v[4 + i] = b[i]; }
  }
  static HS_DEVICE void st(float* p, const float (&v)[8]) {
    *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
  }
};
template <> struct Row<unsigned short, 8> {
  static HS_DEVICE void ld(const unsigned short* p, float (&v)[8]) {
    const u16x8 a = *reinterpret_cast<const u16x8*>(p);
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = bf16_to_f32(a[i]);
  }
  static HS_DEVICE void st(unsigned short* p, const float (&v)[8]) {
    u16x8 a;
#pragma unroll
    for (int i = 0; i < 8; ++i) a[i] = f32_to_bf16(v[i]);
    *reinterpret_cast<u16x8*>(p) = a;
  }
};

HS_DEVICE float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }

// Sum over the 16 lanes of a DPP row; every lane of the row gets it.
HS_DEVICE float row_sum(float v) {
  v = dpp_step<0xB1, 0xf, false>(v);   // quad_perm [1, 0, 3, 2]
  v = dpp_step<0x4E, 0xf, false>(v);   // quad_perm [2, 3, 0, 1]
  v = dpp_step<0x141, 0xf, false>(v);  // row_half_mirror
  return dpp_step<0x140, 0xf, false>(v);  // row_mirror
}

// First key (behind the kept ones) that position pos sees: its window's, its chunk's, or the sequence's first.
HS_DEVICE int first_key(int pos, int window, int chunk) {
  return chunk > 0 ? pos - pos % chunk : window > 0 ? max(0, pos - window + 1) : 0;
}

// g sigmoid(1.702 g) (u + 1) of g = min(gate, limit), u = clamp(up, -limit, limit)
HS_DEVICE float clamped_glu_f(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(1.702f * g) * (u + 1.f);
}

}  // namespace hipserve
