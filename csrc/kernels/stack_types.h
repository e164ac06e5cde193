// Element types of the layer-stack kernels: T = bf16 (u16) or 32-bit float.
#pragma once
#include "common.h"

namespace {
using namespace vwa;

template <class T> VWA_DEVICE float ldv(const T* p);
template <> VWA_DEVICE float ldv<u16>(const u16* p) { return bf2f(*p); }
template <> VWA_DEVICE float ldv<float>(const float* p) { return *p; }
VWA_DEVICE void stv(u16* p, float v) { *p = f2bf(v); }
VWA_DEVICE void stv(float* p, float v) { *p = v; }

// four consecutive values
VWA_DEVICE void st4(u16* p, const float (&v)[4]) {
  uint2 o;
  o.x = pack2(v[0], v[1]);
  o.y = pack2(v[2], v[3]);
  *reinterpret_cast<uint2*>(p) = o;
}
VWA_DEVICE void st4(float* p, const float (&v)[4]) { *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]); }
VWA_DEVICE void ld4(const u16* p, float (&v)[4]) {
  const uint2 u = *reinterpret_cast<const uint2*>(p);
  v[0] = __uint_as_float(u.x << 16);
  v[1] = __uint_as_float(u.x & 0xffff0000u);
  v[2] = __uint_as_float(u.y << 16);
  v[3] = __uint_as_float(u.y & 0xffff0000u);
}
VWA_DEVICE void ld4(const float* p, float (&v)[4]) {
  const float4 u = *reinterpret_cast<const float4*>(p);
  v[0] = u.x;
  v[1] = u.y;
  v[2] = u.z;
  v[3] = u.w;
}

// eight consecutive values (16- / 32-byte accesses)
VWA_DEVICE void ld8(const u16* p, float (&v)[8]) { unpack8(*reinterpret_cast<const uint4*>(p), v); }
VWA_DEVICE void ld8(const float* p, float (&v)[8]) {
  const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
  v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w;
  v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
VWA_DEVICE void st8(u16* p, const float (&v)[8]) { *reinterpret_cast<uint4*>(p) = pack8(v); }
VWA_DEVICE void st8(float* p, const float (&v)[8]) {
  reinterpret_cast<float4*>(p)[0] = make_float4(v[0], v[1], v[2], v[3]);
  reinterpret_cast<float4*>(p)[1] = make_float4(v[4], v[5], v[6], v[7]);
}

VWA_DEVICE float sigm(float x) { return 1.f / (1.f + __expf(-x)); }

// 16-byte MFMA fragments: lane (row or column l & 15, group l >> 4) holds EPL consecutive k of a
// KS-deep step.  D[row 4 (l >> 4) + i][column l & 15].
template <class T> struct MM;
template <> struct MM<u16> {
  static constexpr int KS = 32, EPL = 8;
  static VWA_DEVICE f32x4 mma(const uint4& a, const uint4& b, const f32x4& c) { return mfma16(as_bf16x8(a), as_bf16x8(b), c); }
};
template <> struct MM<float> {             // element j of every lane group per MFMA
  static constexpr int KS = 16, EPL = 4;
  static VWA_DEVICE f32x4 mma(const uint4& a, const uint4& b, f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.x), __uint_as_float(b.x), c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.y), __uint_as_float(b.y), c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.z), __uint_as_float(b.z), c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(a.w), __uint_as_float(b.w), c, 0, 0, 0);
  }
};

}  // namespace
