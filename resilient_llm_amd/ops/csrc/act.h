// What the kernels of models with mixed layers share: activation and cache
// element access, matrix fragments.
//
// Every kernel takes its activation type as a template parameter:
// uint16_t (bf16 bits, the serving precision) or float (true 32-bit).
#pragma once

#include "common.h"

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef short s16x8_t __attribute__((ext_vector_type(8)));

DEV_INLINE float act_load(const uint16_t* p) { return bf16_to_f32(*p); }
DEV_INLINE float act_load(const float* p) { return *p; }
DEV_INLINE void act_store(uint16_t* p, float v) { *p = f32_to_bf16(v); }
DEV_INLINE void act_store(float* p, float v) { *p = v; }

// four neighbours at once; the caller guarantees 4-element alignment
DEV_INLINE f32x4_t act_load4(const uint16_t* p) {
  const uint2 r = *reinterpret_cast<const uint2*>(p);
  return f32x4_t{__uint_as_float(r.x << 16),
                 __uint_as_float(r.x & 0xffff0000u),
                 __uint_as_float(r.y << 16),
                 __uint_as_float(r.y & 0xffff0000u)};
}
DEV_INLINE f32x4_t act_load4(const float* p) {
  return *reinterpret_cast<const f32x4_t*>(p);
}
DEV_INLINE void act_store4(uint16_t* p, f32x4_t v) {
  uint2 r;
  r.x = uint32_t(f32_to_bf16(v[0])) | (uint32_t(f32_to_bf16(v[1])) << 16);
  r.y = uint32_t(f32_to_bf16(v[2])) | (uint32_t(f32_to_bf16(v[3])) << 16);
  *reinterpret_cast<uint2*>(p) = r;
}
DEV_INLINE void act_store4(float* p, f32x4_t v) {
  *reinterpret_cast<f32x4_t*>(p) = v;
}

// Cache codec of the 32-bit mode, same interface as CacheBF16/CacheFP8.
struct CacheF32 {
  using elem = float;
  struct vec8 { float f[8]; };
  static DEV_INLINE void to_f32(const vec8& raw, float* out8) {
#pragma unroll
    for (int i = 0; i < 8; ++i) out8[i] = raw.f[i];
  }
};

DEV_INLINE float cache_load(const uint16_t* p) { return bf16_to_f32(*p); }
DEV_INLINE float cache_load(const float* p) { return *p; }
DEV_INLINE float cache_load(const uint8_t* p) {
  return __builtin_amdgcn_cvt_f32_fp8(int(*p), 0);
}
DEV_INLINE void cache_store(uint16_t* p, float v) { *p = f32_to_bf16(v); }
DEV_INLINE void cache_store(float* p, float v) { *p = v; }
DEV_INLINE void cache_store(uint8_t* p, float v) {
  *p = uint8_t(__builtin_amdgcn_cvt_pk_fp8_f32(v, v, 0, false) & 0xff);
}

// Eight consecutive k-values of one matrix row per lane, and the MFMA
// that contracts them: lane l holds row l & 15 and k = (l >> 4) * 8 + j.
// The 32-bit form walks the same eight values with eight 16x16x4 steps,
// pairing slot l >> 4 of step j with k = (l >> 4) * 8 + j on both sides.
template <typename T> struct Frag8;
template <> struct Frag8<uint16_t> {
  s16x8_t v;
  DEV_INLINE void zero() { v = s16x8_t{0, 0, 0, 0, 0, 0, 0, 0}; }
  DEV_INLINE void load(const uint16_t* p) {
    v = *reinterpret_cast<const s16x8_t*>(p);
  }
  static DEV_INLINE f32x4_t mma(const Frag8& a, const Frag8& b, f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
  }
};
template <> struct Frag8<float> {
  f32x4_t lo, hi;
  DEV_INLINE void zero() {
    lo = f32x4_t{0.f, 0.f, 0.f, 0.f};
    hi = lo;
  }
  DEV_INLINE void load(const float* p) {
    lo = *reinterpret_cast<const f32x4_t*>(p);
    hi = *reinterpret_cast<const f32x4_t*>(p + 4);
  }
  static DEV_INLINE f32x4_t mma(const Frag8& a, const Frag8& b, f32x4_t c) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.lo[j], b.lo[j], c, 0, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.hi[j], b.hi[j], c, 0, 0, 0);
    return c;
  }
};

namespace rlli {

// element type of a paged cache
enum CacheKind { kCacheBF16 = 0, kCacheFP8 = 1, kCacheF32 = 2 };

}  // namespace rlli
