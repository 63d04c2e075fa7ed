// Device pieces shared by the recurrence kernels.
#pragma once

#include "rec.h"

namespace rlli {
namespace {

// the hardware exponential is good to a few ulp at these exponents; the
// 32-bit mode takes the exact one
template <typename T> DEV_INLINE float gexp(float x);
template <> DEV_INLINE float gexp<uint16_t>(float x) { return __expf(x); }
template <> DEV_INLINE float gexp<float>(float x) { return expf(x); }

template <typename T>
DEV_INLINE float log_sigmoid(float x) {
  // absolute error is what counts: it enters a sum of logarithms
  if constexpr (sizeof(T) == 2)
    return fminf(x, 0.f) - __logf(1.f + __expf(-fabsf(x)));
  return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
}

// 1 / x for x >= 1, good to an ulp where activations are 16-bit
template <typename T> DEV_INLINE float grcp(float x);
template <> DEV_INLINE float grcp<uint16_t>(float x) {
  return __builtin_amdgcn_rcpf(x);
}
template <> DEV_INLINE float grcp<float>(float x) { return 1.f / x; }

template <typename T>
DEV_INLINE float sigm(float x) {
  // (the exponent is bounded so that the reciprocal stays finite)
  return grcp<T>(1.f + gexp<T>(fminf(-x, 80.f)));
}

template <typename T>
DEV_INLINE float silu(float x) {
  return x * sigm<T>(x);
}

template <typename T>
DEV_INLINE float gtanh(float x) {
  if constexpr (sizeof(T) == 2) return 2.f * sigm<T>(2.f * x) - 1.f;
  return tanhf(x);
}

DEV_INLINE float softplus(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

DEV_INLINE float round_act(uint16_t, float v) {
  return bf16_to_f32(f32_to_bf16(v));
}
DEV_INLINE float round_act(float, float v) { return v; }

// running sum over the 16 lanes of a row
DEV_INLINE float row_prefix(float v) {
  v += dpp_mov_f32<0x111>(v);             // row_shr 1, 2, 4, 8: zeros enter
  v += dpp_mov_f32<0x112>(v);
  v += dpp_mov_f32<0x114>(v);
  v += dpp_mov_f32<0x118>(v);
  return v;
}

// running sum and maximum over a wave
DEV_INLINE float wave_prefix_sum(float v) {
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const float u = __shfl_up(v, off, kWave);
    if (lane >= off) v += u;
  }
  return v;
}
DEV_INLINE float wave_prefix_max(float v) {
  const int lane = threadIdx.x & 63;
#pragma unroll
  for (int off = 1; off < 64; off <<= 1) {
    const float u = __shfl_up(v, off, kWave);
    if (lane >= off) v = fmaxf(v, u);
  }
  return v;
}

DEV_INLINE f32x4_t mma4(float a, float b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

template <typename T>
DEV_INLINE f32x4_t load4_guard(const T* p, int d, int dim, bool row_ok,
                               bool vec) {
  f32x4_t v = f32x4_t{0.f, 0.f, 0.f, 0.f};
  if (!row_ok) return v;
  if (vec && d + 4 <= dim) return act_load4(p + d);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (d + j < dim) v[j] = act_load(p + d + j);
  return v;
}

// four columns as they lie in memory: a load's registers are not touched
// (and so not waited for) until the values are used
template <typename T> struct Raw4;
template <> struct Raw4<uint16_t> {
  uint2 r;
  DEV_INLINE void zero() { r = uint2{0, 0}; }
  DEV_INLINE void load(const uint16_t* p) {
    r = *reinterpret_cast<const uint2*>(p);
  }
  DEV_INLINE void put(int j, uint16_t v) {
    uint32_t& x = j < 2 ? r.x : r.y;
    x |= uint32_t(v) << (j % 2 * 16);
  }
  DEV_INLINE float get(int j) const {
    const uint32_t x = j < 2 ? r.x : r.y;
    return __uint_as_float(j % 2 ? x & 0xffff0000u : x << 16);
  }
};
template <> struct Raw4<float> {
  f32x4_t r;
  DEV_INLINE void zero() { r = f32x4_t{0.f, 0.f, 0.f, 0.f}; }
  DEV_INLINE void load(const float* p) {
    r = *reinterpret_cast<const f32x4_t*>(p);
  }
  DEV_INLINE void put(int j, float v) { r[j] = v; }
  DEV_INLINE float get(int j) const { return r[j]; }
};

template <typename T>
DEV_INLINE Raw4<T> raw_guard(const T* p, int d, int dim, bool row_ok,
                             bool vec) {
  Raw4<T> v;
  if (vec && row_ok && d + 4 <= dim) {
    v.load(p + d);
    return v;
  }
  v.zero();
  if (!row_ok) return v;
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (d + j < dim) v.put(j, p[d + j]);
  return v;
}

// Eight columns of a row as a matrix operand, zeros from ``dim`` on.  The
// row exists: callers take the last one for those behind it, so that no
// load is conditional.  VEC: dim is a multiple of 8 and rows are aligned.
template <bool VEC, typename T>
DEV_INLINE Frag8<T> frag_at(const T* p, int d, int dim) {
  Frag8<T> f;
  if constexpr (VEC) {
    f.load(p + min(d, dim - 8));
    if (d >= dim) f.zero();
  } else {
    f.zero();
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (d + j < dim) {
        if constexpr (sizeof(T) == 2) f.v[j] = short(p[d + j]);
        else if (j < 4) f.lo[j] = p[d + j];
        else f.hi[j - 4] = p[d + j];
      }
  }
  return f;
}

DEV_INLINE float frag_get(const Frag8<uint16_t>& f, int j) {
  return bf16_to_f32(uint16_t(f.v[j]));
}
DEV_INLINE float frag_get(const Frag8<float>& f, int j) {
  return j < 4 ? f.lo[j & 3] : f.hi[j & 3];
}
template <typename T>
DEV_INLINE float frag_sq(const Frag8<T>& f) {
  float s = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) s += frag_get(f, j) * frag_get(f, j);
  return s;
}

// a chunk's keys, columns down: kt [dpad][64], zeros from dim on
template <bool VEC, typename T>
DEV_INLINE void keys_down(const T* k, int64_t stride, int n, int dim,
                          int dpad, T* kt) {
  const int s = threadIdx.x & 63;
  const T* row = k + min(s, n - 1) * stride;
  for (int d = (threadIdx.x >> 6) * 8; d < dpad; d += 32) {
    const Frag8<T> f = frag_at<VEC>(row, d, dim);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      T e;
      if constexpr (sizeof(T) == 2) e = T(f.v[j]);
      else e = frag_get(f, j);
      kt[int64_t(d + j) * kRecChunk + s] = e;
    }
  }
}

}  // namespace
}  // namespace rlli
