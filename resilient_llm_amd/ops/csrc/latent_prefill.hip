// Prompt attention over expanded keys and values (bf16 matrix cores, f32
// softmax): every head has its own keys and values, which two matrix
// products made from a sequence's gathered latents, the values already
// transposed.  Keys of a sequence start at a multiple of 64 in them and
// are padded with zeros to a multiple of 64.
//
// A workgroup owns 128 prompt rows of one head, a wave 32 of them, and
// walks 64-key tiles through double-buffered LDS, the next tile's loads in
// flight under the products.  Scores are computed transposed (keys down,
// queries across), so a lane holds 32 scores of ONE query: the softmax
// needs a single cross-lane step, and the weights are already the second
// product's operand, in registers, with the keys in the order
// 0-3, 8-11 | 4-7, 12-15 per 16; the value tile is laid down in that order.

#include "lat.h"

namespace rlli {
namespace {

typedef float f32x16_t __attribute__((ext_vector_type(16)));
typedef float f32x2_t __attribute__((ext_vector_type(2)));
typedef __bf16 b16x2_t __attribute__((ext_vector_type(2)));

constexpr float kNegInf = -1e30f;
constexpr int KT = 64;
constexpr int VROW = KT + 8;

DEV_INLINE uint32_t pack2(float a, float b) {
  const b16x2_t v = __builtin_convertvector((f32x2_t{a, b}), b16x2_t);
  return __builtin_bit_cast(uint32_t, v);
}

DEV_INLINE f32x16_t mma32(s16x8_t a, s16x8_t b, f32x16_t c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

// P: the larger of the key and value widths, rounded up
template <int P>
__global__ __launch_bounds__(256, P <= 128 ? 2 : 1)
void expanded_attn_kernel(ExpandedAttnArgs a) {
  constexpr int DC = P / 16;              // contraction steps of a score
  constexpr int VT = P / 32;              // value tiles
  constexpr int KROW = P + 8;
  constexpr int BUF = KT * KROW + P * VROW;
  constexpr int NK = KT * (P / 8) / 256;  // vectors a thread stages
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];

  // heads that share an XCD's L2 walk their tiles together, longest first
  int h, tile;
  {
    const int b = blockIdx.x;
    int i = b;
    if (a.heads % 8 == 0) {
      i = b / 8;
      h = (i / a.n_tiles) * 8 + b % 8;
    } else {
      h = i / a.n_tiles;
    }
    tile = a.n_tiles - 1 - i % a.n_tiles;
  }
  const int row0 = a.tiles[tile], pos0 = a.tiles[a.n_tiles + tile];
  const int nrows = a.tiles[2 * a.n_tiles + tile];
  const int seq = a.tiles[3 * a.n_tiles + tile];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int qi = lane & 31, hi = lane >> 5;
  const int sub = w * 32;
  const int64_t base = a.kv_off[seq];
  const int len = pos0 + nrows;
  const int my_row = sub + qi;
  const int qpos = pos0 + min(my_row, nrows - 1);
  const bool active = sub < nrows;
  const int w_last = pos0 + min(sub + 31, nrows - 1);    // of this wave

  const int64_t qw = int64_t(a.heads) * a.dim;
  const int64_t vw = int64_t(a.heads) * a.vdim;
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) +
                      (row0 + min(my_row, nrows - 1)) * qw + h * a.dim;
  s16x8_t qf[DC];
#pragma unroll
  for (int c = 0; c < DC; ++c) {
    uint4 raw = {0, 0, 0, 0};
    const int d = c * 16 + hi * 8;
    if (d < a.dim) raw = *reinterpret_cast<const uint4*>(q + d);
    qf[c] = __builtin_bit_cast(s16x8_t, raw);
  }

  const uint16_t* kp = reinterpret_cast<const uint16_t*>(a.k) + base * qw +
                       h * a.dim;
  const uint16_t* vp = reinterpret_cast<const uint16_t*>(a.vt) +
                       int64_t(h) * a.vdim * a.tokens + base;
  uint4 kr[NK], vr[NK];
  auto fetch = [&](int kv0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = i * 256 + threadIdx.x;
      const int r = e / (P / 8), d = e % (P / 8) * 8;
      kr[i] = uint4{0, 0, 0, 0};
      if (d < a.dim)
        kr[i] = *reinterpret_cast<const uint4*>(kp + (kv0 + r) * qw + d);
      const int vd = e / 8, c = e % 8 * 8;
      vr[i] = uint4{0, 0, 0, 0};
      if (vd < a.vdim)
        vr[i] = *reinterpret_cast<const uint4*>(
            vp + int64_t(vd) * a.tokens + kv0 + c);
    }
  };
  auto stage = [&](uint16_t* buf) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = i * 256 + threadIdx.x;
      *reinterpret_cast<uint4*>(buf + e / (P / 8) * KROW + e % (P / 8) * 8) =
          kr[i];
      // keys 0-3 | 4-7 of an octet go eight apart, odd octets four up
      uint16_t* v = buf + KT * KROW + e / 8 * VROW + e % 8 / 2 * 16 +
                    e % 2 * 4;
      *reinterpret_cast<uint2*>(v) = uint2{vr[i].x, vr[i].y};
      *reinterpret_cast<uint2*>(v + 8) = uint2{vr[i].z, vr[i].w};
    }
  };

  f32x16_t o[VT];
#pragma unroll
  for (int v = 0; v < VT; ++v)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[v][r] = 0.f;
  float m = kNegInf, l = 0.f;
  const float c2 = a.scale * 1.4426950408889634f;

  fetch(0);
  stage(lds);
  __syncthreads();
  int cur = 0;
  for (int kv0 = 0; kv0 < len; kv0 += KT) {
    const bool more = kv0 + KT < len;
    if (more) fetch(kv0 + KT);
    const uint16_t* ks = lds + cur * BUF;
    const uint16_t* vs = ks + KT * KROW;
    if (active && kv0 <= w_last) {
      f32x16_t s[2];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
        for (int r = 0; r < 16; ++r) s[kt][r] = 0.f;
#pragma unroll
        for (int c = 0; c < DC; ++c) {
          if (c * 16 >= a.dim) break;
          const s16x8_t kf = *reinterpret_cast<const s16x8_t*>(
              ks + (kt * 32 + qi) * KROW + c * 16 + hi * 8);
          s[kt] = mma32(kf, qf[c], s[kt]);
        }
      }
      float mx = kNegInf;
      if (kv0 + KT - 1 > pos0 + sub) {      // some query sees only a part
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = kv0 + kt * 32 + (r >> 2) * 8 + hi * 4 + (r & 3);
            s[kt][r] = key <= qpos ? s[kt][r] * c2 : kNegInf;
            mx = fmaxf(mx, s[kt][r]);
          }
      } else {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            s[kt][r] *= c2;
            mx = fmaxf(mx, s[kt][r]);
          }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
      const float mn = fmaxf(m, mx);
      if (!__all(mn == m)) {
        const float corr = __builtin_amdgcn_exp2f(m - mn);
        l *= corr;
#pragma unroll
        for (int v = 0; v < VT; ++v)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[v][r] *= corr;
        m = mn;
      }
      float sum = 0.f;
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          s[kt][r] = __builtin_amdgcn_exp2f(s[kt][r] - m);
          sum += s[kt][r];
        }
      l += sum;                             // this half's keys
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int t = 0; t < 2; ++t) {
          const uint4 raw = {pack2(s[kt][t * 8], s[kt][t * 8 + 1]),
                             pack2(s[kt][t * 8 + 2], s[kt][t * 8 + 3]),
                             pack2(s[kt][t * 8 + 4], s[kt][t * 8 + 5]),
                             pack2(s[kt][t * 8 + 6], s[kt][t * 8 + 7])};
          const s16x8_t pf = __builtin_bit_cast(s16x8_t, raw);
#pragma unroll
          for (int v = 0; v < VT; ++v) {
            if (v * 32 >= a.vdim) break;
            const s16x8_t vf = *reinterpret_cast<const s16x8_t*>(
                vs + (v * 32 + qi) * VROW + kt * 32 + t * 16 + hi * 8);
            o[v] = mma32(vf, pf, o[v]);
          }
        }
    }
    if (more) {
      cur ^= 1;
      stage(lds + cur * BUF);
    }
    __syncthreads();
  }

  if (my_row >= nrows) return;
  l += __shfl_xor(l, 32, kWave);
  const float inv = 1.f / l;
  const uint16_t* gate =
      a.gate ? reinterpret_cast<const uint16_t*>(a.gate) +
                   (row0 + my_row) * a.gate_stride + h * a.vdim
             : nullptr;
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out) +
                  (row0 + my_row) * a.out_stride + h * a.vdim;
#pragma unroll
  for (int v = 0; v < VT; ++v)
#pragma unroll
    for (int r = 0; r < 16; r += 4) {
      const int d = v * 32 + (r >> 2) * 8 + hi * 4;
      if (d >= a.vdim) continue;
      float t[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) t[j] = o[v][r + j] * inv;
      if (gate) {
        const f32x4_t z = act_load4(gate + d);
#pragma unroll
        for (int j = 0; j < 4; ++j) t[j] *= 1.f / (1.f + __expf(-z[j]));
      }
      *reinterpret_cast<uint2*>(out + d) =
          uint2{pack2(t[0], t[1]), pack2(t[2], t[3])};
    }
}

template <int P>
void go(const ExpandedAttnArgs& a, hipStream_t st) {
  constexpr size_t smem = size_t(KT * (P + 8) + P * VROW) * 2 * 2;
  auto* k = expanded_attn_kernel<P>;
  if (smem > 65536)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              int(smem));
  hipLaunchKernelGGL(k, dim3(a.n_tiles * a.heads), dim3(256), smem, st, a);
}

}  // namespace

bool expanded_ok(int dim, int vdim) {
  return dim % 8 == 0 && vdim % 8 == 0 && dim <= 256 && vdim <= 256;
}

void launch_expanded_attn(const ExpandedAttnArgs& a, hipStream_t st) {
  if (a.n_tiles == 0) return;
  const int d = a.dim > a.vdim ? a.dim : a.vdim;
  if (d <= 32) go<32>(a, st);
  else if (d <= 64) go<64>(a, st);
  else if (d <= 96) go<96>(a, st);
  else if (d <= 128) go<128>(a, st);
  else if (d <= 192) go<192>(a, st);
  else go<256>(a, st);
}

}  // namespace rlli
