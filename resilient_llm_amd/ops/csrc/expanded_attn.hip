// Prompt attention over a sequence's keys and values in one piece (bf16
// matrix cores, f32 softmax), values transposed: expanded from gathered
// latents by two matrix products (a key/value head per query head), or
// gathered from their pages (kv_gather).  Keys of a sequence start at a
// multiple of 64 in them and are padded with zeros to a multiple of 64.
// Optional: a distance bias per head, a query temperature by position.
// Differential attention (two maps per head, see attn.h) also has capped
// scores and chunks; its first waves take map 1 of a row, as many others map
// 2 over the same tiles, and the difference is made through LDS.
//
// A workgroup owns 128 prompt rows of one head, a wave 32 of them, and
// walks 64-key tiles through double-buffered LDS, the next tile's loads in
// flight under the products.  Scores are computed transposed (keys down,
// queries across), so a lane holds 32 scores of ONE query: the softmax
// needs a single cross-lane step, and the weights are already the second
// product's operand, in registers, with the keys in the order
// 0-3, 8-11 | 4-7, 12-15 per 16; the value tile is laid down in that order.

#include "attn.h"

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

// P: the larger of the key (all maps) and value widths, rounded up; BIAS: a
// score loses r1 ln(1 + r2 distance)
template <int P, bool BIAS, int MAPS>
__global__ __launch_bounds__(256 * MAPS, P <= 128 || MAPS == 2 ? 2 : 1)
void expanded_attn_kernel(ExpandedAttnArgs a) {
  constexpr int NT = 256 * MAPS;          // threads
  constexpr int DC = P / MAPS / 16;       // contraction steps of a score
  constexpr int VT = P / 32;              // value tiles
  constexpr int KROW = P + 8;
  constexpr int BUF = KT * KROW + P * VROW;
  constexpr int NK = KT * (P / 8) / NT;   // vectors a thread stages
  static_assert(NK * NT == KT * (P / 8), "a tile is staged whole");
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
  const int map = w >> 2, sub = (w & 3) * 32;
  const int64_t base = a.kv_off[seq];
  const int len = pos0 + nrows;
  const int my_row = sub + qi;
  const int qpos = pos0 + min(my_row, nrows - 1);
  const bool active = sub < nrows;
  const int w_last = pos0 + min(sub + 31, nrows - 1);    // of this wave
  // first visible position: of this lane's query, this wave's first query
  // and its last
  int lo = 0, w_lo = 0, w_top = 0, first = 0;
  if constexpr (MAPS == 2)
    if (a.chunk > 0) {
      lo = qpos / a.chunk * a.chunk;
      w_lo = min(pos0 + sub, w_last) / a.chunk * a.chunk;
      w_top = w_last / a.chunk * a.chunk;
      first = pos0 / a.chunk * a.chunk / KT * KT;
    }

  const int64_t kw = int64_t(a.n_kv) * MAPS * a.dim;
  const int kd = MAPS * a.dim;            // a head's
  const int kvh = h / (a.heads / a.n_kv);
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q) +
                      (row0 + min(my_row, nrows - 1)) * a.q_stride +
                      (h * MAPS + map) * a.dim;
  s16x8_t qf[DC];
#pragma unroll
  for (int c = 0; c < DC; ++c) {
    uint4 raw = {0, 0, 0, 0};
    const int d = c * 16 + hi * 8;
    if (d < a.dim) raw = *reinterpret_cast<const uint4*>(q + d);
    qf[c] = __builtin_bit_cast(s16x8_t, raw);
  }

  const uint16_t* kp = reinterpret_cast<const uint16_t*>(a.k) + base * kw +
                       kvh * kd;
  const uint16_t* vp = reinterpret_cast<const uint16_t*>(a.vt) +
                       int64_t(kvh) * a.vdim * a.tokens + base;
  uint4 kr[NK], vr[NK];
  auto fetch = [&](int kv0) {
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int e = i * NT + threadIdx.x;
      const int r = e / (P / 8), d = e % (P / 8) * 8;
      kr[i] = uint4{0, 0, 0, 0};
      if (d < kd)
        kr[i] = *reinterpret_cast<const uint4*>(kp + (kv0 + r) * kw + d);
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
      const int e = i * NT + threadIdx.x;
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
  const float c2 = a.scale * query_temp(qpos, a.temp_coef, a.temp_every) *
                   1.4426950408889634f;
  float r1 = 0.f, r2 = 0.f;
  if constexpr (BIAS) {
    r1 = a.r1[h];
    r2 = a.r2[h];
  }

  const float cap2 = MAPS == 2 && a.cap > 0.f ? kTwoLog2e / a.cap : 0.f;
  fetch(first);
  stage(lds);
  __syncthreads();
  int cur = 0;
  for (int kv0 = first; kv0 < len; kv0 += KT) {
    const bool more = kv0 + KT < len;
    if (more) fetch(kv0 + KT);
    const uint16_t* ks = lds + cur * BUF;
    const uint16_t* vs = ks + KT * KROW;
    if (active && kv0 <= w_last && kv0 + KT > w_lo) {
      f32x16_t s[2];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
        for (int r = 0; r < 16; ++r) s[kt][r] = 0.f;
#pragma unroll
        for (int c = 0; c < DC; ++c) {
          if (c * 16 >= a.dim) break;
          const s16x8_t kf = *reinterpret_cast<const s16x8_t*>(
              ks + (kt * 32 + qi) * KROW + map * a.dim + c * 16 + hi * 8);
          s[kt] = mma32(kf, qf[c], s[kt]);
        }
      }
      if constexpr (BIAS) {
        // r1 ln(x) log2(e) = r1 log2(x)
        const float at = float(qpos - kv0 - hi * 4);
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const float dist = at - float(kt * 32 + (r >> 2) * 8 + (r & 3));
            s[kt][r] = fmaf(-r1, __builtin_amdgcn_logf(fmaf(r2, fmaxf(dist, 0.f), 1.f)),
                            s[kt][r] * c2);
          }
      }
      float c1 = BIAS ? 1.f : c2;
      if constexpr (MAPS == 2)
        if (cap2 > 0.f) {
          const float in = a.scale * cap2, top = a.cap * 1.4426950408889634f;
          c1 = 1.f;
#pragma unroll
          for (int kt = 0; kt < 2; ++kt)
#pragma unroll
            for (int r = 0; r < 16; ++r)
              s[kt][r] = fmaf(
                  -2.f * top,
                  __builtin_amdgcn_rcpf(
                      1.f + __builtin_amdgcn_exp2f(s[kt][r] * in)),
                  top);
        }
      float mx = kNegInf;
      // some query sees only a part
      if (kv0 + KT - 1 > pos0 + sub || kv0 < w_top) {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int key = kv0 + kt * 32 + (r >> 2) * 8 + hi * 4 + (r & 3);
            s[kt][r] = key <= qpos && key >= lo ? s[kt][r] * c1 : kNegInf;
            mx = fmaxf(mx, s[kt][r]);
          }
      } else {
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            s[kt][r] *= c1;
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

  if constexpr (MAPS == 2) {
    l += __shfl_xor(l, 32, kWave);
    const float inv = 1.f / l;
    // map 2's output through LDS, [value column][32 rows] per pair of waves;
    // the tiles are done with (a barrier ends the loop)
    float* side = reinterpret_cast<float*>(lds) + (w & 3) * (P * 32) + qi;
    if (map == 1) {
#pragma unroll
      for (int v = 0; v < VT; ++v)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          side[(v * 32 + (r >> 2) * 8 + hi * 4 + (r & 3)) * 32] =
              o[v][r] * inv;
    }
    __syncthreads();
    if (map == 1 || my_row >= nrows) return;
    float ss = 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        const int d = v * 32 + (r >> 2) * 8 + hi * 4 + (r & 3);
        o[v][r] = o[v][r] * inv - a.lambda * side[d * 32];
        if (d < a.vdim) ss += o[v][r] * o[v][r];
      }
    ss += __shfl_xor(ss, 32, kWave);      // both halves have the same row
    float post = a.out_scale / sqrtf(ss / a.vdim + a.eps);
    if (a.gate)
      post /= 1.f + __expf(-bf16_to_f32(
                        reinterpret_cast<const uint16_t*>(
                            a.gate)[(row0 + my_row) * a.gate_stride + h]));
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out) +
                    (row0 + my_row) * a.out_stride + h * a.vdim;
#pragma unroll
    for (int v = 0; v < VT; ++v)
#pragma unroll
      for (int r = 0; r < 16; r += 4) {
        const int d = v * 32 + (r >> 2) * 8 + hi * 4;
        if (d < a.vdim)
          *reinterpret_cast<uint2*>(out + d) =
              uint2{pack2(o[v][r] * post, o[v][r + 1] * post),
                    pack2(o[v][r + 2] * post, o[v][r + 3] * post)};
      }
    return;
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

// one workgroup per (64 tokens, kv head)
template <typename KC>
__global__ __launch_bounds__(256)
void kv_gather_kernel(KvGatherArgs a) {
  using vec8 = typename KC::vec8;
  using elem = typename KC::elem;
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];   // [vdim][72]
  const int b = blockIdx.x, kvh = blockIdx.y;
  const int seq = a.blocks[b], tok0 = a.blocks[a.n + b];
  const int n = a.blocks[2 * a.n + b];
  const int64_t row0 = a.blocks[3 * a.n + b];
  const int32_t* bt = a.block_tables + int64_t(seq) * a.max_blocks;
  auto cache_row = [&](int r) {
    const int t = tok0 + r;
    return (int64_t(bt[t / a.block_size]) * a.n_kv + kvh) * a.block_size +
           t % a.block_size;
  };
  auto bf16 = [](vec8 raw) {
    float f[8];
    KC::to_f32(raw, f);
    bf16x8 o;
#pragma unroll
    for (int j = 0; j < 8; ++j) o.s[j] = f32_to_bf16(f[j]);
    return o;
  };
  const int k8 = a.dim / 8, v8 = a.vdim / 8;
  const elem* kc = reinterpret_cast<const elem*>(a.k_cache);
  const elem* vc = reinterpret_cast<const elem*>(a.v_cache);
  uint16_t* k = reinterpret_cast<uint16_t*>(a.k) + row0 * a.n_kv * a.dim +
                kvh * a.dim;
  for (int e = threadIdx.x; e < kKvGatherRows * v8; e += 256) {
    const int r = e / v8, d = e % v8 * 8;
    vec8 raw{};
    if (r < n) raw = *reinterpret_cast<const vec8*>(vc + cache_row(r) * a.vdim + d);
    const bf16x8 o = bf16(raw);
#pragma unroll
    for (int j = 0; j < 8; ++j) lds[(d + j) * 72 + r] = o.s[j];
  }
  for (int e = threadIdx.x; e < kKvGatherRows * k8; e += 256) {
    const int r = e / k8, d = e % k8 * 8;
    vec8 raw{};
    if (r < n) raw = *reinterpret_cast<const vec8*>(kc + cache_row(r) * a.dim + d);
    *reinterpret_cast<uint4*>(k + int64_t(r) * a.n_kv * a.dim + d) =
        bf16(raw).u;
  }
  __syncthreads();
  uint16_t* vt = reinterpret_cast<uint16_t*>(a.vt) +
                 int64_t(kvh) * a.vdim * a.tokens + row0;
  for (int e = threadIdx.x; e < a.vdim * 8; e += 256) {
    const int d = e / 8, c = e % 8 * 8;
    *reinterpret_cast<uint4*>(vt + int64_t(d) * a.tokens + c) =
        *reinterpret_cast<const uint4*>(lds + d * 72 + c);
  }
}

template <int P, bool BIAS, int MAPS>
void go(const ExpandedAttnArgs& a, hipStream_t st) {
  constexpr size_t smem = size_t(KT * (P + 8) + P * VROW) * 2 * 2;
  static_assert(smem >= size_t(4) * 32 * P * sizeof(float),
                "map 2's output needs the tiles' room");
  auto* k = expanded_attn_kernel<P, BIAS, MAPS>;
  if (smem > 65536)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              int(smem));
  hipLaunchKernelGGL(k, dim3(a.n_tiles * a.heads), dim3(256 * MAPS), smem,
                     st, a);
}

template <bool BIAS, int MAPS>
void by_width(const ExpandedAttnArgs& a, hipStream_t st) {
  const int d = MAPS * a.dim > a.vdim ? MAPS * a.dim : a.vdim;
  if constexpr (MAPS == 1)
    if (d <= 32) return go<32, BIAS, MAPS>(a, st);
  if (d <= 64) return go<64, BIAS, MAPS>(a, st);
  if constexpr (MAPS == 1)
    if (d <= 96) return go<96, BIAS, MAPS>(a, st);
  if (d <= 128) go<128, BIAS, MAPS>(a, st);
  else if (d <= 192) go<192, BIAS, MAPS>(a, st);
  else go<256, BIAS, MAPS>(a, st);
}

}  // namespace

bool expanded_ok(int dim, int vdim, int maps) {
  // a map's key fragments stop where the next map's begin
  return dim % (8 * maps) == 0 && vdim % 8 == 0 && maps * dim <= 256 &&
         vdim <= 256;
}

void launch_expanded_attn(const ExpandedAttnArgs& a, hipStream_t st) {
  if (a.n_tiles == 0) return;
  if (a.maps == 2) by_width<false, 2>(a, st);
  else if (a.r1) by_width<true, 1>(a, st);
  else by_width<false, 1>(a, st);
}

void launch_kv_gather(const KvGatherArgs& a, hipStream_t st) {
  if (a.n == 0) return;
  const dim3 grid(a.n, a.n_kv);
  const size_t smem = size_t(a.vdim) * 72 * 2;
  if (a.cache_kind == kCacheFP8)
    hipLaunchKernelGGL(kv_gather_kernel<CacheFP8>, grid, dim3(256), smem, st,
                       a);
  else
    hipLaunchKernelGGL(kv_gather_kernel<CacheBF16>, grid, dim3(256), smem, st,
                       a);
}

}  // namespace rlli
