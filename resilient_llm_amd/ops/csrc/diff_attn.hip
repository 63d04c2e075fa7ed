// Differential attention: a head has two maps, queries and keys of their own
// over the same values; its output is map 1 - lambda map 2, over its root
// mean square, times a constant and the sigmoid of the head's gate.  Queries
// and keys are normed per head and map and rotated in pairs (i, i + rot / 2),
// scores capped, and a query sees its chunk of positions, counted from the
// sequence's start.
//
//   diff_append   norm and rotate q in place, norm, rotate and cache k, cache
//                 v; biases of all three go in first
//   diff_decode   one new token per sequence, split over the visible cache
//                 blocks; norms, rotation and append fused
// Prompts: expanded_attn.hip; any sizes and the 32-bit path: attn_rows.h.

#include "attn_rows.h"

#include <algorithm>
#include <type_traits>

namespace rlli {
namespace {

typedef short s16x4_t __attribute__((ext_vector_type(4)));
typedef float f32x2_t __attribute__((ext_vector_type(2)));
typedef __bf16 b16x2_t __attribute__((ext_vector_type(2)));

DEV_INLINE uint32_t pack2(float a, float b) {
  const b16x2_t v = __builtin_convertvector((f32x2_t{a, b}), b16x2_t);
  return __builtin_bit_cast(uint32_t, v);
}

// eight neighbours at ``p + off``, zeros unless ``ok``; p itself can always be
// read, so that no load waits behind a branch
template <typename T>
DEV_INLINE void load8(const T* p, int off, bool ok, float (&x)[8]) {
  p += ok ? off : 0;
  const f32x4_t lo = act_load4(p), hi = act_load4(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    x[j] = ok ? lo[j] : 0.f;
    x[4 + j] = ok ? hi[j] : 0.f;
  }
}

// eight neighbours of an activation or cache row
DEV_INLINE void store8(float* p, const float (&x)[8]) {
  act_store4(p, f32x4_t{x[0], x[1], x[2], x[3]});
  act_store4(p + 4, f32x4_t{x[4], x[5], x[6], x[7]});
}
DEV_INLINE void store8(uint16_t* p, const float (&x)[8]) {
  *reinterpret_cast<uint4*>(p) = CacheBF16::from_f32(x);
}
DEV_INLINE void store8(uint8_t* p, const float (&x)[8]) {
  *reinterpret_cast<uint2*>(p) = CacheFP8::from_f32(x);
}

// ---- append --------------------------------------------------------------
// Sum over a group of W lanes that all get it.
template <int W>
DEV_INLINE float lanes_sum(float v) {
  if constexpr (W <= 16) return group_sum_dpp<W>(v);
  v = group_sum_dpp<16>(v);
#pragma unroll
  for (int off = 16; off < W; off <<= 1) v += __shfl_xor(v, off, kWave);
  return v;
}

// W lanes per vector, 8 dimensions each, vectors of all rows in one list: a
// row's query maps, its key maps, its values.  Widths and half the rotation
// are multiples of 8.
template <typename T, typename CE, int W>
__global__ __launch_bounds__(256)
void diff_append_kernel(WindowAttnArgs a) {
  const int nq = a.maps * a.n_q, nk = a.maps * a.n_kv;
  const int per_row = nq + nk + a.n_kv;
  const int64_t unit = int64_t(blockIdx.x) * (256 / W) + threadIdx.x / W;
  if (unit >= int64_t(a.rows) * per_row) return;    // whole groups leave
  const int row = int(unit / per_row), u = int(unit % per_row);
  const int lane = threadIdx.x & 63, gl = lane & (W - 1), d0 = gl * 8;
  const float* bias = a.bias ? a.bias : a.q_norm;
  T* x = reinterpret_cast<T*>(a.qkv_rw) + int64_t(row) * a.stride;
  const int slot = a.slots[row];
  const int64_t blk = slot / a.block_size, off = slot % a.block_size;
  if (u >= nq + nk) {
    const int h = u - nq - nk;
    const T* v = x + (nq + nk) * a.dim + h * a.vdim;
    CE* o = reinterpret_cast<CE*>(a.v_cache) +
            ((blk * a.n_kv + h) * a.block_size + off) * a.vdim;
    for (int d = d0; d < a.vdim; d += W * 8) {
      float e[8], eb[8];
      load8(v, d, true, e);
      load8(bias, (nq + nk) * a.dim + h * a.vdim + d, a.bias, eb);
#pragma unroll
      for (int j = 0; j < 8; ++j) e[j] += eb[j];
      store8(o + d, e);
    }
    return;
  }
  const bool ok = d0 < a.dim;
  const int half = a.rot / 2;
  // this lane's dimensions and their pairs' other halves
  const int p0 = d0 < half ? d0 + half : d0 < a.rot ? d0 - half : -1;
  const int i0 = d0 < half ? d0 : d0 - half;
  const float* cs = a.rot ? a.cos_sin + int64_t(a.positions[row]) * a.rot
                          : a.q_norm;
  const float* w = u < nq ? a.q_norm : a.k_norm;
  float e[8], eb[8], ew[8], o[8], c[8], s[8];
  load8(x + u * a.dim, d0, ok, e);
  load8(bias, u * a.dim + d0, ok && a.bias, eb);
  load8(w, d0, ok, ew);
  load8(cs, i0, p0 >= 0, c);
  load8(cs, half + i0, p0 >= 0, s);
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    e[j] += eb[j];
    ss += e[j] * e[j];
  }
  const float inv = 1.f / sqrtf(lanes_sum<W>(ss) / a.dim + a.eps);
#pragma unroll
  for (int j = 0; j < 8; ++j) e[j] *= inv * ew[j];
  const int from = p0 < 0 ? lane : (lane & ~(W - 1)) + p0 / 8;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    o[j] = __shfl(e[j], from, kWave);
    if (p0 >= 0) e[j] = e[j] * c[j] + (d0 < half ? -o[j] : o[j]) * s[j];
  }
  if (!ok) return;
  if (u < nq) {
    store8(x + u * a.dim + d0, e);
    return;
  }
  const int h = (u - nq) / a.maps, map = (u - nq) % a.maps;
  store8(reinterpret_cast<CE*>(a.k_cache) +
             (((blk * a.n_kv + h) * a.block_size + off) * a.maps + map) *
                 a.dim + d0, e);
}

// the same at any sizes: a wave per vector, which waits in LDS
template <typename T, typename CE>
__global__ __launch_bounds__(64)
void diff_append_any_kernel(WindowAttnArgs a) {
  extern __shared__ float xs[];
  const int nq = a.maps * a.n_q, nk = a.maps * a.n_kv;
  const int row = blockIdx.x, u = blockIdx.y, lane = threadIdx.x;
  T* x = reinterpret_cast<T*>(a.qkv_rw) + int64_t(row) * a.stride;
  const int slot = a.slots[row];
  const int64_t blk = slot / a.block_size, off = slot % a.block_size;
  if (u >= nq + nk) {
    const int h = u - nq - nk;
    const T* v = x + (nq + nk) * a.dim + h * a.vdim;
    CE* o = reinterpret_cast<CE*>(a.v_cache) +
            ((blk * a.n_kv + h) * a.block_size + off) * a.vdim;
    const float* b = a.bias + (nq + nk) * a.dim + h * a.vdim;
    for (int d = lane; d < a.vdim; d += 64)
      cache_store(o + d, act_load(v + d) + (a.bias ? b[d] : 0.f));
    return;
  }
  T* q = x + u * a.dim;
  const float* w = u < nq ? a.q_norm : a.k_norm;
  float ss = 0.f;
  for (int d = lane; d < a.dim; d += 64) {
    const float e = act_load(q + d) + (a.bias ? a.bias[u * a.dim + d] : 0.f);
    ss += e * e;
    xs[d] = e * w[d];
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / a.dim + a.eps);
  __syncthreads();
  const int half = a.rot / 2;
  const float* cs = a.cos_sin + int64_t(a.positions[row]) * a.rot;
  CE* o = nullptr;
  if (u >= nq)
    o = reinterpret_cast<CE*>(a.k_cache) +
        (((blk * a.n_kv + (u - nq) / a.maps) * a.block_size + off) * a.maps +
         (u - nq) % a.maps) * a.dim;
  for (int d = lane; d < a.dim; d += 64) {
    float e = xs[d];
    if (d < half)
      e = e * cs[d] - xs[half + d] * cs[half + d];
    else if (d < a.rot)
      e = e * cs[d - half] + xs[d - half] * cs[d];
    if (o) cache_store(o + d, e * inv);
    else act_store(q + d, e * inv);
  }
}

// ---- decode ----------------------------------------------------------------
// Workgroup = (split, kv head and eight of its query heads, sequence); four
// waves and the splits interleave over the visible 16-token steps.  Scores
// are computed with keys down and (head, map) columns across, a matrix
// product per map whose other columns are zero, so a lane holds four tokens
// of one column: maximum and sum stay with the lane, and the weights are the
// operand of the second product as they are.  That one is transposed (value
// columns down): row n of tile t is value column 8 n + t, so a lane makes its
// operands of all tiles from the four 16-byte pieces that it loads.  The new
// token's key and value do not come through the cache: the first wave of the
// first split makes them, stores them and takes them as a step of one token.
constexpr int kDiffHeads = 8;

template <typename KC>
DEV_INLINE uint4 bits16(typename KC::vec8 raw) {
  if constexpr (std::is_same_v<KC, CacheBF16>) {
    return raw;
  } else {
    float f[8];
    KC::to_f32(raw, f);
    return uint4{pack2(f[0], f[1]), pack2(f[2], f[3]), pack2(f[4], f[5]),
                 pack2(f[6], f[7])};
  }
}

// DC: 32-wide pieces of a map's query and key; VH: 128-wide ones of the values
template <int DC, int VH, typename KC>
__global__ __launch_bounds__(256, VH == 1 ? 2 : 1)
void diff_decode_kernel(WindowAttnArgs a) {
  using elem = typename KC::elem;
  using vec8 = typename KC::vec8;
  constexpr int VD = VH * 128, VROW = VD + 4;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int group = a.n_q / a.n_kv;
  const int n_hb = (group + kDiffHeads - 1) / kDiffHeads;
  const int split = blockIdx.x, seq = blockIdx.z;
  const int kvh = blockIdx.y / n_hb, hb0 = blockIdx.y % n_hb * kDiffHeads;
  const int nh = min(kDiffHeads, group - hb0), head0 = kvh * group + hb0;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int col = lane & 15, g = lane >> 4;   // column or row; k or row octet
  const int map = col & 1, kw = 2 * a.dim;
  const int pos = a.positions[seq];
  const uint16_t* row =
      reinterpret_cast<const uint16_t*>(a.qkv) + int64_t(seq) * a.stride;
  elem* kc = reinterpret_cast<elem*>(a.k_cache);
  elem* vc = reinterpret_cast<elem*>(a.v_cache);

  // this lane's pieces of a vector of ``dim``, normed, times w, rotated, as
  // 16-bit
  const int half = a.rot / 2;
  const float* cs = a.rot ? a.cos_sin + int64_t(pos) * a.rot : a.q_norm;
  const float* bias = a.bias ? a.bias : a.q_norm;
  auto normed = [&](int at, const float* w, bool live, uint4 (&out)[DC]) {
    const uint16_t* x = row + at;
    float e[DC][8], eb[DC][8], o[DC][8], ob[DC][8], ew[DC][8], ow[DC][8];
    float ec[DC][8], es[DC][8], ss = 0.f;
#pragma unroll
    for (int c = 0; c < DC; ++c) {
      // a piece and its pairs' other halves
      const int d = c * 32 + g * 8;
      const int p = d < half ? d + half : d - half, i = d < half ? d : p;
      const bool turns = d < a.rot, in = live && d < a.dim;
      load8(x, d, in, e[c]);
      load8(bias, at + d, in && a.bias, eb[c]);
      load8(x, p, live && turns, o[c]);
      load8(bias, at + p, live && turns && a.bias, ob[c]);
      load8(w, d, d < a.dim, ew[c]);
      load8(w, p, turns, ow[c]);
      load8(cs, i, turns, ec[c]);
      load8(cs, half + i, turns, es[c]);
    }
#pragma unroll
    for (int c = 0; c < DC; ++c)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        e[c][j] += eb[c][j];
        ss += e[c][j] * e[c][j];
      }
    ss += __shfl_xor(ss, 16, kWave);
    ss += __shfl_xor(ss, 32, kWave);
    const float inv = 1.f / sqrtf(ss / a.dim + a.eps);
#pragma unroll
    for (int c = 0; c < DC; ++c) {
      const int d = c * 32 + g * 8;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float u = e[c][j] * inv * ew[c][j];
        const float v = (o[c][j] + ob[c][j]) * inv * ow[c][j];
        e[c][j] = d < a.rot
                      ? u * ec[c][j] + (d < half ? -v : v) * es[c][j] : u;
      }
      out[c] = uint4{pack2(e[c][0], e[c][1]), pack2(e[c][2], e[c][3]),
                     pack2(e[c][4], e[c][5]), pack2(e[c][6], e[c][7])};
    }
  };

  s16x8_t q[2][DC];                     // by map: zero in the other's columns
  {
    uint4 own[DC];
    normed((head0 + min(col / 2, nh - 1)) * kw + map * a.dim, a.q_norm,
           col < 2 * nh, own);
#pragma unroll
    for (int c = 0; c < DC; ++c) {
      const uint4 none = {0, 0, 0, 0};
      q[0][c] = __builtin_bit_cast(s16x8_t, map == 0 ? own[c] : none);
      q[1][c] = __builtin_bit_cast(s16x8_t, map == 1 ? own[c] : none);
    }
  }

  constexpr float kLog2e = 1.4426950408889634f;
  const float cap_in = a.cap > 0.f ? a.scale * kTwoLog2e / a.cap : 0.f;
  const float top = a.cap * kLog2e, plain = a.scale * kLog2e;
  float m = kNegInf, l = 0.f;
  f32x4_t o[VH][8];
#pragma unroll
  for (int v = 0; v < VH; ++v)
#pragma unroll
    for (int t = 0; t < 8; ++t) o[v][t] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  // one step: k[map][piece] of token ``col``, v[piece][token] of tokens
  // 4 g .., which are visible where ``ok``
  auto consume = [&](const uint4 (&k)[2][DC], uint4 (&v)[VH][4],
                     const bool (&ok)[4], bool whole) {
    f32x4_t s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int mp = 0; mp < 2; ++mp)
#pragma unroll
      for (int c = 0; c < DC; ++c)
        s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            __builtin_bit_cast(s16x8_t, k[mp][c]), q[mp][c], s, 0, 0, 0);
    if (a.cap > 0.f) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        s[r] = fmaf(-2.f * top,
                    __builtin_amdgcn_rcpf(
                        1.f + __builtin_amdgcn_exp2f(s[r] * cap_in)),
                    top);
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r) s[r] *= plain;
    }
    if (!whole) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (ok[r]) continue;
        s[r] = kNegInf;
        // slots past the end hold whatever an earlier owner left
#pragma unroll
        for (int h = 0; h < VH; ++h) v[h][r] = uint4{0, 0, 0, 0};
      }
    }
    float mx = fmaxf(fmaxf(s[0], s[1]), fmaxf(s[2], s[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
    mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
    if (__any(mx > m)) {
      const float mn = fmaxf(m, mx);
      const float corr = __builtin_amdgcn_exp2f(m - mn);
      m = mn;
      l *= corr;
#pragma unroll
      for (int h = 0; h < VH; ++h)
#pragma unroll
        for (int t = 0; t < 8; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[h][t][r] *= corr;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[r] = __builtin_amdgcn_exp2f(s[r] - m);
      l += s[r];
    }
    const uint2 praw = {pack2(s[0], s[1]), pack2(s[2], s[3])};
    const s16x4_t p = __builtin_bit_cast(s16x4_t, praw);
#pragma unroll
    for (int h = 0; h < VH; ++h)
#pragma unroll
      for (int t = 0; t < 8; ++t) {
        auto word = [&](const uint4& x) {
          return t / 2 == 0 ? x.x : t / 2 == 1 ? x.y : t / 2 == 2 ? x.z : x.w;
        };
        // the t-th value column of four tokens
        constexpr uint32_t kLow = 0x05040100u, kHigh = 0x07060302u;
        const uint32_t sel = t % 2 ? kHigh : kLow;
        const uint2 raw = {
            __builtin_amdgcn_perm(word(v[h][1]), word(v[h][0]), sel),
            __builtin_amdgcn_perm(word(v[h][3]), word(v[h][2]), sel)};
        o[h][t] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(
            __builtin_bit_cast(s16x4_t, raw), p, o[h][t], 0, 0, 0);
      }
  };

  if (wave == 0 && split == 0) {
    // the new token: its key in columns 0 and 1, then token 0 of a step
    uint4 key[DC], k[2][DC], v[VH][4];
    normed((a.n_q + kvh) * kw + map * a.dim, a.k_norm, true, key);
    const int slot = a.slots[seq];
    const int64_t rowi =
        (int64_t(slot / a.block_size) * a.n_kv + kvh) * a.block_size +
        slot % a.block_size;
    elem* kd = kc + rowi * kw;
    elem* vd = vc + rowi * a.vdim;
    const int v_at = (a.n_q + a.n_kv) * kw + kvh * a.vdim;
#pragma unroll
    for (int c = 0; c < DC; ++c) {
      const int d = c * 32 + g * 8;
      float f[8];
      CacheBF16::to_f32(key[c], f);
      const vec8 raw = [&] {
        if constexpr (std::is_same_v<KC, CacheBF16>) return key[c];
        else return KC::from_f32(f);
      }();
      if (hb0 == 0 && col < 2 && d < a.dim)
        *reinterpret_cast<vec8*>(kd + map * a.dim + d) = raw;
      key[c] = bits16<KC>(raw);
#pragma unroll
      for (int mp = 0; mp < 2; ++mp) {
        // from the lane that has this octet of the map's key
        uint4 x;
        x.x = __shfl(int(key[c].x), g * 16 + mp, kWave);
        x.y = __shfl(int(key[c].y), g * 16 + mp, kWave);
        x.z = __shfl(int(key[c].z), g * 16 + mp, kWave);
        x.w = __shfl(int(key[c].w), g * 16 + mp, kWave);
        k[mp][c] = col == 0 ? x : uint4{0, 0, 0, 0};
      }
    }
    bool ok[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) ok[r] = g == 0 && r == 0;
#pragma unroll
    for (int h = 0; h < VH; ++h) {
      const int d = h * 128 + col * 8;
      float f[8], b[8];
      load8(row, v_at + d, d < a.vdim, f);
      load8(bias, v_at + d, d < a.vdim && a.bias, b);
#pragma unroll
      for (int j = 0; j < 8; ++j) f[j] += b[j];
      const vec8 raw = KC::from_f32(f);
      if (hb0 == 0 && g == 0 && d < a.vdim)
        *reinterpret_cast<vec8*>(vd + d) = raw;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[h][r] = bits16<KC>(raw);
    }
    consume(k, v, ok, false);
  }

  const int lo = first_seen(a, pos), len = pos;     // cached tokens
  const int step0 = lo / 16, n_steps = (len + 15) / 16 - step0;
  const int32_t* bt = a.block_tables + int64_t(seq) * a.max_blocks;
  auto fetch_phys = [&](int b) { return bt[(b * 16) / a.block_size]; };
  // past a key's or value's end a lane loads its first piece: there the
  // queries are zero, and nobody reads the output columns
  auto issue = [&](int b, int phys, vec8 (&kr)[2][DC], vec8 (&vr)[VH][4]) {
    const int64_t base = (int64_t(phys) * a.n_kv + kvh) * a.block_size +
                         (b * 16) % a.block_size;
    const elem* kp = kc + (base + col) * kw;
    const elem* vp = vc + (base + g * 4) * a.vdim;
#pragma unroll
    for (int mp = 0; mp < 2; ++mp)
#pragma unroll
      for (int c = 0; c < DC; ++c) {
        const int d = c * 32 + g * 8;
        kr[mp][c] = *reinterpret_cast<const vec8*>(
            kp + mp * a.dim + (d < a.dim ? d : 0));
      }
#pragma unroll
    for (int h = 0; h < VH; ++h) {
      const int d = h * 128 + col * 8;
#pragma unroll
      for (int r = 0; r < 4; ++r)
        vr[h][r] = *reinterpret_cast<const vec8*>(
            vp + r * a.vdim + (d < a.vdim ? d : 0));
    }
  };
  auto take = [&](int b, const vec8 (&kr)[2][DC], const vec8 (&vr)[VH][4]) {
    uint4 k[2][DC], v[VH][4];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp)
#pragma unroll
      for (int c = 0; c < DC; ++c) k[mp][c] = bits16<KC>(kr[mp][c]);
#pragma unroll
    for (int h = 0; h < VH; ++h)
#pragma unroll
      for (int r = 0; r < 4; ++r) v[h][r] = bits16<KC>(vr[h][r]);
    bool ok[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = b * 16 + g * 4 + r;
      ok[r] = j < len && j >= lo;
    }
    consume(k, v, ok, b * 16 >= lo && b * 16 + 16 <= len);
  };

  // two steps in registers: one in use, the next one's loads in flight, and
  // the block number of the one after
  const int stride = 4 * a.n_split;
  int i = split * 4 + wave;
  if (i < n_steps) {
    vec8 kA[2][DC], vA[VH][4], kB[2][DC], vB[VH][4];
    int phys = 0;
    issue(step0 + i, fetch_phys(step0 + i), kA, vA);
    if (i + stride < n_steps) phys = fetch_phys(step0 + i + stride);
    while (true) {
      if (i + stride < n_steps) {
        issue(step0 + i + stride, phys, kB, vB);
        if (i + 2 * stride < n_steps)
          phys = fetch_phys(step0 + i + 2 * stride);
      }
      take(step0 + i, kA, vA);
      i += stride;
      if (i >= n_steps) break;
      if (i + stride < n_steps) {
        issue(step0 + i + stride, phys, kA, vA);
        if (i + 2 * stride < n_steps)
          phys = fetch_phys(step0 + i + 2 * stride);
      }
      take(step0 + i, kB, vB);
      i += stride;
      if (i >= n_steps) break;
    }
  }

  // the waves' results side by side: [wave][column][VROW], then (m, l)
  l += __shfl_xor(l, 16, kWave);
  l += __shfl_xor(l, 32, kWave);
  float* s_ml = lds + 4 * 16 * VROW;
  if (col < 2 * nh) {
    float* out = lds + (wave * 16 + col) * VROW;
#pragma unroll
    for (int h = 0; h < VH; ++h)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float* p = out + h * 128 + (g * 4 + r) * 8;
        act_store4(p, f32x4_t{o[h][0][r], o[h][1][r], o[h][2][r], o[h][3][r]});
        act_store4(p + 4,
                   f32x4_t{o[h][4][r], o[h][5][r], o[h][6][r], o[h][7][r]});
      }
    if (g == 0) {
      s_ml[(wave * 16 + col) * 2] = m;
      s_ml[(wave * 16 + col) * 2 + 1] = l;
    }
  }
  __syncthreads();
  // a wave per head; a lane holds columns lane, lane + 64, ..
  constexpr int NV = VD / 64;
  for (int h = wave; h < nh; h += 4) {
    float x[2][NV];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
      const int u = h * 2 + mp;
      float mm = kNegInf, ll = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) mm = fmaxf(mm, s_ml[(w * 16 + u) * 2]);
#pragma unroll
      for (int i = 0; i < NV; ++i) x[mp][i] = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const float c = __builtin_amdgcn_exp2f(s_ml[(w * 16 + u) * 2] - mm);
        ll += s_ml[(w * 16 + u) * 2 + 1] * c;
#pragma unroll
        for (int i = 0; i < NV; ++i)
          x[mp][i] += lds[(w * 16 + u) * VROW + i * 64 + lane] * c;
      }
      if (a.n_split > 1) {
        const int64_t pi =
            ((int64_t(seq) * a.n_q + head0 + h) * 2 + mp) * a.n_split + split;
#pragma unroll
        for (int i = 0; i < NV; ++i)
          if (i * 64 + lane < a.vdim)
            a.part_acc[pi * a.vdim + i * 64 + lane] = x[mp][i];
        if (lane == 0) {
          a.part_ml[pi * 2] = mm;
          a.part_ml[pi * 2 + 1] = ll;
        }
      } else {
        const float inv = 1.f / ll;
#pragma unroll
        for (int i = 0; i < NV; ++i) x[mp][i] *= inv;
      }
    }
    if (a.n_split > 1) continue;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      x[0][i] -= a.lambda * x[1][i];
      if (i * 64 + lane < a.vdim) ss += x[0][i] * x[0][i];
    }
    float post = a.out_scale / sqrtf(wave_sum(ss) / a.vdim + a.eps);
    if (a.gate)
      post /= 1.f + __expf(-act_load(reinterpret_cast<const uint16_t*>(
                                         a.gate) +
                                     seq * a.gate_stride + head0 + h));
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out) +
                    (int64_t(seq) * a.n_q + head0 + h) * a.vdim;
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (i * 64 + lane < a.vdim)
        act_store(out + i * 64 + lane, x[0][i] * post);
  }
}

// One workgroup per (sequence, head), half its threads per map, one value
// column each: the splits (maxima in powers of two), the maps' difference, its
// norm and gate.
// SPLITS: at least as many as there are.
template <int SPLITS>
__global__ __launch_bounds__(512)
void diff_combine_kernel(WindowAttnArgs a) {
  __shared__ float second[256], part[4];
  const int64_t row = blockIdx.x;               // seq * n_q + head
  const int cols = blockDim.x / 2, map = int(threadIdx.x) >= cols;
  const int lane = threadIdx.x & 63, d = threadIdx.x - map * cols;
  const bool mine = lane < a.n_split, live = d < a.vdim;
  const int64_t p0 = (row * 2 + map) * a.n_split;
  const float* p = a.part_acc + p0 * a.vdim + (live ? d : 0);
  float x[SPLITS];
#pragma unroll
  for (int s = 0; s < SPLITS; ++s)
    x[s] = p[min(s, a.n_split - 1) * a.vdim];
  const float2 ml = reinterpret_cast<const float2*>(
      a.part_ml)[p0 + (mine ? lane : 0)];
  const float mm = wave_max(mine ? ml.x : kNegInf);
  const float c = mine ? __builtin_amdgcn_exp2f(ml.x - mm) : 0.f;
  const float ll = wave_sum(c * ml.y);
  float t = 0.f;
#pragma unroll
  for (int s = 0; s < SPLITS; ++s)         // weight 0 past the last
    t += x[s] * __shfl(c, s, kWave);
  t /= ll;
  if (map) second[d] = t;
  __syncthreads();
  float v = 0.f;
  if (!map) {
    if (live) v = t - a.lambda * second[d];
    const float ws = wave_sum(v * v);
    if (lane == 0) part[threadIdx.x >> 6] = ws;
  }
  __syncthreads();
  if (map || !live) return;
  float ss = 0.f;
  for (int w = 0; w < cols / 64; ++w) ss += part[w];
  float post = a.out_scale / sqrtf(ss / a.vdim + a.eps);
  if (a.gate)
    post /= 1.f + __expf(-act_load(reinterpret_cast<const uint16_t*>(a.gate) +
                                   row / a.n_q * a.gate_stride + row % a.n_q));
  act_store(reinterpret_cast<uint16_t*>(a.out) + row * a.vdim + d, v * post);
}

template <typename F>
void with_cache(const WindowAttnArgs& a, F f) {
  if (a.cache == kCacheFP8) f(uint16_t{}, uint8_t{});
  else if (a.f32) f(float{}, float{});
  else f(uint16_t{}, uint16_t{});
}

template <int DC, int VH, typename KC>
void run_decode(const WindowAttnArgs& a, hipStream_t st) {
  constexpr size_t smem = size_t(4) * 16 * (VH * 128 + 4 + 2) * sizeof(float);
  auto* k = diff_decode_kernel<DC, VH, KC>;
  if (smem > 65536)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              int(smem));
  hipLaunchKernelGGL(
      k, dim3(a.n_split, a.n_kv * diff_head_blocks(a.n_q / a.n_kv), a.rows),
      dim3(256), smem, st, a);
}

}  // namespace

int diff_head_blocks(int group) {
  return (group + kDiffHeads - 1) / kDiffHeads;
}

bool diff_fast_ok(const WindowAttnArgs& a) {
  return !a.f32 && a.dim % 8 == 0 && a.rot % 16 == 0 && a.vdim % 8 == 0 &&
         a.dim <= 128 && a.vdim <= 256 && a.block_size % 16 == 0 &&
         a.stride % 8 == 0;
}

void launch_diff_append(const WindowAttnArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  const int per_row = a.maps * a.n_q + (a.maps + 1) * a.n_kv;
  const bool vec = a.dim % 8 == 0 && a.rot % 16 == 0 && a.vdim % 8 == 0 &&
                   a.stride % 8 == 0 && a.dim <= 256;
  with_cache(a, [&](auto t, auto c) {
    using T = decltype(t);
    using CE = decltype(c);
    auto run = [&](auto w) {
      constexpr int W = decltype(w)::value;
      const int64_t threads = int64_t(a.rows) * per_row * W;
      hipLaunchKernelGGL((diff_append_kernel<T, CE, W>),
                         dim3(uint32_t((threads + 255) / 256)), dim3(256), 0,
                         st, a);
    };
    if (!vec)
      hipLaunchKernelGGL((diff_append_any_kernel<T, CE>),
                         dim3(a.rows, per_row), dim3(64),
                         a.dim * sizeof(float), st, a);
    else if (a.dim <= 32) run(std::integral_constant<int, 4>{});
    else if (a.dim <= 64) run(std::integral_constant<int, 8>{});
    else if (a.dim <= 128) run(std::integral_constant<int, 16>{});
    else run(std::integral_constant<int, 32>{});
  });
}

void launch_diff_rows(const WindowAttnArgs& a, bool decode, hipStream_t st) {
  with_cache(a, [&](auto t, auto c) {
    run_window_rows<decltype(t), decltype(c), 8, 2>(a, decode, st);
  });
}

void launch_diff_decode(const WindowAttnArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  auto go = [&](auto dc, auto vh) {
    constexpr int DC = decltype(dc)::value, VH = decltype(vh)::value;
    if (a.cache == kCacheFP8) run_decode<DC, VH, CacheFP8>(a, st);
    else run_decode<DC, VH, CacheBF16>(a, st);
  };
  auto by_value = [&](auto dc) {
    if (a.vdim <= 128) go(dc, std::integral_constant<int, 1>{});
    else go(dc, std::integral_constant<int, 2>{});
  };
  if (a.dim <= 32) by_value(std::integral_constant<int, 1>{});
  else if (a.dim <= 64) by_value(std::integral_constant<int, 2>{});
  else by_value(std::integral_constant<int, 4>{});
  if (a.n_split == 1) return;
  auto combine = [&](auto* k) {
    hipLaunchKernelGGL(k, dim3(a.rows * a.n_q),
                       dim3((a.vdim + 63) / 64 * 128), 0, st, a);
  };
  if (a.n_split <= 2) combine(diff_combine_kernel<2>);
  else if (a.n_split <= 8) combine(diff_combine_kernel<8>);
  else combine(diff_combine_kernel<16>);
}

}  // namespace rlli
