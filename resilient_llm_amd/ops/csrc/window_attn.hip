// Attention with a sliding window, kept first tokens and a sink.
//
// A query at position i sees key j when j <= i and (i - j < window or
// j < keep_first); the softmax denominator carries one extra exp(sink)
// per head.  Rotation is the interleaved layout (pairs 2i, 2i+1) over
// the first `rot` dimensions (0: none).  Key and value widths may differ,
// and a layer may read keys and values that an earlier layer cached.
// Optional: a distance bias per head (a score loses r1 ln(1 + r2 distance)),
// a query temperature by position (in the scale), values cached over their
// root mean square.
//
// Differential attention (two maps per head, see attn.h) comes with normed
// queries and keys, rotation of pairs (i, i + rot / 2), capped scores and
// chunks instead of a window: a query sees what lies in its chunk of
// positions, counted from the sequence's start.
//
// Kernels here:
//   window_rope_append  rotate q in place, rotate and cache k, cache v
//   diff_append         the same for two maps, norms included
//   window_decode       one new token per sequence, split over the
//                       visible cache blocks; norms, rotation and append
//                       fused; one map or two
// attn_rows.h has window_rows, any sizes and dtypes: the 32-bit path and
// the shapes that the tiled kernels do not take.
// The tiled prefill kernel is window_prefill.hip.

#include "attn_rows.h"

#include <algorithm>
#include <type_traits>

namespace rlli {
namespace {

template <typename T, typename CE>
__global__ __launch_bounds__(256)
void rope_append_kernel(WindowAttnArgs a) {
  const int row = blockIdx.x;
  const int pos = a.positions[row];
  const int half = a.rot / 2;
  const float* cs = a.cos_sin + int64_t(pos) * a.rot;
  T* q = reinterpret_cast<T*>(a.qkv_rw) + int64_t(row) * a.stride;
  for (int e = threadIdx.x; e < a.n_q * half; e += blockDim.x) {
    const int h = e / half, i = e % half;
    T* p = q + h * a.dim + 2 * i;
    const float u = act_load(p), v = act_load(p + 1);
    act_store(p, u * cs[i] - v * cs[half + i]);
    act_store(p + 1, v * cs[i] + u * cs[half + i]);
  }
  if (!a.has_kv) return;
  const int slot = a.slots[row];
  const int64_t blk = slot / a.block_size;
  const int off = slot % a.block_size;
  CE* kc = reinterpret_cast<CE*>(a.k_cache);
  CE* vc = reinterpret_cast<CE*>(a.v_cache);
  const T* k = q + a.n_q * a.dim;
  for (int e = threadIdx.x; e < a.n_kv * a.dim; e += blockDim.x) {
    const int h = e / a.dim, d = e % a.dim;
    float val = act_load(k + e);
    if (d < a.rot) {
      const int i = d >> 1;
      const float other = act_load(k + e + ((d & 1) ? -1 : 1));
      val = (d & 1) ? val * cs[i] + other * cs[half + i]
                    : val * cs[i] - other * cs[half + i];
    }
    cache_store(kc + ((blk * a.n_kv + h) * a.block_size + off) * a.dim + d,
                val);
  }
  const T* v = k + a.n_kv * a.dim;
  if (a.v_norm) {                         // one wave per head
    const int lane = threadIdx.x & 63;
    for (int h = threadIdx.x >> 6; h < a.n_kv; h += 4) {
      CE* o = vc + ((blk * a.n_kv + h) * a.block_size + off) * a.vdim;
      float ss = 0.f;
      for (int d = lane; d < a.vdim; d += 64) {
        const float x = act_load(v + h * a.vdim + d);
        ss += x * x;
      }
      const float inv = 1.f / sqrtf(wave_sum(ss) / a.vdim + a.v_eps);
      for (int d = lane; d < a.vdim; d += 64)
        cache_store(o + d, act_load(v + h * a.vdim + d) * inv);
    }
    return;
  }
  for (int e = threadIdx.x; e < a.n_kv * a.vdim; e += blockDim.x) {
    const int h = e / a.vdim, d = e % a.vdim;
    cache_store(vc + ((blk * a.n_kv + h) * a.block_size + off) * a.vdim + d,
                act_load(v + e));
  }
}

// ---- normed and half-rotated vectors -----------------------------------
// Sum over a group of W lanes that all get it.
template <int W>
DEV_INLINE float lanes_sum(float v) {
  if constexpr (W <= 16) return group_sum_dpp<W>(v);
  v = group_sum_dpp<16>(v);
#pragma unroll
  for (int off = 16; off < W; off <<= 1) v += __shfl_xor(v, off, kWave);
  return v;
}

// What a lane needs for its 8 dimensions d0.. of a vector of ``dim``: the
// norm's weights, cosines and sines, and the lane with the other halves of
// its pairs.  Widths are multiples of 8, half the rotation too.
struct HalfTurn {
  float c[8], s[8];
  int partner;               // lane of the group, or -1
  DEV_INLINE void load(const WindowAttnArgs& a, int pos, int d0, int gl) {
    const int half = a.rot / 2;
    partner = d0 < half ? gl + half / 8 : d0 < a.rot ? gl - half / 8 : -1;
    const float* cs = a.cos_sin + int64_t(pos) * a.rot;
    const int i0 = d0 < half ? d0 : d0 - half;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      c[j] = partner < 0 ? 1.f : cs[i0 + j];
      s[j] = partner < 0 ? 0.f : d0 < half ? -cs[half + i0 + j]
                                           : cs[half + i0 + j];
    }
  }
};

// x (zeros past the end) normed over W lanes, times w, rotated
template <int W>
DEV_INLINE void norm_turn(float (&x)[8], const float (&w)[8],
                          const HalfTurn& turn, int dim, float eps,
                          int lane) {
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) ss += x[j] * x[j];
  const float inv = 1.f / sqrtf(lanes_sum<W>(ss) / dim + eps);
  const int from = turn.partner < 0 ? lane : (lane & ~(W - 1)) + turn.partner;
#pragma unroll
  for (int j = 0; j < 8; ++j) x[j] *= inv * w[j];
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const float other = __shfl(x[j], from, kWave);
    x[j] = x[j] * turn.c[j] + other * turn.s[j];
  }
}

template <typename T>
DEV_INLINE void load8(const T* p, bool ok, float (&x)[8]) {
#pragma unroll
  for (int j = 0; j < 8; ++j) x[j] = 0.f;
  if (!ok) return;
  const f32x4_t lo = act_load4(p), hi = act_load4(p + 4);
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    x[j] = lo[j];
    x[4 + j] = hi[j];
  }
}

// W lanes per vector, vectors of all rows in one list: a row's query maps,
// its key maps, its values
template <typename T, typename CE, int W>
__global__ __launch_bounds__(256)
void diff_append_kernel(WindowAttnArgs a) {
  const int nq = a.maps * a.n_q, nk = a.maps * a.n_kv;
  const int per_row = nq + nk + a.n_kv;
  const int64_t unit = int64_t(blockIdx.x) * (256 / W) + threadIdx.x / W;
  if (unit >= int64_t(a.rows) * per_row) return;    // whole groups leave
  const int row = int(unit / per_row), u = int(unit % per_row);
  const int lane = threadIdx.x & 63, gl = lane & (W - 1), d0 = gl * 8;
  T* x = reinterpret_cast<T*>(a.qkv_rw) + int64_t(row) * a.stride;
  const int slot = a.slots[row];
  const int64_t blk = slot / a.block_size, off = slot % a.block_size;
  if (u >= nq + nk) {
    const int h = u - nq - nk;
    const T* v = x + (nq + nk) * a.dim + h * a.vdim;
    CE* o = reinterpret_cast<CE*>(a.v_cache) +
            ((blk * a.n_kv + h) * a.block_size + off) * a.vdim;
    for (int d = d0; d < a.vdim; d += W * 8) {
      float e[8];
      load8(v + d, true, e);
#pragma unroll
      for (int j = 0; j < 8; ++j) cache_store(o + d + j, e[j]);
    }
    return;
  }
  const bool ok = d0 < a.dim;
  float e[8], w[8];
  HalfTurn turn;
  load8(x + u * a.dim + d0, ok, e);
  load8((u < nq ? a.q_norm : a.k_norm) + d0, ok, w);
  turn.load(a, a.positions[row], d0, gl);
  norm_turn<W>(e, w, turn, a.dim, a.eps, lane);
  if (!ok) return;
  if (u < nq) {
    T* q = x + u * a.dim + d0;
    act_store4(q, f32x4_t{e[0], e[1], e[2], e[3]});
    act_store4(q + 4, f32x4_t{e[4], e[5], e[6], e[7]});
    return;
  }
  const int h = (u - nq) / a.maps, map = (u - nq) % a.maps;
  CE* o = reinterpret_cast<CE*>(a.k_cache) +
          (((blk * a.n_kv + h) * a.block_size + off) * a.maps + map) * a.dim +
          d0;
#pragma unroll
  for (int j = 0; j < 8; ++j) cache_store(o + j, e[j]);
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
    for (int d = lane; d < a.vdim; d += 64) cache_store(o + d, act_load(v + d));
    return;
  }
  T* q = x + u * a.dim;
  const float* w = u < nq ? a.q_norm : a.k_norm;
  float ss = 0.f;
  for (int d = lane; d < a.dim; d += 64) {
    const float e = act_load(q + d);
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

// ---- decode: one new token per sequence -------------------------------
// Workgroup = (sequence, kv head, HB query heads, split).  A wave splits
// into 64/GW lane groups of GW lanes; a lane owns 8 dimensions, a group
// walks TPG of the 16 tokens of a step, waves and splits interleave over
// the visible steps.  The new token's own term never touches the cache:
// group 0 of wave 0 of split 0 folds it in from registers while it
// appends, so no wave waits on a cache write of this launch.
// Two maps: the halves of a lane group hold a map's query and key each, and
// its maximum and sum; every lane weights its values with both maps.
template <int GW, int HB, typename KC, bool BIAS, int MAPS>
__global__ __launch_bounds__(256)
void window_decode_kernel(WindowAttnArgs a) {
  constexpr int GPW = 64 / GW;
  constexpr int LW = GW / MAPS;                // lanes of a query or key
  constexpr int TPG = 16 / GPW > 0 ? 16 / GPW : 1;
  constexpr int DMAX = GW * 8;
  using elem = typename KC::elem;
  using vec8 = typename KC::vec8;
  const int split = blockIdx.x;
  const int group = a.n_q / a.n_kv;
  const int n_hb = (group + HB - 1) / HB;
  const int kvh = blockIdx.y / n_hb;
  const int hb0 = (blockIdx.y % n_hb) * HB;
  const int nh = min(HB, group - hb0);         // live heads here
  const int seq = blockIdx.z;
  const int lane = threadIdx.x & 63;
  const int wave = threadIdx.x >> 6;
  const int grp = lane / GW;
  const int gl = lane % GW;
  const int d0 = gl * 8;                       // of the values
  const int map = gl / LW, e0 = (gl % LW) * 8; // of a map's queries and keys
  const int kw = MAPS * a.dim, k0 = map * a.dim + e0;
  const bool kd = e0 < a.dim, vd = d0 < a.vdim;
  const int pos = a.positions[seq];
  const int head0 = kvh * group + hb0;

  const uint16_t* qrow =
      reinterpret_cast<const uint16_t*>(a.qkv) + int64_t(seq) * a.stride;
  const float* cs = a.cos_sin + int64_t(pos) * a.rot;
  const int half = a.rot / 2;

  // in-lane rotation: a lane's 8 dims are 4 whole pairs
  float rc[4], rs[4];
  HalfTurn turn;
  float qw[8];
  if constexpr (MAPS == 1) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int p = d0 / 2 + i;
      rc[i] = p < half ? cs[p] : 1.f;
      rs[i] = p < half ? cs[half + p] : 0.f;
    }
  } else {
    turn.load(a, pos, e0, gl % LW);
    load8(a.q_norm + e0, kd, qw);
  }
  auto load8_rot = [&](const uint16_t* p, bool ok, float* out8) {
    bf16x8 raw;
    raw.u = uint4{0, 0, 0, 0};
    if (ok) raw.u = *reinterpret_cast<const uint4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float u = bf16_to_f32(raw.s[2 * i]);
      const float v = bf16_to_f32(raw.s[2 * i + 1]);
      out8[2 * i] = u * rc[i] - v * rs[i];
      out8[2 * i + 1] = v * rc[i] + u * rs[i];
    }
  };

  const float scale = a.scale * query_temp(pos, a.temp_coef, a.temp_every);
  float r1[HB], r2[HB];
  if constexpr (BIAS)
#pragma unroll
    for (int h = 0; h < HB; ++h) {
      r1[h] = h < nh ? a.r1[head0 + h] : 0.f;
      r2[h] = h < nh ? a.r2[head0 + h] : 0.f;
    }
  const float c2 = a.cap > 0.f ? kTwoLog2e / a.cap : 0.f;
  // acc: of the lane's own map; oth: of the other one
  float qv[HB][8], m[HB], l[HB], acc[HB][8], oth[MAPS == 2 ? HB : 1][8];
#pragma unroll
  for (int h = 0; h < HB; ++h) {
    const uint16_t* q = qrow + (head0 + h) * kw + k0;
    if constexpr (MAPS == 1) {
      load8_rot(q, kd && h < nh, qv[h]);
    } else {
      load8(q, kd && h < nh, qv[h]);
      norm_turn<LW>(qv[h], qw, turn, a.dim, a.eps, lane);
#pragma unroll
      for (int i = 0; i < 8; ++i) oth[h][i] = 0.f;
    }
    // the prompt path rounds rotated queries to bf16 for its matrix
    // cores; round here too so both paths score the same values
#pragma unroll
    for (int i = 0; i < 8; ++i) qv[h][i] = bf16_to_f32(f32_to_bf16(qv[h][i]));
    m[h] = kNegInf;
    l[h] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[h][i] = 0.f;
  }

  auto gsum = [&](float v) { return lanes_sum<LW>(v); };
  // what the lanes of the other map hold, the same in all of them
  auto other = [&](float v) {
    if constexpr (LW == 2) return dpp_mov_f32<0x4E>(v);
    else if constexpr (LW == 4) return dpp_mov_f32<0x141>(v);
    else if constexpr (LW == 8) return dpp_mov_f32<0x140>(v);
    else return __shfl_xor(v, LW, kWave);
  };

  elem* kc = reinterpret_cast<elem*>(a.k_cache);
  elem* vc = reinterpret_cast<elem*>(a.v_cache);
  int len = pos + 1;                            // cached tokens to walk
  if (a.has_kv) {
    len = pos;
    if (wave == 0 && grp == 0 && split == 0) {
      float kf[8], vf[8];
      const uint16_t* kr = qrow + (a.n_q + kvh) * kw + k0;
      if constexpr (MAPS == 1) {
        load8_rot(kr, kd, kf);
      } else {
        float w[8];
        load8(a.k_norm + e0, kd, w);
        load8(kr, kd, kf);
        norm_turn<LW>(kf, w, turn, a.dim, a.eps, lane);
      }
      bf16x8 vr;
      vr.u = uint4{0, 0, 0, 0};
      if (vd)
        vr.u = *reinterpret_cast<const uint4*>(
            qrow + (a.n_q + a.n_kv) * kw + kvh * a.vdim + d0);
#pragma unroll
      for (int i = 0; i < 8; ++i) vf[i] = bf16_to_f32(vr.s[i]);
      if (a.v_norm) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += vf[i] * vf[i];
        const float inv = 1.f / sqrtf(gsum(ss) / a.vdim + a.v_eps);
#pragma unroll
        for (int i = 0; i < 8; ++i) vf[i] *= inv;
      }
      const int slot = a.slots[seq];
      const int64_t rowi =
          (int64_t(slot / a.block_size) * a.n_kv + kvh) * a.block_size +
          slot % a.block_size;
      const vec8 kraw = KC::from_f32(kf);
      const vec8 vw = KC::from_f32(vf);
      if (hb0 == 0) {
        if (kd) *reinterpret_cast<vec8*>(kc + rowi * kw + k0) = kraw;
        if (vd) *reinterpret_cast<vec8*>(vc + rowi * a.vdim + d0) = vw;
      }
      KC::to_f32(kraw, kf);
      KC::to_f32(vw, vf);
#pragma unroll
      for (int h = 0; h < HB; ++h) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) s += qv[h][i] * kf[i];
        m[h] = gsum(s) * scale;
        if (a.cap > 0.f) m[h] = fast_cap(m[h], a.cap, c2);
        l[h] = 1.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          acc[h][i] = vf[i];
          if constexpr (MAPS == 2) oth[h][i] = vf[i];
        }
      }
    }
  }

  // visible 16-token steps: those of the kept tokens, then the window's
  const int lo = first_seen(a, pos);
  const int n_all = (len + 15) / 16;
  int w0 = lo / 16;
  int kb = min((a.keep_first + 15) / 16, n_all);
  if (kb >= w0) {
    kb = 0;
    if (a.keep_first > 0) w0 = 0;
  }
  const int n_steps = kb + max(0, n_all - w0);
  const int32_t* bt = a.block_tables + int64_t(seq) * a.max_blocks;

  auto step_block = [&](int i) { return i < kb ? i : w0 + (i - kb); };
  auto fetch_phys = [&](int b) { return bt[(b * 16) / a.block_size]; };
  auto issue = [&](int b, int phys, vec8 (&kr)[TPG], vec8 (&vr)[TPG]) {
    const int64_t base = (int64_t(phys) * a.n_kv + kvh) * a.block_size +
                         (b * 16) % a.block_size;
#pragma unroll
    for (int i = 0; i < TPG; ++i) {
      const int tok = grp + GPW * i;
      kr[i] = vec8{};
      vr[i] = vec8{};
      if (kd) kr[i] = *reinterpret_cast<const vec8*>(
          kc + (base + tok) * kw + k0);
      if (vd) vr[i] = *reinterpret_cast<const vec8*>(
          vc + (base + tok) * a.vdim + d0);
    }
  };
  auto consume = [&](int b, const vec8 (&kr)[TPG], const vec8 (&vr)[TPG]) {
    float vf[TPG][8], sv[HB][TPG];
#pragma unroll
    for (int i = 0; i < TPG; ++i) {
      const int j = b * 16 + grp + GPW * i;
      const bool ok = j < len && (j >= lo || j < a.keep_first);
      float kf[8];
      KC::to_f32(kr[i], kf);
      KC::to_f32(vr[i], vf[i]);
#pragma unroll
      for (int h = 0; h < HB; ++h) {
        float s = 0.f;
#pragma unroll
        for (int d = 0; d < 8; ++d) s += qv[h][d] * kf[d];
        s = gsum(s) * scale;
        if constexpr (MAPS == 2)
          if (a.cap > 0.f) s = fast_cap(s, a.cap, c2);
        if constexpr (BIAS)
          s -= r1[h] * __logf(fmaf(r2[h], float(max(pos - j, 0)), 1.f));
        sv[h][i] = ok ? s : kNegInf;
      }
      // slots past the end hold whatever an earlier owner left
      if (!ok) {
#pragma unroll
        for (int d = 0; d < 8; ++d) vf[i][d] = 0.f;
      }
    }
#pragma unroll
    for (int h = 0; h < HB; ++h) {
      float mn = m[h];
#pragma unroll
      for (int i = 0; i < TPG; ++i) mn = fmaxf(mn, sv[h][i]);
      const float corr = __expf(m[h] - mn);
      float p[TPG], ps = 0.f;
#pragma unroll
      for (int i = 0; i < TPG; ++i) {
        p[i] = __expf(sv[h][i] - mn);
        ps += p[i];
      }
      m[h] = mn;
      l[h] = l[h] * corr + ps;
#pragma unroll
      for (int d = 0; d < 8; ++d) {
        float t = acc[h][d] * corr;
#pragma unroll
        for (int i = 0; i < TPG; ++i) t += p[i] * vf[i][d];
        acc[h][d] = t;
      }
      if constexpr (MAPS == 2) {
        const float co = other(corr);
#pragma unroll
        for (int i = 0; i < TPG; ++i) p[i] = other(p[i]);
#pragma unroll
        for (int d = 0; d < 8; ++d) {
          float t = oth[h][d] * co;
#pragma unroll
          for (int i = 0; i < TPG; ++i) t += p[i] * vf[i][d];
          oth[h][d] = t;
        }
      }
    }
  };

  const int stride = 4 * a.n_split;
  int i = split * 4 + wave;
  if (i < n_steps) {
    vec8 kA[TPG], vA[TPG], kB[TPG], vB[TPG];
    int bA = step_block(i), bB = 0, physB = 0;
    issue(bA, fetch_phys(bA), kA, vA);
    if (i + stride < n_steps) {
      bB = step_block(i + stride);
      physB = fetch_phys(bB);
    }
    while (true) {
      int physA = 0, bN = 0;
      if (i + stride < n_steps) {
        issue(bB, physB, kB, vB);
        if (i + 2 * stride < n_steps) {
          bN = step_block(i + 2 * stride);
          physA = fetch_phys(bN);
        }
      }
      consume(bA, kA, vA);
      i += stride;
      if (i >= n_steps) break;
      bA = bN;
      int bN2 = 0;
      if (i + stride < n_steps) {
        issue(bA, physA, kA, vA);
        if (i + 2 * stride < n_steps) {
          bN2 = step_block(i + 2 * stride);
          physB = fetch_phys(bN2);
        }
      }
      consume(bB, kB, vB);
      i += stride;
      if (i >= n_steps) break;
      bB = bN2;
    }
  }

  // merge sibling lane groups, then waves
#pragma unroll
  for (int off = GW; off < 64; off <<= 1) {
#pragma unroll
    for (int h = 0; h < HB; ++h) {
      const float mo = __shfl_xor(m[h], off, kWave);
      const float lo2 = __shfl_xor(l[h], off, kWave);
      const float mn = fmaxf(m[h], mo);
      const float ca = __expf(m[h] - mn), cb = __expf(mo - mn);
      m[h] = mn;
      l[h] = l[h] * ca + lo2 * cb;
#pragma unroll
      for (int d = 0; d < 8; ++d)
        acc[h][d] = acc[h][d] * ca + __shfl_xor(acc[h][d], off, kWave) * cb;
      if constexpr (MAPS == 2) {
        const float oa = other(ca), ob = other(cb);
#pragma unroll
        for (int d = 0; d < 8; ++d)
          oth[h][d] = oth[h][d] * oa + __shfl_xor(oth[h][d], off, kWave) * ob;
      }
    }
  }
  __shared__ float s_acc[4][HB * MAPS][DMAX];
  __shared__ float s_ml[4][HB * MAPS][2];
  if (grp == 0) {
#pragma unroll
    for (int h = 0; h < HB; ++h) {
#pragma unroll
      for (int d = 0; d < 8; ++d)
        s_acc[wave][h * MAPS + map][d0 + d] = acc[h][d];
      if constexpr (MAPS == 2)
#pragma unroll
        for (int d = 0; d < 8; ++d)
          s_acc[wave][h * MAPS + 1 - map][d0 + d] = oth[h][d];
      if (gl % LW == 0) {
        s_ml[wave][h * MAPS + map][0] = m[h];
        s_ml[wave][h * MAPS + map][1] = l[h];
      }
    }
  }
  __syncthreads();
  if constexpr (MAPS == 2) {
    // a wave per head; a lane holds columns lane, lane + 64, ..
    constexpr int NV = (DMAX + 63) / 64;
    for (int h = wave; h < nh; h += 4) {
      float o[2][NV];
#pragma unroll
      for (int mp = 0; mp < 2; ++mp) {
        const int u = h * 2 + mp;
        float mm = s_ml[0][u][0], ll = 0.f;
#pragma unroll
        for (int w = 1; w < 4; ++w) mm = fmaxf(mm, s_ml[w][u][0]);
#pragma unroll
        for (int i = 0; i < NV; ++i) o[mp][i] = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          const float c = __expf(s_ml[w][u][0] - mm);
          ll += s_ml[w][u][1] * c;
#pragma unroll
          for (int i = 0; i < NV; ++i)
            if (i * 64 + lane < a.vdim)
              o[mp][i] += s_acc[w][u][i * 64 + lane] * c;
        }
        if (a.n_split > 1) {
          const int64_t pi =
              ((int64_t(seq) * a.n_q + head0 + h) * 2 + mp) * a.n_split +
              split;
#pragma unroll
          for (int i = 0; i < NV; ++i)
            if (i * 64 + lane < a.vdim)
              a.part_acc[pi * a.vdim + i * 64 + lane] = o[mp][i];
          if (lane == 0) {
            a.part_ml[pi * 2] = mm;
            a.part_ml[pi * 2 + 1] = ll;
          }
        }
        const float inv = 1.f / ll;
#pragma unroll
        for (int i = 0; i < NV; ++i) o[mp][i] *= inv;
      }
      if (a.n_split > 1) continue;
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        o[0][i] -= a.lambda * o[1][i];
        ss += o[0][i] * o[0][i];
      }
      float post = a.out_scale / sqrtf(wave_sum(ss) / a.vdim + a.eps);
      if (a.gate)
        post /= 1.f + __expf(-act_load(
                          reinterpret_cast<const uint16_t*>(a.gate) +
                          seq * a.gate_stride + head0 + h));
      uint16_t* out = reinterpret_cast<uint16_t*>(a.out) +
                      (int64_t(seq) * a.n_q + head0 + h) * a.vdim;
#pragma unroll
      for (int i = 0; i < NV; ++i)
        if (i * 64 + lane < a.vdim)
          act_store(out + i * 64 + lane, o[0][i] * post);
    }
    return;
  }
  for (int e = threadIdx.x; e < nh * a.vdim; e += 256) {
    const int h = e / a.vdim, d = e % a.vdim;
    float mm = s_ml[0][h][0];
#pragma unroll
    for (int w = 1; w < 4; ++w) mm = fmaxf(mm, s_ml[w][h][0]);
    const bool last = a.n_split == 1;
    const float snk = (last && a.sink) ? a.sink[head0 + h] : kNegInf;
    mm = fmaxf(mm, snk);
    float o = 0.f, ll = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float c = __expf(s_ml[w][h][0] - mm);
      o += s_acc[w][h][d] * c;
      ll += s_ml[w][h][1] * c;
    }
    if (last) {
      if (a.sink) ll += __expf(snk - mm);
      reinterpret_cast<uint16_t*>(a.out)[(int64_t(seq) * a.n_q + head0 + h) *
                                             a.vdim + d] =
          f32_to_bf16(o / ll);
    } else {
      const int64_t pi =
          (int64_t(seq) * a.n_q + head0 + h) * a.n_split + split;
      a.part_acc[pi * a.vdim + d] = o;
      if (d == 0) {
        a.part_ml[pi * 2] = mm;
        a.part_ml[pi * 2 + 1] = ll;
      }
    }
  }
}

// one wave per 64 value columns; lane s holds the weight of split s
__global__ __launch_bounds__(256)
void window_combine_kernel(WindowAttnArgs a) {
  const int64_t row = blockIdx.x;               // seq * n_q + head
  const int h = int(row % a.n_q), lane = threadIdx.x & 63;
  const float snk = a.sink ? a.sink[h] : kNegInf;
  const bool mine = lane < a.n_split;
  const float2 ml = reinterpret_cast<const float2*>(
      a.part_ml)[row * a.n_split + (mine ? lane : 0)];
  const float mm = fmaxf(snk, wave_max(mine ? ml.x : kNegInf));
  const float c = mine ? __expf(ml.x - mm) : 0.f;
  const float ll = wave_sum(c * ml.y) + (a.sink ? __expf(snk - mm) : 0.f);
  for (int d = threadIdx.x; d < a.vdim; d += blockDim.x) {
    const float* p = a.part_acc + row * a.n_split * a.vdim + d;
    float o = 0.f;
#pragma unroll 4
    for (int s = 0; s < a.n_split; ++s)
      o += p[s * a.vdim] * __shfl(c, s, kWave);
    reinterpret_cast<uint16_t*>(a.out)[row * a.vdim + d] =
        f32_to_bf16(o / ll);
  }
}

// one workgroup per (sequence, head); both maps' splits, their difference,
// its norm and gate.  A thread has at most one column, vdim <= 256
__global__ __launch_bounds__(256)
void diff_combine_kernel(WindowAttnArgs a) {
  __shared__ float part[4];
  const int64_t row = blockIdx.x;               // seq * n_q + head
  const int lane = threadIdx.x & 63, d = threadIdx.x;
  const bool mine = lane < a.n_split, live = d < a.vdim;
  float o[2];
#pragma unroll
  for (int mp = 0; mp < 2; ++mp) {
    const int64_t p0 = (row * 2 + mp) * a.n_split;
    const float2 ml = reinterpret_cast<const float2*>(
        a.part_ml)[p0 + (mine ? lane : 0)];
    const float mm = wave_max(mine ? ml.x : kNegInf);
    const float c = mine ? __expf(ml.x - mm) : 0.f;
    const float ll = wave_sum(c * ml.y);
    const float* p = a.part_acc + p0 * a.vdim + (live ? d : 0);
    float t = 0.f;
#pragma unroll 4
    for (int s = 0; s < a.n_split; ++s)
      t += p[s * a.vdim] * __shfl(c, s, kWave);
    o[mp] = t / ll;
  }
  const float v = live ? o[0] - a.lambda * o[1] : 0.f;
  const float ws = wave_sum(v * v);
  if (lane == 0) part[threadIdx.x >> 6] = ws;
  __syncthreads();
  float ss = 0.f;
  for (int w = 0; w < int(blockDim.x >> 6); ++w) ss += part[w];
  float post = a.out_scale / sqrtf(ss / a.vdim + a.eps);
  if (a.gate)
    post /= 1.f + __expf(-act_load(reinterpret_cast<const uint16_t*>(a.gate) +
                                   row / a.n_q * a.gate_stride + row % a.n_q));
  if (live)
    act_store(reinterpret_cast<uint16_t*>(a.out) + row * a.vdim + d, v * post);
}

template <typename F>
void with_cache(const WindowAttnArgs& a, F f) {
  if (a.cache == kCacheFP8) f(uint16_t{}, uint8_t{});
  else if (a.f32) f(float{}, float{});
  else f(uint16_t{}, uint16_t{});
}

}  // namespace

bool window_fast_ok(const WindowAttnArgs& a) {
  return !a.f32 && a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 256 &&
         a.vdim <= 256 && a.block_size % 16 == 0;
}

int window_decode_heads_per_wg(int group) {
  return group == 1 ? 1 : group == 2 ? 2 : 4;
}

void launch_window_rope_append(const WindowAttnArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  with_cache(a, [&](auto t, auto c) {
    hipLaunchKernelGGL((rope_append_kernel<decltype(t), decltype(c)>),
                       dim3(a.rows), dim3(256), 0, st, a);
  });
}

void launch_window_rows(const WindowAttnArgs& a, bool decode,
                        hipStream_t st) {
  with_cache(a, [&](auto t, auto c) {
    run_window_rows<decltype(t), decltype(c), 8>(a, decode, st);
  });
}

namespace {

// the decode kernel of a head size, heads per workgroup and cache
template <bool BIAS, int MAPS>
void run_decode(const WindowAttnArgs& a, hipStream_t st) {
  const int group = a.n_q / a.n_kv;
  const int hb = window_decode_heads_per_wg(group);
  const dim3 grid(a.n_split, a.n_kv * ((group + hb - 1) / hb), a.rows);
  auto go = [&](auto gw, auto hbc, auto kc) {
    hipLaunchKernelGGL(
        (window_decode_kernel<decltype(gw)::value, decltype(hbc)::value,
                              decltype(kc), BIAS, MAPS>),
        grid, dim3(256), 0, st, a);
  };
  auto by_cache = [&](auto gw, auto hbc) {
    if (a.cache == kCacheFP8) go(gw, hbc, CacheFP8{});
    else go(gw, hbc, CacheBF16{});
  };
  auto by_heads = [&](auto gw) {
    if (hb == 1) by_cache(gw, std::integral_constant<int, 1>{});
    else if (hb == 2) by_cache(gw, std::integral_constant<int, 2>{});
    else by_cache(gw, std::integral_constant<int, 4>{});
  };
  const int d = std::max(MAPS * a.dim, a.vdim);
  if (d <= 32) by_heads(std::integral_constant<int, 4>{});
  else if (d <= 64) by_heads(std::integral_constant<int, 8>{});
  else if (d <= 128) by_heads(std::integral_constant<int, 16>{});
  else by_heads(std::integral_constant<int, 32>{});
}

}  // namespace

void launch_window_decode(const WindowAttnArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  if (a.r1) run_decode<true, 1>(a, st);
  else run_decode<false, 1>(a, st);
  if (a.n_split > 1)
    hipLaunchKernelGGL(window_combine_kernel, dim3(a.rows * a.n_q),
                       dim3(std::min(256, (a.vdim + 63) / 64 * 64)), 0, st,
                       a);
}

bool diff_fast_ok(const WindowAttnArgs& a) {
  return !a.f32 && a.dim % 8 == 0 && a.rot % 16 == 0 && a.vdim % 8 == 0 &&
         a.dim <= 128 && a.vdim <= 256 && a.block_size % 16 == 0;
}

void launch_diff_append(const WindowAttnArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  const int64_t units =
      int64_t(a.rows) * (a.maps * a.n_q + (a.maps + 1) * a.n_kv);
  const bool vec = a.dim % 8 == 0 && a.rot % 16 == 0 && a.vdim % 8 == 0 &&
                   a.stride % 8 == 0 && a.dim <= 256;
  with_cache(a, [&](auto t, auto c) {
    using T = decltype(t);
    using CE = decltype(c);
    auto run = [&](auto w) {
      constexpr int W = decltype(w)::value;
      hipLaunchKernelGGL((diff_append_kernel<T, CE, W>),
                         dim3(uint32_t((units * W + 255) / 256)), dim3(256),
                         0, st, a);
    };
    if (!vec)
      hipLaunchKernelGGL((diff_append_any_kernel<T, CE>),
                         dim3(a.rows, uint32_t(units / a.rows)), dim3(64),
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
  run_decode<false, 2>(a, st);
  if (a.n_split > 1)
    hipLaunchKernelGGL(diff_combine_kernel, dim3(a.rows * a.n_q),
                       dim3((a.vdim + 63) / 64 * 64), 0, st, a);
}

}  // namespace rlli
