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
// Kernels here:
//   window_rope_append  rotate q in place, rotate and cache k, cache v
//   window_decode       one new token per sequence, split over the
//                       visible cache blocks; rotation and append fused
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

// ---- decode: one new token per sequence -------------------------------
// Workgroup = (sequence, kv head, HB query heads, split).  A wave splits
// into 64/GW lane groups of GW lanes; a lane owns 8 dimensions, a group
// walks TPG of the 16 tokens of a step, waves and splits interleave over
// the visible steps.  The new token's own term never touches the cache:
// group 0 of wave 0 of split 0 folds it in from registers while it
// appends, so no wave waits on a cache write of this launch.
template <int GW, int HB, typename KC, bool BIAS>
__global__ __launch_bounds__(256)
void window_decode_kernel(WindowAttnArgs a) {
  constexpr int GPW = 64 / GW;
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
  const int d0 = gl * 8;
  const bool kd = d0 < a.dim, vd = d0 < a.vdim;
  const int pos = a.positions[seq];
  const int head0 = kvh * group + hb0;

  const uint16_t* qrow =
      reinterpret_cast<const uint16_t*>(a.qkv) + int64_t(seq) * a.stride;
  const float* cs = a.cos_sin + int64_t(pos) * a.rot;
  const int half = a.rot / 2;

  // in-lane rotation: a lane's 8 dims are 4 whole pairs
  float rc[4], rs[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int p = d0 / 2 + i;
    rc[i] = p < half ? cs[p] : 1.f;
    rs[i] = p < half ? cs[half + p] : 0.f;
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
  float qv[HB][8], m[HB], l[HB], acc[HB][8];
#pragma unroll
  for (int h = 0; h < HB; ++h) {
    load8_rot(qrow + (head0 + h) * a.dim + d0, kd && h < nh, qv[h]);
    // the prompt path rounds rotated queries to bf16 for its matrix
    // cores; round here too so both paths score the same values
#pragma unroll
    for (int i = 0; i < 8; ++i) qv[h][i] = bf16_to_f32(f32_to_bf16(qv[h][i]));
    m[h] = kNegInf;
    l[h] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[h][i] = 0.f;
  }

  auto gsum = [&](float v) {
    if constexpr (GW <= 16) return group_sum_dpp<GW>(v);
    v = group_sum_dpp<16>(v);
    return v + __shfl_xor(v, 16, kWave);
  };

  elem* kc = reinterpret_cast<elem*>(a.k_cache);
  elem* vc = reinterpret_cast<elem*>(a.v_cache);
  int len = pos + 1;                            // cached tokens to walk
  if (a.has_kv) {
    len = pos;
    if (wave == 0 && grp == 0 && split == 0) {
      float kf[8], vf[8];
      const uint16_t* kr = qrow + a.n_q * a.dim + kvh * a.dim + d0;
      load8_rot(kr, kd, kf);
      bf16x8 vr;
      vr.u = uint4{0, 0, 0, 0};
      if (vd)
        vr.u = *reinterpret_cast<const uint4*>(
            qrow + (a.n_q + a.n_kv) * a.dim + kvh * a.vdim + d0);
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
      const vec8 kw = KC::from_f32(kf);
      const vec8 vw = KC::from_f32(vf);
      if (hb0 == 0) {
        if (kd) *reinterpret_cast<vec8*>(kc + rowi * a.dim + d0) = kw;
        if (vd) *reinterpret_cast<vec8*>(vc + rowi * a.vdim + d0) = vw;
      }
      KC::to_f32(kw, kf);
      KC::to_f32(vw, vf);
#pragma unroll
      for (int h = 0; h < HB; ++h) {
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) s += qv[h][i] * kf[i];
        m[h] = gsum(s) * scale;
        l[h] = 1.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[h][i] = vf[i];
      }
    }
  }

  // visible 16-token steps: those of the kept tokens, then the window's
  const int lo = max(0, pos - a.window + 1);
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
          kc + (base + tok) * a.dim + d0);
      if (vd) vr[i] = *reinterpret_cast<const vec8*>(
          vc + (base + tok) * a.vdim + d0);
    }
  };
  auto consume = [&](int b, const vec8 (&kr)[TPG], const vec8 (&vr)[TPG]) {
    float vf[TPG][8], sv[HB][TPG];
#pragma unroll
    for (int i = 0; i < TPG; ++i) {
      const int j = b * 16 + grp + GPW * i;
      const bool ok = j < len && (pos - j < a.window || j < a.keep_first);
      float kf[8];
      KC::to_f32(kr[i], kf);
      KC::to_f32(vr[i], vf[i]);
#pragma unroll
      for (int h = 0; h < HB; ++h) {
        float s = 0.f;
#pragma unroll
        for (int d = 0; d < 8; ++d) s += qv[h][d] * kf[d];
        s = gsum(s) * scale;
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
    }
  }
  __shared__ float s_acc[4][HB][DMAX];
  __shared__ float s_ml[4][HB][2];
  if (grp == 0) {
#pragma unroll
    for (int h = 0; h < HB; ++h) {
#pragma unroll
      for (int d = 0; d < 8; ++d) s_acc[wave][h][d0 + d] = acc[h][d];
      if (gl == 0) {
        s_ml[wave][h][0] = m[h];
        s_ml[wave][h][1] = l[h];
      }
    }
  }
  __syncthreads();
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

void launch_window_decode(const WindowAttnArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  const int group = a.n_q / a.n_kv;
  const int hb = window_decode_heads_per_wg(group);
  const dim3 grid(a.n_split, a.n_kv * ((group + hb - 1) / hb), a.rows);
  auto go = [&](auto gw, auto hbc, auto kc) {
    if (a.r1)
      hipLaunchKernelGGL(
          (window_decode_kernel<decltype(gw)::value, decltype(hbc)::value,
                                decltype(kc), true>),
          grid, dim3(256), 0, st, a);
    else
      hipLaunchKernelGGL(
          (window_decode_kernel<decltype(gw)::value, decltype(hbc)::value,
                                decltype(kc), false>),
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
  const int d = a.dim > a.vdim ? a.dim : a.vdim;
  if (d <= 32) by_heads(std::integral_constant<int, 4>{});
  else if (d <= 64) by_heads(std::integral_constant<int, 8>{});
  else if (d <= 128) by_heads(std::integral_constant<int, 16>{});
  else by_heads(std::integral_constant<int, 32>{});
  if (a.n_split > 1)
    hipLaunchKernelGGL(window_combine_kernel, dim3(a.rows * a.n_q),
                       dim3(std::min(256, (a.vdim + 63) / 64 * 64)), 0, st,
                       a);
}

}  // namespace rlli
