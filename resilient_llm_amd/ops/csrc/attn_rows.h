// Paged attention (window or chunk, kept tokens, sink, distance bias, query
// temperature, capped scores, one map or two) at any sizes and dtypes, one
// wave per (row, head), scalar everywhere: the 32-bit path, and the shapes
// that the tiled kernels do not take.  Keys and values may be one tensor (a
// cached latent that serves as both).
#pragma once

#include "attn.h"

namespace rlli {
namespace {

constexpr float kNegInf = -1e30f;

// Rows come from decode batches (one row per sequence, block table row =
// row index) or from tiles of prompt rows.
// MAXV bounds the value width: vdim <= 64 * MAXV
template <typename T, typename CE, int MAXV, int MAPS = 1>
__global__ __launch_bounds__(64)
void window_rows_kernel(WindowAttnArgs a, bool decode) {
  extern __shared__ float qs[];
  const int lane = threadIdx.x;
  const int h = blockIdx.y;
  int row, pos, seq;
  if (decode) {
    row = blockIdx.x;
    seq = row;
    pos = a.positions[row];
  } else {
    const int tile = blockIdx.x / a.tile_rows;
    const int r = blockIdx.x % a.tile_rows;
    if (r >= a.tiles[2 * a.n_tiles + tile]) return;
    row = a.tiles[tile] + r;
    pos = a.tiles[a.n_tiles + tile] + r;
    seq = a.tiles[3 * a.n_tiles + tile];
  }
  const int kvh = h / (a.n_q / a.n_kv);
  const int kw = MAPS * a.dim;
  const T* q = reinterpret_cast<const T*>(a.qkv) + int64_t(row) * a.stride +
               h * kw;
  for (int d = lane; d < kw; d += 64) qs[d] = act_load(q + d);
  __syncthreads();
  const int32_t* bt = a.block_tables + int64_t(seq) * a.max_blocks;
  const CE* kc = reinterpret_cast<const CE*>(a.k_cache);
  const CE* vc = reinterpret_cast<const CE*>(a.v_cache);

  const float scale = a.scale * query_temp(pos, a.temp_coef, a.temp_every);
  const float r1 = a.r1 ? a.r1[h] : 0.f, r2 = a.r1 ? a.r2[h] : 0.f;
  const int lo = first_seen(a, pos);
  const int kept = min(a.keep_first, lo);
  // visible keys as one list: kept tokens, then the window
  const int n_vis = kept + (pos - lo + 1);
  float first[MAXV];                      // the first map's output
#pragma unroll
  for (int map = 0; map < MAPS; ++map) {
    float m = kNegInf, l = 0.f, acc[MAXV];
#pragma unroll
    for (int i = 0; i < MAXV; ++i) acc[i] = 0.f;
    for (int base = 0; base < n_vis; base += 64) {
      const int idx = base + lane;
      const int j = idx < kept ? idx : lo + (idx - kept);
      float s = kNegInf;
      int64_t vrow = 0;
      if (idx < n_vis) {
        const int64_t blk = bt[j / a.block_size];
        const int64_t rowi =
            (blk * a.n_kv + kvh) * a.block_size + j % a.block_size;
        const CE* kr = kc + rowi * kw + map * a.dim;
        const float* qm = qs + map * a.dim;
        float dot = 0.f;
        for (int d = 0; d < a.dim; ++d) dot += qm[d] * cache_load(kr + d);
        s = dot * scale;
        if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
        if (a.r1) s -= r1 * logf(1.f + r2 * float(pos - j));
        vrow = rowi * a.vdim;
      }
      const float m_new = fmaxf(m, wave_max(s));
      const float corr = expf(m - m_new);
      const float p = idx < n_vis ? expf(s - m_new) : 0.f;
      l = l * corr + wave_sum(p);
      m = m_new;
#pragma unroll
      for (int i = 0; i < MAXV; ++i) acc[i] *= corr;
      const int cnt = min(64, n_vis - base);
      for (int t = 0; t < cnt; ++t) {
        const float pt = __shfl(p, t, kWave);
        const int vlo = __shfl(int(vrow & 0xffffffff), t, kWave);
        const int vhi = __shfl(int(vrow >> 32), t, kWave);
        const CE* vr = vc + ((int64_t(vhi) << 32) | uint32_t(vlo));
#pragma unroll
        for (int i = 0; i < MAXV; ++i) {
          const int d = i * 64 + lane;
          if (d < a.vdim) acc[i] += pt * cache_load(vr + d);
        }
      }
    }
    if (a.sink) {
      const float m_new = fmaxf(m, a.sink[h]);
      const float corr = expf(m - m_new);
      l = l * corr + expf(a.sink[h] - m_new);
#pragma unroll
      for (int i = 0; i < MAXV; ++i) acc[i] *= corr;
    }
    T* out = reinterpret_cast<T*>(a.out) +
             (int64_t(row) * a.n_q + h) * a.vdim;
    if (map + 1 < MAPS) {
#pragma unroll
      for (int i = 0; i < MAXV; ++i) first[i] = acc[i] / l;
      continue;
    }
    float post = 1.f;
    if constexpr (MAPS == 2) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < MAXV; ++i) {
        acc[i] = first[i] - a.lambda * (acc[i] / l);
        if (i * 64 + lane < a.vdim) ss += acc[i] * acc[i];
      }
      l = 1.f;
      post = a.out_scale / sqrtf(wave_sum(ss) / a.vdim + a.eps);
      if (a.gate)
        post /= 1.f + expf(-act_load(reinterpret_cast<const T*>(a.gate) +
                                     row * a.gate_stride + h));
    }
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int d = i * 64 + lane;
      if (d < a.vdim)
        act_store(out + d, MAPS == 2 ? acc[i] * post : acc[i] / l);
    }
  }
}

template <typename T, typename CE, int MAXV, int MAPS = 1>
void run_window_rows(const WindowAttnArgs& a, bool decode, hipStream_t st) {
  const int n = decode ? a.rows : a.n_tiles * a.tile_rows;
  if (n == 0) return;
  hipLaunchKernelGGL((window_rows_kernel<T, CE, MAXV, MAPS>),
                     dim3(n, a.n_q), dim3(64), MAPS * a.dim * sizeof(float),
                     st, a, decode);
}

}  // namespace
}  // namespace rlli
