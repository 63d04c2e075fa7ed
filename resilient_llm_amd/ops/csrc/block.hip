// Residual blocks: the residual and the (grouped) norm around it, short
// causal convolutions, gated activations, the output's soft cap.
//
// A parallel block reads h = norm(x) once, runs its mixer on h + conv(h) and its
// feed-forward on h, and adds both: their output products are one matrix
// product over the concatenated activations, so the residual is read and
// written once per block.  Writing it and norming the next block's input
// is one pass; for single decoded tokens the convolution and its state are
// in that pass too.  Residual, norms and convolution sums are 32-bit.
//
// The last inputs of a sequence sit in a ring by position, so advancing it
// writes one row and moves nothing.  A used slot needs no clearing: what a
// row reads before position 0 is zero by position.
//
// A convolution may have several branches (its own taps and output each):
// h + (h' - h) mu with the previous row's h' is the two taps mu, -mu, so
// mixing a row with the one before it for several projections is one of
// these.  A block may also end in two outputs, each with a norm of its own,
// half their sum being what the residual takes (merge), or in one per chosen
// expert (parts), where identity experts give their weight of the block's
// input.

#include "blk.h"

#include <algorithm>

namespace rlli {
namespace {

DEV_INLINE float round_act(uint16_t, float v) {
  return bf16_to_f32(f32_to_bf16(v));
}
DEV_INLINE float round_act(float, float v) { return v; }

template <typename T>
DEV_INLINE float sigm(float x) {
  return 1.f / (1.f + (sizeof(T) == 2 ? __expf(-x) : expf(-x)));
}

template <typename T, int V>
DEV_INLINE void load_v(const T* p, float (&out)[V]) {
  if constexpr (V == 4) {
    const f32x4_t v = act_load4(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) out[j] = v[j];
  } else {
    out[0] = act_load(p);
  }
}

template <typename T, int V>
DEV_INLINE void store_v(T* p, const float (&in)[V]) {
  if constexpr (V == 4) act_store4(p, f32x4_t{in[0], in[1], in[2], in[3]});
  else act_store(p, in[0]);
}

// IT vectors of V columns per thread; IT = 0 walks the row twice.  CONV:
// there are decoded rows, which also convolve
template <typename T, int WAVES, int IT, int V, bool EMBED, bool MERGE,
          bool CONV, bool PARTS>
__global__ __launch_bounds__(WAVES * 64)
void block_step_kernel(BlockArgs a) {
  extern __shared__ float sq[];           // [width / V] squares, [groups]
  constexpr int NT = WAVES * 64;
  const int n = blockIdx.x;
  const int64_t row = a.rows ? a.rows[n] : n;
  const int W = a.width, nv = W / V, gv = nv / a.groups;
  float* scale = sq + nv;
  // scalar loads that later addresses wait for come first
  const bool conv = CONV && n < a.n_decode;
  const int back = a.n_taps - 1;          // earlier inputs that count
  int pos = 0, at = 0;                    // position, its row of the ring
  T* ring = nullptr;
  if (conv) {
    pos = a.positions[n];
    if (back > 0) {
      ring = reinterpret_cast<T*>(a.tail) + int64_t(a.slots[n]) * a.ring * W;
      at = pos % a.ring;
    }
  }
  float* xr = a.x + row * W;
  const T* yr = EMBED ? nullptr
                      : reinterpret_cast<const T*>(a.y) +
                            row * (PARTS ? a.parts : 1) * W;
  // the first parts: where they come from and what they count
  constexpr int PE = PARTS ? 4 : 1;
  const T* part[PE];
  float part_w[PE];
  auto find_part = [&](int k, const T*& p, float& w) {
    const bool own = a.part_ids[row * a.parts + k] < a.part_limit;
    p = own ? yr + int64_t(k) * W
            : reinterpret_cast<const T*>(a.part_h) + row * W;
    w = own ? 1.f : a.part_w[row * a.parts + k];
  };
  if constexpr (PARTS)
#pragma unroll
    for (int k = 0; k < PE; ++k) {
      find_part(min(k, a.parts - 1), part[k], part_w[k]);
      if (k >= a.parts) part_w[k] = 0.f;
    }
  const T* y2r = MERGE ? reinterpret_cast<const T*>(a.y2) + row * W : nullptr;
  float s1 = 0.f, s2 = 0.f;               // half over the root mean squares
  auto merge = [&](int c, const float (&p)[V], const float (&q)[V],
                   float (&t)[V]) {
    float g1[V], g2[V];
    load_v<float, V>(a.gain1 + c, g1);
    load_v<float, V>(a.gain2 + c, g2);
#pragma unroll
    for (int j = 0; j < V; ++j) t[j] = p[j] * s1 * g1[j] + q[j] * s2 * g2[j];
  };
  const T *er = nullptr, *pr = nullptr;
  if constexpr (EMBED) {
    er = reinterpret_cast<const T*>(a.table) + int64_t(a.ids[n]) * W;
    if (a.pos_table)
      pr = reinterpret_cast<const T*>(a.pos_table) +
           int64_t(min(a.positions[n], a.n_positions - 1)) * W;
  }
  const bool biased = !EMBED && !MERGE && !PARTS && a.y_bias;
  auto add_bias = [&](int c, float (&t)[V]) {
    if (!biased) return;
    float b[V];
    load_v<float, V>(a.y_bias + c, b);
#pragma unroll
    for (int j = 0; j < V; ++j) t[j] += b[j];
  };
  // the two summands of a row's new value
  auto summands = [&](int c, float (&u)[V], float (&t)[V]) {
    if constexpr (EMBED) {
      load_v<T, V>(er + c, u);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] *= a.embed_scale;
      if (pr) {
        load_v<T, V>(pr + c, t);
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j) t[j] = 0.f;
      }
    } else {
      load_v<float, V>(xr + c, u);
      if constexpr (PARTS) {
        float e[PE][V];
#pragma unroll
        for (int k = 0; k < PE; ++k) load_v<T, V>(part[k] + c, e[k]);
#pragma unroll
        for (int j = 0; j < V; ++j) {
          t[j] = 0.f;
#pragma unroll
          for (int k = 0; k < PE; ++k) t[j] += part_w[k] * e[k][j];
        }
        for (int k = PE; k < a.parts; ++k) {
          const T* p;
          float w;
          find_part(k, p, w);
          load_v<T, V>(p + c, e[0]);
#pragma unroll
          for (int j = 0; j < V; ++j) t[j] += w * e[0][j];
        }
      } else {
        load_v<T, V>(yr + c, t);
        if constexpr (!MERGE && IT == 0) add_bias(c, t);
      }
      if constexpr (MERGE && IT == 0) {
        float q[V];
        load_v<T, V>(y2r + c, q);
        merge(c, t, q, t);
      }
    }
  };
  // IT > 0: everything a row needs is asked for up front, so that one
  // memory latency covers it; long convolutions and the plain walk load
  // the rest late
  constexpr int ITS = IT > 0 ? IT : 1;
  constexpr int EARLY = CONV && (IT == 1 || IT == 2) ? 4 : 0;   // taps
  float u[ITS][V], t[ITS][V], gain[ITS][V], bias[ITS][V];
  float tap[ITS][EARLY + 1][V], past[ITS][EARLY + 1][V];
  constexpr int MORE = EARLY > 0 ? 4 : 0; // further branches of two taps
  float btap[ITS][MORE + 1][2][V];
  auto every = [&](auto body) {           // over this thread's vectors
    if constexpr (IT > 0) {
#pragma unroll
      for (int i = 0; i < IT; ++i)
        if (i * NT + int(threadIdx.x) < nv) body(i * NT + threadIdx.x, i);
    } else {
      for (int v = threadIdx.x; v < nv; v += NT) body(v, 0);
    }
  };
  auto load_tap = [&](int b, int k, int c, float (&w)[V]) {
    load_v<float, V>(a.taps + (int64_t(b) * a.n_taps + back - k) * W + c, w);
  };
  float t2[MERGE ? ITS : 1][V];
  if constexpr (IT > 0) {
    every([&](int v, int i) { summands(v * V, u[i], t[i]); });
    if constexpr (MERGE)
      every([&](int v, int i) { load_v<T, V>(y2r + v * V, t2[i]); });
    every([&](int v, int i) { load_v<float, V>(a.gain + v * V, gain[i]); });
    if (biased)
      every([&](int v, int i) { load_v<float, V>(a.y_bias + v * V, bias[i]); });
    if (conv)
      every([&](int v, int i) {
#pragma unroll
        for (int k = 0; k < EARLY; ++k)
          if (k <= back) load_tap(0, k, v * V, tap[i][k]);
        if (a.n_taps == 2)
#pragma unroll
          for (int b = 0; b < MORE; ++b)
            if (b + 1 < a.branches) {
              load_tap(b + 1, 0, v * V, btap[i][b][0]);
              load_tap(b + 1, 1, v * V, btap[i][b][1]);
            }
      });
  }
  auto load_ring = [&](int k, int c, float (&e)[V]) {
    const int r = at - k < 0 ? at - k + a.ring : at - k;
    load_v<T, V>(ring + int64_t(r) * W + c, e);
  };
  if (conv)
    every([&](int v, int i) {
#pragma unroll
      for (int k = 1; k < EARLY; ++k)
        if (k <= back && k <= pos) load_ring(k, v * V, past[i][k]);
    });

  if constexpr (MERGE) {
    __shared__ float part[2][WAVES];
    every([&](int v, int i) {
      if constexpr (IT == 0) {
        load_v<T, V>(yr + v * V, t[0]);
        load_v<T, V>(y2r + v * V, t2[0]);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) {
        s1 += t[i][j] * t[i][j];
        s2 += t2[i][j] * t2[i][j];
      }
    });
    s1 = wave_sum(s1);
    s2 = wave_sum(s2);
    if ((threadIdx.x & 63) == 0) {
      part[0][threadIdx.x >> 6] = s1;
      part[1][threadIdx.x >> 6] = s2;
    }
    __syncthreads();
    s1 = s2 = 0.f;
#pragma unroll
    for (int w = 0; w < WAVES; ++w) {
      s1 += part[0][w];
      s2 += part[1][w];
    }
    s1 = 0.5f / sqrtf(s1 / W + a.eps);
    s2 = 0.5f / sqrtf(s2 / W + a.eps);
    if constexpr (IT > 0)
      every([&](int v, int i) { merge(v * V, t[i], t2[i], t[i]); });
  }
  float mine = 0.f;                       // one group: this thread's squares
  every([&](int v, int i) {
    if constexpr (IT == 0) summands(v * V, u[0], t[0]);
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      u[i][j] += t[i][j];
      if constexpr (IT > 0)
        if (biased) u[i][j] += bias[i][j];
      s += u[i][j] * u[i][j];
    }
    if (a.groups == 1) mine += s;
    else sq[v] = s;
    if constexpr (IT > 0)
      if (a.keep) store_v<float, V>(xr + v * V, u[i]);
  });
  float whole = 0.f;                      // one group: its scale
  if (a.groups == 1) {
    // sums of 16 lanes on the VALU, then four per wave through LDS
    mine = group_sum_dpp<16>(mine);
    if ((threadIdx.x & 15) == 0) sq[threadIdx.x >> 4] = mine;
    __syncthreads();
#pragma unroll
    for (int w = 0; w < WAVES * 4; ++w) whole += sq[w];
    whole = 1.f / sqrtf(whole / W + a.eps);
  } else {
    __syncthreads();
    for (int g = threadIdx.x >> 6; g < a.groups; g += WAVES) {
      float s = 0.f;
      for (int v = threadIdx.x & 63; v < gv; v += 64) s += sq[g * gv + v];
      s = wave_sum(s);
      if ((threadIdx.x & 63) == 0)
        scale[g] = 1.f / sqrtf(s / (gv * V) + a.eps);
    }
    __syncthreads();
  }
  T* hr = reinterpret_cast<T*>(a.h) + int64_t(n) * W;
  every([&](int v, int i) {
    const int c = v * V;
    if constexpr (IT == 0) {
      summands(c, u[0], t[0]);
#pragma unroll
      for (int j = 0; j < V; ++j) u[0][j] += t[0][j];
      if (a.keep) store_v<float, V>(xr + c, u[0]);
      load_v<float, V>(a.gain + c, gain[0]);
    }
    float hv[V];
    const float inv = a.groups == 1 ? whole : scale[v / gv];
#pragma unroll
    for (int j = 0; j < V; ++j)
      hv[j] = round_act(T{}, u[i][j] * inv * gain[i][j]);
    store_v<T, V>(hr + c, hv);
    if (conv) {
      int b0 = 0;
      if (MORE > 0 && a.n_taps == 2 && a.branches > 1) {
        b0 = min(a.branches, MORE + 1);
#pragma unroll
        for (int b = 0; b < MORE + 1; ++b) {
          if (b >= a.branches) break;
          float o[V];
#pragma unroll
          for (int j = 0; j < V; ++j) {
            o[j] = hv[j] + (b == 0 ? tap[i][0][j] : btap[i][b - 1][0][j]) *
                               hv[j];
            if (pos > 0)
              o[j] += (b == 0 ? tap[i][MORE > 0 ? 1 : 0][j]
                              : btap[i][b - 1][1][j]) *
                      past[i][MORE > 0 ? 1 : 0][j];
          }
          store_v<T, V>(reinterpret_cast<T*>(a.hc) +
                            (int64_t(b) * a.n + n) * W + c, o);
        }
      }
      for (int b = b0; b < a.branches; ++b) {
        float o[V];
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] = hv[j];
        auto add = [&](const float (&w)[V], const float (&e)[V]) {
#pragma unroll
          for (int j = 0; j < V; ++j) o[j] += w[j] * e[j];
        };
#pragma unroll
        for (int k = 0; k < EARLY; ++k)
          if (k <= back && k <= pos) {
            if (b > 0) load_tap(b, k, c, tap[i][k]);
            add(tap[i][k], k == 0 ? hv : past[i][k]);
          }
        for (int k = EARLY; k <= back && k <= pos; ++k) {
          float w[V], e[V];
          load_tap(b, k, c, w);
          if (k > 0) load_ring(k, c, e);
          add(w, k == 0 ? hv : e);
        }
        store_v<T, V>(reinterpret_cast<T*>(a.hc) +
                          (int64_t(b) * a.n + n) * W + c, o);
      }
      if (back > 0) store_v<T, V>(ring + int64_t(at) * W + c, hv);
    }
  });
}

// prompt rows of one span, V columns per thread, the window in registers
// (K taps; K = 0: any number, re-read).  SILU: silu(conv(h)) instead of
// h + conv(h)
template <typename T, int K, int V, bool SILU>
__global__ __launch_bounds__(256)
void conv_prompt_kernel(ConvArgs a) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= a.width) return;
  const int s = blockIdx.x, ns = a.n_spans;
  const int row0 = a.spans[s], pos0 = a.spans[ns + s];
  const int rows = a.spans[2 * ns + s], off = a.spans[3 * ns + s];
  const int taps = K > 0 ? K : a.n_taps, back = taps - 1;
  const int64_t W = a.width, HS = a.h_stride, OS = a.out_stride;
  const T* h = reinterpret_cast<const T*>(a.h) + c;
  T* out = reinterpret_cast<T*>(a.out) + blockIdx.z * a.branch_stride + c;
  const float* tap = a.taps + blockIdx.z * taps * W + c;
  const T* ring = reinterpret_cast<const T*>(a.tail) +
                  int64_t(a.spans[4 * ns + s]) * a.ring * W + c;
  auto finish = [&](float (&o)[V]) {
    if constexpr (SILU)
#pragma unroll
      for (int j = 0; j < V; ++j)
        o[j] *= sigm<T>(o[j]);
  };
  // the input at row r of the span, r may be negative
  auto input = [&](int r, float (&v)[V]) {
    if (off + r >= 0) {
      load_v<T, V>(h + int64_t(row0 + r) * HS, v);
    } else if (pos0 + r >= 0) {
      load_v<T, V>(ring + int64_t((pos0 + r) % (back > 0 ? a.ring : 1)) * W,
                   v);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
    }
  };
  if constexpr (K > 0) {
    constexpr int KB = K > 1 ? K - 1 : 1;
    float w[K][V], win[KB][V];
#pragma unroll
    for (int k = 0; k < K; ++k)
      load_v<float, V>(tap + k * W, w[k]);
#pragma unroll
    for (int k = 0; k < K - 1; ++k) input(k - (K - 1), win[k]);
#pragma unroll 4
    for (int r = 0; r < rows; ++r) {
      float cur[V], o[V];
      load_v<T, V>(h + int64_t(row0 + r) * HS, cur);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        o[j] = (SILU ? 0.f : cur[j]) + w[K - 1][j] * cur[j];
#pragma unroll
        for (int k = K - 2; k >= 0; --k) o[j] += w[k][j] * win[k][j];
      }
      finish(o);
      store_v<T, V>(out + int64_t(row0 + r) * OS, o);
#pragma unroll
      for (int k = 0; k < K - 1; ++k)
#pragma unroll
        for (int j = 0; j < V; ++j)
          win[k][j] = k + 1 < K - 1 ? win[k + 1 < KB ? k + 1 : k][j] : cur[j];
    }
  } else {
    for (int r = 0; r < rows; ++r) {
      float o[V], e[V], w[V];
      input(r, e);
      load_v<float, V>(tap + int64_t(back) * W, w);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = (SILU ? 0.f : e[j]) + w[j] * e[j];
      for (int k = 1; k <= back; ++k) {
        input(r - k, e);
        load_v<float, V>(tap + int64_t(back - k) * W, w);
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] += w[j] * e[j];
      }
      finish(o);
      store_v<T, V>(out + int64_t(row0 + r) * OS, o);
    }
  }
}

// the ring after a step: a launch of its own, because the first rows of a
// portion read what its last rows replace
template <typename T>
__global__ __launch_bounds__(256)
void conv_tail_kernel(ConvArgs a) {
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= a.width) return;
  const int s = blockIdx.x, np = a.n_portions, ring_rows = a.ring;
  const int row0 = a.portions[s], pos0 = a.portions[np + s];
  const int rows = a.portions[2 * np + s];
  const T* h = reinterpret_cast<const T*>(a.h) + c;
  T* ring = reinterpret_cast<T*>(a.tail) +
            int64_t(a.portions[4 * np + s]) * ring_rows * a.width + c;
  for (int r = max(0, rows - ring_rows); r < rows; ++r)
    ring[int64_t((pos0 + r) % ring_rows) * a.width] =
        h[int64_t(row0 + r) * a.h_stride];
}

template <int ACT, typename T>
DEV_INLINE float gated(float x, float u, float limit) {
  if constexpr (ACT == kActRelu) return fmaxf(x, 0.f) * u;
  if constexpr (ACT == kActSilu) return x * sigm<T>(x) * u;
  x = fminf(x, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return x * sigm<T>(1.702f * x) * (u + 1.f);
}

template <typename T, int ACT, int V>
__global__ __launch_bounds__(256)
void gate_act_kernel(const T* __restrict__ gu, T* __restrict__ out, int ff,
                     int64_t out_stride, int nb, float limit) {
  const int64_t row = blockIdx.x / nb;
  const int c = ((blockIdx.x % nb) * 256 + threadIdx.x) * V;
  if (c >= ff) return;
  const T* g = gu + row * 2 * ff + c;
  T* o = out + row * out_stride + c;
  constexpr int P = V >= 4 ? 4 : 1;
#pragma unroll
  for (int i = 0; i < V / P; ++i) {
    float a[P], b[P];
    load_v<T, P>(g + i * P, a);
    load_v<T, P>(g + ff + i * P, b);
#pragma unroll
    for (int j = 0; j < P; ++j) a[j] = gated<ACT, T>(a[j], b[j], limit);
    store_v<T, P>(o + i * P, a);
  }
}

template <typename T>
__global__ __launch_bounds__(256)
void soft_cap_kernel(const T* __restrict__ x, float* __restrict__ out,
                     int64_t n, float cap) {
  const int64_t i = (int64_t(blockIdx.x) * 256 + threadIdx.x) * 4;
  const float inv = 1.f / cap;
  if (i + 4 <= n) {
    f32x4_t v = act_load4(x + i);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = cap * tanhf(v[j] * inv);
    *reinterpret_cast<f32x4_t*>(out + i) = v;
  } else {
    for (int64_t k = i; k < n; ++k) out[k] = cap * tanhf(act_load(x + k) * inv);
  }
}

template <typename T, bool EMBED, bool MERGE, bool CONV, bool PARTS = false>
void step(const BlockArgs& a, hipStream_t st) {
  auto run = [&](auto* k, int threads, int v) {
    hipLaunchKernelGGL(k, dim3(a.n), dim3(threads),
                       std::max(a.width / v + a.groups, threads / 16) *
                           sizeof(float), st, a);
  };
  if (a.width / a.groups % 4 || a.width > 8192)
    run(block_step_kernel<T, 4, 0, 1, EMBED, MERGE, CONV, PARTS>, 256, 1);
  else if (a.width <= 256)
    run(block_step_kernel<T, 1, 1, 4, EMBED, MERGE, CONV, PARTS>, 64, 4);
  else if (a.width <= 1024)
    run(block_step_kernel<T, 4, 1, 4, EMBED, MERGE, CONV, PARTS>, 256, 4);
  else if (a.width <= 2048 && CONV)       // few rows: latency counts
    run(block_step_kernel<T, 8, 1, 4, EMBED, MERGE, CONV, PARTS>, 512, 4);
  else if (a.width <= 2048)
    run(block_step_kernel<T, 4, 2, 4, EMBED, MERGE, CONV, PARTS>, 256, 4);
  else if (a.width <= 4096 && CONV)
    run(block_step_kernel<T, 16, 1, 4, EMBED, MERGE, CONV, PARTS>, 1024, 4);
  else if (a.width <= 4096)
    run(block_step_kernel<T, 8, 2, 4, EMBED, MERGE, CONV, PARTS>, 512, 4);
  else
    run(block_step_kernel<T, 8, 4, 4, EMBED, MERGE, CONV, PARTS>, 512, 4);
}

template <typename T, bool EMBED>
void step(const BlockArgs& a, hipStream_t st) {
  const bool conv = a.hc && a.n_decode;
  if constexpr (!EMBED) {
    if (a.part_ids) {
      if (conv) step<T, false, false, true, true>(a, st);
      else step<T, false, false, false, true>(a, st);
      return;
    }
    if (a.y2) {
      if (conv) step<T, false, true, true>(a, st);
      else step<T, false, true, false>(a, st);
      return;
    }
  }
  if (conv) step<T, EMBED, false, true>(a, st);
  else step<T, EMBED, false, false>(a, st);
}

template <typename T, bool SILU>
void conv(const ConvArgs& a, hipStream_t st) {
  const bool vec = a.width % 4 == 0 && a.h_stride % 4 == 0 &&
                   a.out_stride % 4 == 0 &&
                   (reinterpret_cast<uintptr_t>(a.h) |
                    reinterpret_cast<uintptr_t>(a.out)) %
                           (4 * sizeof(T)) == 0;
  const int v = vec ? 4 : 1;
  const dim3 grid(a.n_spans, (a.width + 256 * v - 1) / (256 * v), a.branches);
  auto run = [&](auto* k) {
    hipLaunchKernelGGL(k, grid, dim3(256), 0, st, a);
  };
  if (v == 1) {
    run(conv_prompt_kernel<T, 0, 1, SILU>);
  } else {
    switch (a.n_taps) {
      case 1: run(conv_prompt_kernel<T, 1, 4, SILU>); break;
      case 2: run(conv_prompt_kernel<T, 2, 4, SILU>); break;
      case 3: run(conv_prompt_kernel<T, 3, 4, SILU>); break;
      case 4: run(conv_prompt_kernel<T, 4, 4, SILU>); break;
      default: run(conv_prompt_kernel<T, 0, 4, SILU>); break;
    }
  }
  if (a.n_taps > 1)
    hipLaunchKernelGGL(conv_tail_kernel<T>,
                       dim3(a.n_portions, (a.width + 255) / 256), dim3(256),
                       0, st, a);
}

template <typename T, int ACT>
void gate_act(const T* gu, T* out, int rows, int ff, int64_t stride,
              float limit, hipStream_t st) {
  const bool vec = ff % 8 == 0 && stride % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0;
  const int v = vec ? 8 : 1;
  const int nb = (ff + 256 * v - 1) / (256 * v);
  const dim3 grid(uint32_t(rows) * nb);
  if (vec)
    hipLaunchKernelGGL((gate_act_kernel<T, ACT, 8>), grid, dim3(256), 0, st,
                       gu, out, ff, stride, nb, limit);
  else
    hipLaunchKernelGGL((gate_act_kernel<T, ACT, 1>), grid, dim3(256), 0, st,
                       gu, out, ff, stride, nb, limit);
}

}  // namespace

void launch_block_step(const BlockArgs& a, hipStream_t st) {
  if (a.n == 0) return;
  if (a.f32) {
    if (a.table) step<float, true>(a, st);
    else step<float, false>(a, st);
  } else {
    if (a.table) step<uint16_t, true>(a, st);
    else step<uint16_t, false>(a, st);
  }
}

void launch_conv_prompt(const ConvArgs& a, hipStream_t st) {
  if (a.n_spans == 0) return;
  auto go = [&](auto t) {
    using T = decltype(t);
    if (a.silu) conv<T, true>(a, st);
    else conv<T, false>(a, st);
  };
  if (a.f32) go(float{});
  else go(uint16_t{});
}

void launch_gate_act(const void* gu, void* out, int rows, int ff,
                     int64_t stride, int act, float limit, bool f32,
                     hipStream_t st) {
  if (rows == 0) return;
  auto go = [&](auto* g, auto* o) {
    using T = std::remove_pointer_t<decltype(o)>;
    if (act == kActRelu)
      gate_act<T, kActRelu>(g, o, rows, ff, stride, limit, st);
    else if (act == kActSilu)
      gate_act<T, kActSilu>(g, o, rows, ff, stride, limit, st);
    else
      gate_act<T, kActClampGlu>(g, o, rows, ff, stride, limit, st);
  };
  if (f32) go(static_cast<const float*>(gu), static_cast<float*>(out));
  else go(static_cast<const uint16_t*>(gu), static_cast<uint16_t*>(out));
}

void launch_soft_cap(const void* x, float* out, int64_t n, float cap,
                     bool f32, hipStream_t st) {
  if (n == 0) return;
  const dim3 grid(uint32_t((n + 1023) / 1024));
  if (f32)
    hipLaunchKernelGGL(soft_cap_kernel<float>, grid, dim3(256), 0, st,
                       static_cast<const float*>(x), out, n, cap);
  else
    hipLaunchKernelGGL(soft_cap_kernel<uint16_t>, grid, dim3(256), 0, st,
                       static_cast<const uint16_t*>(x), out, n, cap);
}

}  // namespace rlli
