// Parallel residual block: the residual and the grouped norm around it,
// the short causal convolution ahead of a mixer, and a gated activation.
//
// A block reads h = norm(x) once, runs its mixer on h + conv(h) and its
// feed-forward on h, and adds both: their output products are one matrix
// product over the concatenated activations, so the residual is read and
// written once per block.  Writing it and norming the next block's input
// is one pass; for single decoded tokens the convolution and its state are
// in that pass too.  Residual, norms and convolution sums are 32-bit.
//
// The last n_taps - 1 inputs of a sequence sit in a ring by position, so
// advancing it writes one row and moves nothing.  A used slot needs no
// clearing: what a row reads before position 0 is zero by position.

#include "lat.h"

namespace rlli {
namespace {

DEV_INLINE float round_act(uint16_t, float v) {
  return bf16_to_f32(f32_to_bf16(v));
}
DEV_INLINE float round_act(float, float v) { return v; }

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
template <typename T, int WAVES, int IT, int V, bool EMBED, bool CONV>
__global__ __launch_bounds__(WAVES * 64)
void block_step_kernel(BlockArgs a) {
  extern __shared__ float sq[];           // [width / V] squares, [groups]
  constexpr int NT = WAVES * 64;
  const int n = blockIdx.x;
  const int64_t row = a.rows ? a.rows[n] : n;
  const int W = a.width, nv = W / V, gv = nv / a.groups;
  float* scale = sq + nv;
  float* xr = a.x + row * W;
  const T* yr = EMBED ? nullptr
                      : reinterpret_cast<const T*>(a.y) + row * W;
  const T *er = nullptr, *pr = nullptr;
  if constexpr (EMBED) {
    er = reinterpret_cast<const T*>(a.table) + int64_t(a.ids[n]) * W;
    if (a.pos_table)
      pr = reinterpret_cast<const T*>(a.pos_table) +
           int64_t(min(a.positions[n], a.n_positions - 1)) * W;
  }
  // the two summands of a row's new value
  auto summands = [&](int c, float (&u)[V], float (&t)[V]) {
    if constexpr (EMBED) {
      load_v<T, V>(er + c, u);
      if (pr) {
        load_v<T, V>(pr + c, t);
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j) t[j] = 0.f;
      }
    } else {
      load_v<float, V>(xr + c, u);
      load_v<T, V>(yr + c, t);
    }
  };
  // IT > 0: everything a row needs is asked for up front, so that one
  // memory latency covers it; long convolutions and the plain walk load
  // the rest late
  constexpr int ITS = IT > 0 ? IT : 1;
  constexpr int EARLY = CONV && (IT == 1 || IT == 2) ? 4 : 0;   // taps
  float u[ITS][V], t[ITS][V], gain[ITS][V];
  float tap[ITS][EARLY + 1][V], past[ITS][EARLY + 1][V];
  auto every = [&](auto body) {           // over this thread's vectors
    if constexpr (IT > 0) {
#pragma unroll
      for (int i = 0; i < IT; ++i)
        if (i * NT + int(threadIdx.x) < nv) body(i * NT + threadIdx.x, i);
    } else {
      for (int v = threadIdx.x; v < nv; v += NT) body(v, 0);
    }
  };
  const bool conv = CONV && n < a.n_decode;
  const int back = a.n_taps - 1;          // earlier inputs in the ring
  auto load_tap = [&](int k, int c, float (&w)[V]) {
    load_v<float, V>(a.taps + int64_t(back - k) * W + c, w);
  };
  if constexpr (IT > 0) {
    every([&](int v, int i) { summands(v * V, u[i], t[i]); });
    every([&](int v, int i) { load_v<float, V>(a.gain + v * V, gain[i]); });
    if (conv)
      every([&](int v, int i) {
#pragma unroll
        for (int k = 0; k < EARLY; ++k)
          if (k <= back) load_tap(k, v * V, tap[i][k]);
      });
  }
  int pos = 0, at = 0;                    // position, its row of the ring
  T* ring = nullptr;
  if (conv) {
    pos = a.positions[n];
    if (back > 0) {
      ring = reinterpret_cast<T*>(a.tail) + int64_t(a.slots[n]) * back * W;
      at = pos % back;
    }
  }
  auto load_ring = [&](int k, int c, float (&e)[V]) {
    const int r = at - k < 0 ? at - k + back : at - k;
    load_v<T, V>(ring + int64_t(r) * W + c, e);
  };
  if (conv)
    every([&](int v, int i) {
#pragma unroll
      for (int k = 1; k < EARLY; ++k)
        if (k <= back && k <= pos) load_ring(k, v * V, past[i][k]);
    });

  every([&](int v, int i) {
    if constexpr (IT == 0) summands(v * V, u[0], t[0]);
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) {
      u[i][j] += t[i][j];
      s += u[i][j] * u[i][j];
    }
    sq[v] = s;
    if constexpr (IT > 0)
      if (a.keep) store_v<float, V>(xr + v * V, u[i]);
  });
  __syncthreads();
  for (int g = threadIdx.x >> 6; g < a.groups; g += WAVES) {
    float s = 0.f;
    for (int v = threadIdx.x & 63; v < gv; v += 64) s += sq[g * gv + v];
    s = wave_sum(s);
    if ((threadIdx.x & 63) == 0)
      scale[g] = 1.f / sqrtf(s / (gv * V) + a.eps);
  }
  __syncthreads();
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
    const float inv = scale[v / gv];
#pragma unroll
    for (int j = 0; j < V; ++j)
      hv[j] = round_act(T{}, u[i][j] * inv * gain[i][j]);
    store_v<T, V>(hr + c, hv);
    if (conv) {
      float o[V];
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = hv[j];
      auto add = [&](const float (&w)[V], const float (&e)[V]) {
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] += w[j] * e[j];
      };
#pragma unroll
      for (int k = 0; k < EARLY; ++k)
        if (k <= back && k <= pos) add(tap[i][k], k == 0 ? hv : past[i][k]);
      for (int k = EARLY; k <= back && k <= pos; ++k) {
        float w[V], e[V];
        load_tap(k, c, w);
        if (k > 0) load_ring(k, c, e);
        add(w, k == 0 ? hv : e);
      }
      store_v<T, V>(reinterpret_cast<T*>(a.hc) + int64_t(n) * W + c, o);
      if (back > 0) store_v<T, V>(ring + int64_t(at) * W + c, hv);
    }
  });
}

// prompt rows of one span, V columns per thread, the window in registers
// (K taps; K = 0: any number, re-read)
template <typename T, int K, int V>
__global__ __launch_bounds__(256)
void conv_prompt_kernel(ConvArgs a) {
  const int c = (blockIdx.y * 256 + threadIdx.x) * V;
  if (c >= a.width) return;
  const int s = blockIdx.x, ns = a.n_spans;
  const int row0 = a.spans[s], pos0 = a.spans[ns + s];
  const int rows = a.spans[2 * ns + s], off = a.spans[3 * ns + s];
  const int taps = K > 0 ? K : a.n_taps, back = taps - 1;
  const int64_t W = a.width;
  const T* h = reinterpret_cast<const T*>(a.h) + c;
  T* out = reinterpret_cast<T*>(a.out) + c;
  const T* ring = reinterpret_cast<const T*>(a.tail) +
                  int64_t(a.spans[4 * ns + s]) * back * W + c;
  // the input at row r of the span, r may be negative
  auto input = [&](int r, float (&v)[V]) {
    if (off + r >= 0) {
      load_v<T, V>(h + int64_t(row0 + r) * W, v);
    } else if (pos0 + r >= 0) {
      load_v<T, V>(ring + int64_t((pos0 + r) % (back > 0 ? back : 1)) * W, v);
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
      load_v<float, V>(a.taps + k * W + c, w[k]);
#pragma unroll
    for (int k = 0; k < K - 1; ++k) input(k - (K - 1), win[k]);
#pragma unroll 4
    for (int r = 0; r < rows; ++r) {
      float cur[V], o[V];
      load_v<T, V>(h + int64_t(row0 + r) * W, cur);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        o[j] = cur[j] + w[K - 1][j] * cur[j];
#pragma unroll
        for (int k = K - 2; k >= 0; --k) o[j] += w[k][j] * win[k][j];
      }
      store_v<T, V>(out + int64_t(row0 + r) * W, o);
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
      load_v<float, V>(a.taps + int64_t(back) * W + c, w);
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = e[j] + w[j] * e[j];
      for (int k = 1; k <= back; ++k) {
        input(r - k, e);
        load_v<float, V>(a.taps + int64_t(back - k) * W + c, w);
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] += w[j] * e[j];
      }
      store_v<T, V>(out + int64_t(row0 + r) * W, o);
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
  const int s = blockIdx.x, np = a.n_portions, back = a.n_taps - 1;
  const int row0 = a.portions[s], pos0 = a.portions[np + s];
  const int rows = a.portions[2 * np + s];
  const T* h = reinterpret_cast<const T*>(a.h) + c;
  T* ring = reinterpret_cast<T*>(a.tail) +
            int64_t(a.portions[4 * np + s]) * back * a.width + c;
  for (int r = max(0, rows - back); r < rows; ++r)
    ring[int64_t((pos0 + r) % back) * a.width] =
        h[int64_t(row0 + r) * a.width];
}

template <int ACT>
DEV_INLINE float activate(float x) {
  if constexpr (ACT == kActRelu) return fmaxf(x, 0.f);
  return x / (1.f + __expf(-x));
}

template <typename T, int ACT, int V>
__global__ __launch_bounds__(256)
void gate_act_kernel(const T* __restrict__ gu, T* __restrict__ out, int ff,
                     int64_t out_stride, int nb) {
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
    for (int j = 0; j < P; ++j) a[j] = activate<ACT>(a[j]) * b[j];
    store_v<T, P>(o + i * P, a);
  }
}

template <typename T, bool EMBED, bool CONV>
void step(const BlockArgs& a, hipStream_t st) {
  auto run = [&](auto* k, int threads, int v) {
    hipLaunchKernelGGL(k, dim3(a.n), dim3(threads),
                       (a.width / v + a.groups) * sizeof(float), st, a);
  };
  if (a.width / a.groups % 4 || a.width > 8192)
    run(block_step_kernel<T, 4, 0, 1, EMBED, CONV>, 256, 1);
  else if (a.width <= 256)
    run(block_step_kernel<T, 1, 1, 4, EMBED, CONV>, 64, 4);
  else if (a.width <= 1024)
    run(block_step_kernel<T, 4, 1, 4, EMBED, CONV>, 256, 4);
  else if (a.width <= 2048)
    run(block_step_kernel<T, 4, 2, 4, EMBED, CONV>, 256, 4);
  else if (a.width <= 4096)
    run(block_step_kernel<T, 8, 2, 4, EMBED, CONV>, 512, 4);
  else
    run(block_step_kernel<T, 8, 4, 4, EMBED, CONV>, 512, 4);
}

template <typename T, bool EMBED>
void step(const BlockArgs& a, hipStream_t st) {
  if (a.hc && a.n_decode) step<T, EMBED, true>(a, st);
  else step<T, EMBED, false>(a, st);
}

template <typename T>
void conv(const ConvArgs& a, hipStream_t st) {
  const int v = a.width % 4 ? 1 : 4;
  const dim3 grid(a.n_spans, (a.width + 256 * v - 1) / (256 * v));
  auto run = [&](auto* k) {
    hipLaunchKernelGGL(k, grid, dim3(256), 0, st, a);
  };
  if (v == 1) {
    run(conv_prompt_kernel<T, 0, 1>);
  } else {
    switch (a.n_taps) {
      case 1: run(conv_prompt_kernel<T, 1, 4>); break;
      case 2: run(conv_prompt_kernel<T, 2, 4>); break;
      case 3: run(conv_prompt_kernel<T, 3, 4>); break;
      case 4: run(conv_prompt_kernel<T, 4, 4>); break;
      default: run(conv_prompt_kernel<T, 0, 4>); break;
    }
  }
  if (a.n_taps > 1)
    hipLaunchKernelGGL(conv_tail_kernel<T>,
                       dim3(a.n_portions, (a.width + 255) / 256), dim3(256),
                       0, st, a);
}

template <typename T, int ACT>
void gate_act(const T* gu, T* out, int rows, int ff, int64_t stride,
              hipStream_t st) {
  const bool vec = ff % 8 == 0 && stride % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(out) % 16 == 0;
  const int v = vec ? 8 : 1;
  const int nb = (ff + 256 * v - 1) / (256 * v);
  const dim3 grid(uint32_t(rows) * nb);
  if (vec)
    hipLaunchKernelGGL((gate_act_kernel<T, ACT, 8>), grid, dim3(256), 0, st,
                       gu, out, ff, stride, nb);
  else
    hipLaunchKernelGGL((gate_act_kernel<T, ACT, 1>), grid, dim3(256), 0, st,
                       gu, out, ff, stride, nb);
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
  if (a.f32) conv<float>(a, st);
  else conv<uint16_t>(a, st);
}

void launch_gate_act(const void* gu, void* out, int rows, int ff,
                     int64_t stride, int act, bool f32, hipStream_t st) {
  if (rows == 0) return;
  auto go = [&](auto* g, auto* o) {
    using T = std::remove_pointer_t<decltype(o)>;
    if (act == kActRelu) gate_act<T, kActRelu>(g, o, rows, ff, stride, st);
    else gate_act<T, kActSilu>(g, o, rows, ff, stride, st);
  };
  if (f32) go(static_cast<const float*>(gu), static_cast<float*>(out));
  else go(static_cast<const uint16_t*>(gu), static_cast<uint16_t*>(out));
}

}  // namespace rlli
