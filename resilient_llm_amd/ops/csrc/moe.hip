// Mixture of experts, two kinds.  Gated: the routing weight (a sigmoid)
// multiplies the expert's INPUT, y = sum over the chosen experts of
// expert(w * h), clamped swish-like gate.  Squared relu: y = sum of
// w expert(h), weights a softmax over all routes, scaled to sum to one over
// the chosen; a correction may shift the choice, routes may be chosen by
// groups, and the last routes may be identity experts (w h), which run
// nothing here: whoever sums a token's outputs adds them.
//
//   moe_route     router logits (f32 accumulation over the activation's
//                 own values), scores, top-k
//   moe_plan      (token, choice) pairs in expert order + row tiles; one
//                 workgroup for decode-sized batches, three small grids
//                 for prompts; no host round trip, so it is capturable
//   moe_experts   two grouped GEMMs.  Up: w * (W h) is scaled in the
//                 accumulator, gated in registers (gate and up rows are
//                 packed in alternating blocks of 16) and leaves as one
//                 [pairs, ff] tensor; or w relu(W h)^2, which the down
//                 product carries through.  Down: scatters every pair's row to
//                 [token, choice]; the sum over choices happens in the
//                 residual kernel that reads it anyway.
// Small row counts stream the weights straight into MFMA fragments, K
// split over the waves; large ones run 128 x 128 tiles through LDS.

#include "mix.h"

namespace rlli {
namespace {

// ------------------------------------------------------------- router
// Wave-wide reductions on the VALU, the result in every lane: rows of 16,
// then across rows, then out of the last lane.
template <int CTRL>
DEV_INLINE float dpp_or_own(float v) {
  const int b = __builtin_bit_cast(int, v);
  return __builtin_bit_cast(
      float, __builtin_amdgcn_update_dpp(b, b, CTRL, 0xf, 0xf, false));
}
DEV_INLINE float last_lane(float v) {
  return __builtin_bit_cast(
      float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), 63));
}
DEV_INLINE float wave_sum_dpp(float v) {
  v = group_sum_dpp<16>(v);
  // rows 0 + 1 | 2 + 3, then all four, in the last lane
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
           0, __builtin_bit_cast(int, v), 0x142, 0xa, 0xf, false));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(
           0, __builtin_bit_cast(int, v), 0x143, 0xc, 0xf, false));
  return last_lane(v);
}
DEV_INLINE float wave_max_dpp(float v) {
  v = fmaxf(v, dpp_or_own<0x111>(v));     // row_shr 1, 2, 4, 8
  v = fmaxf(v, dpp_or_own<0x112>(v));
  v = fmaxf(v, dpp_or_own<0x114>(v));
  v = fmaxf(v, dpp_or_own<0x118>(v));
  v = fmaxf(v, dpp_or_own<0x142>(v));     // row_bcast 15, 31
  v = fmaxf(v, dpp_or_own<0x143>(v));
  return last_lane(v);
}

// 16 rows per workgroup, K split over eight waves
template <typename T, int ET>
__global__ __launch_bounds__(512)
void moe_route_kernel(MoeArgs a) {
  constexpr int E16 = ET * 16, NW = 8;
  __shared__ float part[NW][16][E16 + 1];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int row0 = blockIdx.x * 16;
  const T* h = reinterpret_cast<const T*>(a.h) +
               int64_t(min(row0 + lr, a.rows - 1)) * a.width;
  const T* wr = reinterpret_cast<const T*>(a.router);
  const T* wp[ET];
  f32x4_t acc[ET];
#pragma unroll
  for (int e = 0; e < ET; ++e) {
    // columns past the last route repeat it; nobody reads them
    wp[e] = wr + int64_t(min(e * 16 + lr, a.routes - 1)) * a.width;
    acc[e] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  }
  constexpr int U = ET <= 4 ? 4 : 1;      // k steps with loads in flight
  int k0 = w * 32;
  for (; k0 + (U - 1) * NW * 32 + 32 <= a.width; k0 += U * NW * 32) {
    Frag8<T> fa[U], fb[U][ET];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * NW * 32 + g * 8;
      fa[u].load(h + k);
#pragma unroll
      for (int e = 0; e < ET; ++e) fb[u][e].load(wp[e] + k);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int e = 0; e < ET; ++e)
        acc[e] = Frag8<T>::mma(fa[u], fb[u][e], acc[e]);
  }
  for (; k0 < a.width; k0 += NW * 32) {
    const int k = k0 + g * 8;
    Frag8<T> fa;
    fa.zero();
    if (k < a.width) fa.load(h + k);
#pragma unroll
    for (int e = 0; e < ET; ++e) {
      Frag8<T> fb;
      fb.zero();
      if (k < a.width) fb.load(wp[e] + k);
      acc[e] = Frag8<T>::mma(fa, fb, acc[e]);
    }
  }
#pragma unroll
  for (int e = 0; e < ET; ++e)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      part[w][g * 4 + r][e * 16 + lr] = acc[e][r];
  __syncthreads();
  // each wave ranks two rows, lane l holding routes l, l + 64, ...
  constexpr int EL = (E16 + 63) / 64;
  constexpr float kNone = -INFINITY;      // cannot be chosen
  auto wave_fence = [] {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  };
  for (int t = w * 2; t < w * 2 + 2; ++t) {
    const int row = row0 + t;
    if (row >= a.rows) break;
    float s[EL], choice[EL];
#pragma unroll
    for (int i = 0; i < EL; ++i) {
      const int e = i * 64 + lane;
      s[i] = kNone;
      if (e < a.routes) {
        s[i] = 0.f;
#pragma unroll
        for (int p = 0; p < NW; ++p) s[i] += part[p][t][e];
      }
    }
    if (a.softmax) {
      float mx = kNone, sum = 0.f;
#pragma unroll
      for (int i = 0; i < EL; ++i) mx = fmaxf(mx, s[i]);
      mx = wave_max_dpp(mx);
#pragma unroll
      for (int i = 0; i < EL; ++i) {
        s[i] = expf(s[i] - mx);           // 0 past the last route
        sum += s[i];
      }
      sum = wave_sum_dpp(sum);
#pragma unroll
      for (int i = 0; i < EL; ++i) s[i] /= sum;
    } else {
#pragma unroll
      for (int i = 0; i < EL; ++i) s[i] = 1.f / (1.f + expf(-s[i]));
    }
#pragma unroll
    for (int i = 0; i < EL; ++i) {
      const int e = i * 64 + lane;
      choice[i] = kNone;
      if (e < a.routes)
        choice[i] = s[i] + (a.correction ? a.correction[e] : 0.f);
    }
    if (a.keep < a.groups) {
      // this row's part sums are read; their place holds the choice scores,
      // the groups' best ones, and which groups stay
      float *cs = part[0][t], *best = part[1][t], *stays = part[2][t];
      const int size = a.routes / a.groups;
      wave_fence();
#pragma unroll
      for (int i = 0; i < EL; ++i)
        if (i * 64 + lane < a.routes) cs[i * 64 + lane] = choice[i];
      wave_fence();
      for (int g = lane; g < a.groups; g += 64) {
        float b = kNone;
        for (int e = g * size; e < (g + 1) * size; ++e) b = fmaxf(b, cs[e]);
        best[g] = b;
      }
      wave_fence();
      for (int g = lane; g < a.groups; g += 64) {
        int ahead = 0;
        for (int o = 0; o < a.groups; ++o)
          ahead += best[o] > best[g] || (best[o] == best[g] && o < g);
        stays[g] = ahead < a.keep ? 1.f : 0.f;
      }
      wave_fence();
#pragma unroll
      for (int i = 0; i < EL; ++i) {
        const int e = i * 64 + lane;
        if (e < a.routes && stays[e / size] == 0.f) choice[i] = kNone;
      }
    }
    float won[EL], total = 0.f;           // lane c & 63 keeps weight c
    for (int c = 0; c < a.top; ++c) {
      // the best score left, and the first route that has it
      float bv = choice[0];
#pragma unroll
      for (int i = 1; i < EL; ++i) bv = fmaxf(bv, choice[i]);
      bv = wave_max_dpp(bv);
      int bi = 0x7fffffff;
#pragma unroll
      for (int i = EL - 1; i >= 0; --i) {
        const uint64_t has = __ballot(choice[i] == bv);
        if (has) bi = i * 64 + __builtin_ctzll(has);
      }
#pragma unroll
      for (int i = 0; i < EL; ++i)
        if (i * 64 + lane == bi) choice[i] = kNone;
      bi = min(bi, a.routes - 1);       // a NaN row still names a route
      float mine = s[0];
#pragma unroll
      for (int i = 1; i < EL; ++i)
        if (bi >> 6 == i) mine = s[i];
      mine = __builtin_bit_cast(
          float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, mine),
                                           bi & 63));
      total += mine;
#pragma unroll
      for (int i = 0; i < EL; ++i)
        if (c == i * 64 + lane) won[i] = mine;
      if (lane == 0) a.ids[int64_t(row) * a.top + c] = bi;
    }
    const float scale = a.softmax ? 1.f / (total + 1e-20f) : 1.f;
#pragma unroll
    for (int i = 0; i < EL; ++i)
      if (i * 64 + lane < a.top)
        a.weights[int64_t(row) * a.top + i * 64 + lane] = won[i] * scale;
  }
}

// --------------------------------------------------------------- plan
constexpr int MAXE = 256;

// start of each expert's rows, and (thread 0 of the writer) the tile list
DEV_INLINE void write_tiles(const MoeArgs& a, const int* count,
                            const int* start, int tid, int nthr) {
  // tile index of expert e's first tile
  __shared__ int tfirst[MAXE + 1];
  if (tid == 0) {
    int t = 0;
    for (int e = 0; e < a.experts; ++e) {
      tfirst[e] = t;
      t += (count[e] + a.tile_m - 1) / a.tile_m;
    }
    tfirst[a.experts] = t;
  }
  __syncthreads();
  for (int e = tid; e < a.experts; e += nthr)
    for (int t = tfirst[e]; t < tfirst[e + 1]; ++t) {
      const int r = (t - tfirst[e]) * a.tile_m;
      a.tile_expert[t] = e;
      a.tile_row0[t] = start[e] + r;
      a.tile_rows[t] = min(a.tile_m, count[e] - r);
    }
  for (int t = tfirst[a.experts] + tid; t < a.max_tiles; t += nthr)
    a.tile_rows[t] = 0;
}

__global__ __launch_bounds__(256)
void moe_plan_one_kernel(MoeArgs a) {
  __shared__ int count[MAXE], start[MAXE], cursor[MAXE];
  const int tid = threadIdx.x;
  const int P = a.rows * a.top;
  for (int e = tid; e < a.experts; e += 256) count[e] = 0;
  __syncthreads();
  for (int p = tid; p < P; p += 256)
    if (a.ids[p] < a.experts) atomicAdd(&count[a.ids[p]], 1);
  __syncthreads();
  if (tid == 0) {
    int s = 0;
    for (int e = 0; e < a.experts; ++e) {
      start[e] = s;
      cursor[e] = s;
      s += count[e];
    }
  }
  __syncthreads();
  for (int p = tid; p < P; p += 256)
    if (a.ids[p] < a.experts) a.perm[atomicAdd(&cursor[a.ids[p]], 1)] = p;
  write_tiles(a, count, start, tid, 256);
}

__global__ void moe_zero_kernel(MoeArgs a) {
  for (int e = threadIdx.x; e < 2 * a.experts; e += blockDim.x)
    a.counters[e] = 0;
}

constexpr int PLAN_PAIRS = 2048;          // pairs per workgroup

__global__ __launch_bounds__(256)
void moe_count_kernel(MoeArgs a) {
  __shared__ int count[MAXE];
  const int tid = threadIdx.x;
  const int P = a.rows * a.top;
  const int p0 = blockIdx.x * PLAN_PAIRS;
  for (int e = tid; e < a.experts; e += 256) count[e] = 0;
  __syncthreads();
  for (int p = p0 + tid; p < min(P, p0 + PLAN_PAIRS); p += 256)
    if (a.ids[p] < a.experts) atomicAdd(&count[a.ids[p]], 1);
  __syncthreads();
  for (int e = tid; e < a.experts; e += 256)
    if (count[e]) atomicAdd(&a.counters[e], count[e]);
}

__global__ __launch_bounds__(256)
void moe_scatter_kernel(MoeArgs a) {
  __shared__ int count[MAXE], start[MAXE], total[MAXE], base[MAXE];
  const int tid = threadIdx.x;
  const int P = a.rows * a.top;
  const int p0 = blockIdx.x * PLAN_PAIRS;
  for (int e = tid; e < a.experts; e += 256) {
    total[e] = a.counters[e];
    count[e] = 0;
  }
  __syncthreads();
  if (tid == 0) {
    int s = 0;
    for (int e = 0; e < a.experts; ++e) {
      start[e] = s;
      s += total[e];
    }
  }
  for (int p = p0 + tid; p < min(P, p0 + PLAN_PAIRS); p += 256)
    if (a.ids[p] < a.experts) atomicAdd(&count[a.ids[p]], 1);
  __syncthreads();
  for (int e = tid; e < a.experts; e += 256)
    base[e] = start[e] +
              (count[e] ? atomicAdd(&a.counters[a.experts + e], count[e]) : 0);
  __syncthreads();
  for (int p = p0 + tid; p < min(P, p0 + PLAN_PAIRS); p += 256)
    if (a.ids[p] < a.experts) a.perm[atomicAdd(&base[a.ids[p]], 1)] = p;
  if (blockIdx.x == 0) write_tiles(a, total, start, tid, 256);
}

template <typename T>
DEV_INLINE float expert_gate(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  // the result is rounded to bf16: hardware exponential and reciprocal do
  if constexpr (sizeof(T) == 2)
    return g * __builtin_amdgcn_rcpf(1.f + __expf(-1.702f * g)) * (u + 1.f);
  return g / (1.f + expf(-1.702f * g)) * (u + 1.f);
}

DEV_INLINE float relu_squared(float x) {
  x = fmaxf(x, 0.f);
  return x * x;
}

// --------------------------------------- small row counts: stream weights
// One workgroup per (16-row tile, 32 weight rows); its waves split K.
template <typename T, bool UP, bool GATED>
__global__ __launch_bounds__(256)
void moe_small_kernel(MoeArgs a) {
  __shared__ float part[4][2][16][17];
  const int tile = blockIdx.y;
  const int rows = a.tile_rows[tile];
  if (rows == 0) return;
  const int e = a.tile_expert[tile];
  const int p0 = a.tile_row0[tile];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int K = UP ? a.width : a.ffp;
  const int N = UP ? (GATED ? 2 : 1) * a.ffp : a.width;
  const int n0 = blockIdx.x * 32;

  const int pr = p0 + min(lr, rows - 1);
  const T* arow;
  if constexpr (UP)
    arow = reinterpret_cast<const T*>(a.h) +
           int64_t(a.perm[pr] / a.top) * a.width;
  else
    arow = reinterpret_cast<const T*>(a.act) + int64_t(pr) * a.ffp;
  const T* wb = reinterpret_cast<const T*>(UP ? a.w_up : a.w_down) +
                int64_t(e) * N * K;
  const T* b0 = wb + int64_t(min(n0 + lr, N - 1)) * K;
  const T* b1 = wb + int64_t(min(n0 + 16 + lr, N - 1)) * K;
  f32x4_t acc0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, acc1 = acc0;
  // a wave takes 128 consecutive k (whole lines of every weight row),
  // all loads before the MFMAs
  for (int k0 = w * 128; k0 < K; k0 += 512) {
    Frag8<T> fa[4], f0[4], f1[4];
    if (k0 + 128 <= K) {
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = k0 + u * 32 + g * 8;
        f0[u].load(b0 + k);
        f1[u].load(b1 + k);
        fa[u].load(arow + k);
      }
    } else {
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = k0 + u * 32 + g * 8;
        fa[u].zero();
        f0[u].zero();
        f1[u].zero();
        if (k < K) {
          fa[u].load(arow + k);
          f0[u].load(b0 + k);
          f1[u].load(b1 + k);
        }
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      acc0 = Frag8<T>::mma(fa[u], f0[u], acc0);
      acc1 = Frag8<T>::mma(fa[u], f1[u], acc1);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    part[w][0][g * 4 + r][lr] = acc0[r];
    part[w][1][g * 4 + r][lr] = acc1[r];
  }
  __syncthreads();
  const int row = threadIdx.x >> 4, col = threadIdx.x & 15;
  if (row >= rows) return;
  float s0 = 0.f, s1 = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    s0 += part[i][0][row][col];
    s1 += part[i][1][row][col];
  }
  const int pair = a.perm[p0 + row];
  if constexpr (UP) {
    const float wt = a.weights[pair];
    T* o = reinterpret_cast<T*>(a.act) + int64_t(p0 + row) * a.ffp;
    if constexpr (GATED) {
      act_store(o + blockIdx.x * 16 + col,
                expert_gate<T>(s0 * wt, s1 * wt, a.limit));
    } else {
      act_store(o + n0 + col, relu_squared(s0) * wt);
      act_store(o + n0 + 16 + col, relu_squared(s1) * wt);
    }
  } else {
    T* y = reinterpret_cast<T*>(a.y) + int64_t(pair) * a.width;
    if (n0 + col < N) act_store(y + n0 + col, s0);
    if (n0 + 16 + col < N) act_store(y + n0 + 16 + col, s1);
  }
}

// ------------------------------------------- large row counts: LDS tiles
// (32 WM) x (16 WN) MFMA blocks per wave pair grid, K step 64, double-
// buffered through direct global->LDS loads.  A row's eight 16-byte
// pieces land XOR-swizzled by the row number (the swizzle is applied to
// the global address), which spreads the fragment reads of 16 rows over
// all banks.  Two heights: 256 x 256 with eight waves of 128 x 64 each
// (fewest LDS bytes per MFMA), and 128 x 128 with four of 64 x 64 for
// experts with fewer rows.
constexpr int BK = 64;

DEV_INLINE void lds_load16(const void* g, void* l) {
  __builtin_amdgcn_global_load_lds(
      (const __attribute__((address_space(1))) void*)g,
      (__attribute__((address_space(3))) void*)l, 16, 0, 0);
}

template <bool UP, int TT, bool GATED>
__global__ __launch_bounds__(TT == 256 ? 512 : 256, 2)
void moe_tile_kernel(MoeArgs a, int n_blocks) {
  constexpr int NT = TT == 256 ? 512 : 256;       // threads
  constexpr int NCOL = TT == 256 ? 4 : 2;         // waves along columns
  constexpr int MI = TT == 256 ? 8 : 4;           // 16-row blocks per wave
  constexpr int PIECES = TT * 8 / NT;
  extern __shared__ __attribute__((aligned(16))) uint16_t lds[];
  // consecutive workgroups go to different XCDs; give each XCD whole
  // runs of one tile's column blocks so its L2 holds the rows once
  const int total = gridDim.x;
  const int per = (total + 7) / 8;
  const int wid = (blockIdx.x % 8) * per + blockIdx.x / 8;
  if (wid >= n_blocks * a.max_tiles) return;
  const int tile = wid / n_blocks, nb = wid % n_blocks;
  const int rows = a.tile_rows[tile];
  if (rows == 0) return;
  const int e = a.tile_expert[tile];
  const int p0 = a.tile_row0[tile];
  const int K = UP ? a.width : a.ffp;
  const int N = UP ? (GATED ? 2 : 1) * a.ffp : a.width;
  const int n0 = nb * TT;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int lr = lane & 15, g = lane >> 4;

  // the rows' pairs and weights, for the gather and the epilogue
  __shared__ int s_pair[TT];
  __shared__ float s_weight[TT];
  for (int r = tid; r < TT; r += NT) {
    const int pair = a.perm[p0 + min(r, rows - 1)];
    s_pair[r] = pair;
    if constexpr (UP) s_weight[r] = a.weights[pair];
  }
  __syncthreads();

  // piece i of this thread: tile row i * NT/8 + tid / 8, 16-byte column
  // tid % 8, holding global column (tid % 8) ^ (row & 7)
  const uint16_t* abase =
      reinterpret_cast<const uint16_t*>(UP ? a.h : a.act);
  const uint16_t* bbase =
      reinterpret_cast<const uint16_t*>(UP ? a.w_up : a.w_down) +
      int64_t(e) * N * K;
  uint32_t ap[PIECES], bp[PIECES];        // element offsets
#pragma unroll
  for (int i = 0; i < PIECES; ++i) {
    const int r = i * (NT / 8) + (tid >> 3);
    const int c = ((tid & 7) ^ (r & 7)) * 8;
    if constexpr (UP)
      ap[i] = uint32_t(s_pair[r] / a.top) * K + c;
    else
      ap[i] = uint32_t(p0 + min(r, rows - 1)) * K + c;
    bp[i] = uint32_t(min(n0 + r, N - 1)) * K + c;
  }
  auto stage = [&](int buf, int k0) {
    uint16_t* la = lds + buf * 2 * TT * BK;
    uint16_t* lb = la + TT * BK;
#pragma unroll
    for (int i = 0; i < PIECES; ++i) {
      // wave-uniform LDS base; lane l lands at base + 16 l
      lds_load16(abase + k0 + ap[i], la + (i * (NT / 8) + w * 8) * BK);
      lds_load16(bbase + k0 + bp[i], lb + (i * (NT / 8) + w * 8) * BK);
    }
  };

  const int wm = (w / NCOL) * MI * 16, wn = (w % NCOL) * 64;
  f32x4_t acc[MI][4];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  const int nk = K / BK;
  stage(0, 0);
  for (int kt = 0; kt < nk; ++kt) {
    // this wave's pieces of stage kt have landed, then everybody's
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (kt + 1 < nk) stage((kt + 1) & 1, (kt + 1) * BK);
    const uint16_t* la = lds + (kt & 1) * 2 * TT * BK;
    const uint16_t* lb = la + TT * BK;
    auto frag = [&](const uint16_t* base, int row, int kk) {
      return *reinterpret_cast<const s16x8_t*>(
          base + row * BK + (((kk * 4 + g) ^ (row & 7)) * 8));
    };
    // all of the first half's fragments, then the second half's one by
    // one under the first half's MFMAs
    s16x8_t fa[2][MI], fb[2][4];
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
#pragma unroll
      for (int j = 0; j < 4; ++j) fb[kk][j] = frag(lb, wn + j * 16 + lr, kk);
#pragma unroll
      for (int i = 0; i < MI; ++i) fa[kk][i] = frag(la, wm + i * 16 + lr, kk);
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              fa[kk][i], fb[kk][j], acc[i][j], 0, 0, 0);
    constexpr int MFMA = 0x8, DS_READ = 0x100;
    __builtin_amdgcn_sched_group_barrier(DS_READ, 4 + MI, 0);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      __builtin_amdgcn_sched_group_barrier(MFMA, 4, 0);
      __builtin_amdgcn_sched_group_barrier(DS_READ, 2, 0);
    }
#pragma unroll
    for (int i = 4; i < MI; ++i) {
      __builtin_amdgcn_sched_group_barrier(MFMA, 4, 0);
      __builtin_amdgcn_sched_group_barrier(DS_READ, 1, 0);
    }
    __builtin_amdgcn_sched_group_barrier(MFMA, 4 * MI, 0);
  }

#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tr = wm + i * 16 + g * 4 + r;
      if (tr >= rows) continue;
      const int pair = s_pair[tr];
      if constexpr (UP) {
        const float wt = s_weight[tr];
        uint16_t* o = reinterpret_cast<uint16_t*>(a.act) +
                      int64_t(p0 + tr) * a.ffp;
        if constexpr (GATED) {
#pragma unroll
          for (int j = 0; j < 4; j += 2) {
            const int f = (n0 + wn + j * 16) / 2 + lr;
            if (f < a.ffp)
              o[f] = f32_to_bf16(expert_gate<uint16_t>(
                  acc[i][j][r] * wt, acc[i][j + 1][r] * wt, a.limit));
          }
        } else {
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int f = n0 + wn + j * 16 + lr;
            if (f < a.ffp)
              o[f] = f32_to_bf16(relu_squared(acc[i][j][r]) * wt);
          }
        }
      } else {
        uint16_t* o = reinterpret_cast<uint16_t*>(a.y) +
                      int64_t(pair) * a.width;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int c = n0 + wn + j * 16 + lr;
          if (c < N) o[c] = f32_to_bf16(acc[i][j][r]);
        }
      }
    }
}

template <typename T>
void route(const MoeArgs& a, hipStream_t st) {
  const dim3 grid((a.rows + 15) / 16), blk(512);
  if (a.routes <= 16)
    hipLaunchKernelGGL((moe_route_kernel<T, 1>), grid, blk, 0, st, a);
  else if (a.routes <= 32)
    hipLaunchKernelGGL((moe_route_kernel<T, 2>), grid, blk, 0, st, a);
  else if (a.routes <= 48)
    hipLaunchKernelGGL((moe_route_kernel<T, 3>), grid, blk, 0, st, a);
  else if (a.routes <= 64)
    hipLaunchKernelGGL((moe_route_kernel<T, 4>), grid, blk, 0, st, a);
  else if (a.routes <= 128)
    hipLaunchKernelGGL((moe_route_kernel<T, 8>), grid, blk, 0, st, a);
  else
    hipLaunchKernelGGL((moe_route_kernel<T, 16>), grid, blk, 0, st, a);
}

template <typename T>
void small(const MoeArgs& a, hipStream_t st) {
  if (a.gated)
    hipLaunchKernelGGL((moe_small_kernel<T, true, true>),
                       dim3(2 * a.ffp / 32, a.max_tiles), dim3(256), 0, st,
                       a);
  else
    hipLaunchKernelGGL((moe_small_kernel<T, true, false>),
                       dim3(a.ffp / 32, a.max_tiles), dim3(256), 0, st, a);
  hipLaunchKernelGGL((moe_small_kernel<T, false, false>),
                     dim3((a.width + 31) / 32, a.max_tiles), dim3(256), 0, st,
                     a);
}

template <bool UP, int TT, bool GATED>
void tiled_one(const MoeArgs& a, hipStream_t st) {
  const size_t smem = size_t(4) * TT * BK * 2;
  const int nb = ((UP ? (GATED ? 2 : 1) * a.ffp : a.width) + TT - 1) / TT;
  auto* k = moe_tile_kernel<UP, TT, GATED>;
  if (smem > 65536)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              int(smem));
  hipLaunchKernelGGL(k, dim3((nb * a.max_tiles + 7) / 8 * 8),
                     dim3(TT == 256 ? 512 : 256), smem, st, a, nb);
}

template <int TT>
void tiled(const MoeArgs& a, hipStream_t st) {
  if (a.gated) tiled_one<true, TT, true>(a, st);
  else tiled_one<true, TT, false>(a, st);
  tiled_one<false, TT, false>(a, st);
}

}  // namespace

void launch_moe_route(const MoeArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  if (a.f32) route<float>(a, st);
  else route<uint16_t>(a, st);
}

void launch_moe_plan(const MoeArgs& a, hipStream_t st) {
  const int P = a.rows * a.top;
  if (P == 0) return;
  if (P <= 2 * PLAN_PAIRS) {
    hipLaunchKernelGGL(moe_plan_one_kernel, dim3(1), dim3(256), 0, st, a);
    return;
  }
  const dim3 grid((P + PLAN_PAIRS - 1) / PLAN_PAIRS);
  hipLaunchKernelGGL(moe_zero_kernel, dim3(1), dim3(256), 0, st, a);
  hipLaunchKernelGGL(moe_count_kernel, grid, dim3(256), 0, st, a);
  hipLaunchKernelGGL(moe_scatter_kernel, grid, dim3(256), 0, st, a);
}

void launch_moe_experts(const MoeArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  if (a.f32) {
    small<float>(a, st);
  } else if (a.tile_m == 16) {
    small<uint16_t>(a, st);
  } else {
    if (a.tile_m == 256) tiled<256>(a, st);
    else tiled<128>(a, st);
  }
}

}  // namespace rlli
