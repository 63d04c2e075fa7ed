// Latent attention over a paged cache of one latent per token.
//
// A token caches only its normed latent c (kv_rank values).  With k = Uk c
// and v = Uv c per head, q . k = (Uk^T q) . c and sum p v = Uv (sum p c):
// queries that are absorbed this way score against the latents directly,
// all heads sharing one key/value row, and the value product runs once per
// query.  That is the decode form (and that of short portions):
//   latent_prep      norms of the query and key/value latents, the latter
//                    straight into its cache slot
//   head_linear      y[t,h] = W[h] x[t,h], optionally gated; Uk^T before
//                    and Uv after the attention
//   latent_attn      (rows x heads) against the latents, split over keys;
//                    a 32-token latent tile in LDS is both K and V
//   latent_combine   joins the splits
//   latent_gather    a sequence's latents as one matrix, for the expanded
//                    form of long portions (latent_prefill.hip)
// The 32-bit path and odd sizes take attn_rows.h with the latent as key
// and value.

#include "attn_rows.h"
#include "lat.h"

#include <type_traits>

namespace rlli {
namespace {

// -------------------------------------------------------------- prep
template <int V, typename T>
DEV_INLINE void load_vec(const T* p, float (&o)[V]) {
  if constexpr (V == 8) {
    const f32x4_t a = act_load4(p), b = act_load4(p + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o[j] = a[j];
      o[4 + j] = b[j];
    }
  } else {
    o[0] = act_load(p);
  }
}

// wave 0 norms the query latent, wave 1 the key/value latent
template <typename T, typename CE, int V>
__global__ __launch_bounds__(128)
void latent_prep_kernel(LatentPrepArgs a) {
  const int row = blockIdx.x, lane = threadIdx.x & 63;
  const bool kv = threadIdx.x >= 64;
  const T* p = reinterpret_cast<const T*>(a.proj) + int64_t(row) * a.stride +
               (kv ? a.q_rank : 0);
  const int n = kv ? a.kv_rank : a.q_rank;
  float ss = 0.f;
  for (int c = lane * V; c < n; c += 64 * V) {
    float v[V];
    load_vec<V>(p + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += v[j] * v[j];
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / n + a.eps);
  const float* gain = kv ? a.kv_norm : a.q_norm;
  for (int c = lane * V; c < n; c += 64 * V) {
    float v[V];
    load_vec<V>(p + c, v);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = v[j] * inv * gain[c + j];
    if (kv) {
      CE* o = reinterpret_cast<CE*>(a.cache) +
              int64_t(a.slots[row]) * n + c;
#pragma unroll
      for (int j = 0; j < V; ++j) cache_store(o + j, v[j]);
    } else {
      T* o = reinterpret_cast<T*>(a.cq) + int64_t(row) * n + c;
      if constexpr (V == 8) {
        act_store4(o, f32x4_t{v[0], v[1], v[2], v[3]});
        act_store4(o + 4, f32x4_t{v[4], v[5], v[6], v[7]});
      } else {
        act_store(o, v[0]);
      }
    }
  }
}

// ------------------------------------------------------- head_linear
template <typename T>
DEV_INLINE void load_frag(Frag8<T>& f, const T* p, int k, int n, bool vec) {
  f.zero();
  if (k >= n) return;
  if (vec) {
    f.load(p + k);
    return;
  }
  alignas(16) T tmp[8];
#pragma unroll
  for (int j = 0; j < 8; ++j) tmp[j] = k + j < n ? p[k + j] : T(0);
  f.load(tmp);
}

// 16 * MT rows of one head.  KS = 1: each wave has 16 columns of its own;
// KS = 4: the waves split k over the same 16 columns.
template <typename T, int MT, int KS>
__global__ __launch_bounds__(256)
void head_linear_kernel(HeadLinearArgs a, bool vec_w, bool vec_x) {
  __shared__ float part[KS > 1 ? KS : 1][MT * 16][KS > 1 ? 17 : 1];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int h = blockIdx.y, r0 = blockIdx.z * MT * 16;
  const int n0 = (blockIdx.x * (KS > 1 ? 1 : 4) + (KS > 1 ? 0 : w)) * 16;
  if (KS == 1 && n0 >= a.n) return;
  const T* wp = reinterpret_cast<const T*>(a.w) +
                (int64_t(h) * a.n + min(n0 + lr, a.n - 1)) * a.k;
  const T* xp[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
    xp[m] = reinterpret_cast<const T*>(a.x) +
            int64_t(min(r0 + m * 16 + lr, a.rows - 1)) * a.x_stride +
            int64_t(h) * a.k;
  f32x4_t acc[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) acc[m] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  constexpr int U = MT <= 2 ? 4 : 2;      // k steps with loads in flight
  for (int k0 = KS > 1 ? w * 32 : 0; k0 < a.k; k0 += 32 * KS * U) {
    Frag8<T> fw[U], fx[U][MT];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = k0 + u * 32 * KS + g * 8;
      load_frag(fw[u], wp, k, a.k, vec_w);
#pragma unroll
      for (int m = 0; m < MT; ++m) load_frag(fx[u][m], xp[m], k, a.k, vec_x);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int m = 0; m < MT; ++m)
        acc[m] = Frag8<T>::mma(fx[u][m], fw[u], acc[m]);
  }
  auto put = [&](int row, int n, float v) {
    if (row >= a.rows || n >= a.n) return;
    const int64_t c = int64_t(h) * a.n + n;
    if (a.gate) {
      const float z = act_load(reinterpret_cast<const T*>(a.gate) +
                               row * a.gate_stride + c);
      v *= 1.f / (1.f + expf(-z));
    }
    act_store(reinterpret_cast<T*>(a.y) + row * a.y_stride + c, v);
  };
  if constexpr (KS > 1) {
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        part[w][m * 16 + g * 4 + r][lr] = acc[m][r];
    __syncthreads();
    for (int e = threadIdx.x; e < MT * 256; e += 256) {
      const int row = e / 16, c = e % 16;
      float v = 0.f;
#pragma unroll
      for (int s = 0; s < KS; ++s) v += part[s][row][c];
      put(r0 + row, n0 + c, v);
    }
  } else {
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        put(r0 + m * 16 + g * 4 + r, n0 + lr, acc[m][r]);
  }
}

// ------------------------------------------------------- latent_attn
constexpr int KT = 32;                    // keys of a tile
constexpr int SROW = KT + 4;              // score row in LDS

typedef float f32x2_t __attribute__((ext_vector_type(2)));
typedef __bf16 b16x2_t __attribute__((ext_vector_type(2)));

DEV_INLINE uint32_t pack2(float a, float b) {
  const b16x2_t v = __builtin_convertvector((f32x2_t{a, b}), b16x2_t);
  return __builtin_bit_cast(uint32_t, v);
}

template <typename KC>
DEV_INLINE uint4 to_bf16x8(const typename KC::vec8& raw) {
  if constexpr (std::is_same_v<KC, CacheBF16>) {
    return raw;
  } else {
    float f[8];
    KC::to_f32(raw, f);
    return uint4{pack2(f[0], f[1]), pack2(f[2], f[3]), pack2(f[4], f[5]),
                 pack2(f[6], f[7])};
  }
}

// MT (1 or 2) tiles of 16 query vectors.  Waves pair up over the tile's two
// groups of 16 keys to score: with half of the rank each (MT = 1, the
// softmax adds the halves) or with a query tile each.  Then every wave
// weighs all keys and accumulates 16 * NC of the output columns.
template <int MT, int NC, typename KC>
__global__ __launch_bounds__(256, MT == 1 ? 3 : 2)
void latent_attn_kernel(LatentAttnArgs a) {
  using vec8 = typename KC::vec8;
  using elem = typename KC::elem;
  constexpr int RP = NC * 64, RS = RP + 8, KS = RP / 32;
  constexpr int PF = KT * RP / 8 / 256;   // vectors a thread stages
  constexpr int KW = MT > 1 ? KS : KS / 2;
  constexpr int SP = MT > 1 ? 1 : 2;      // score parts to add
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* cs = reinterpret_cast<uint16_t*>(smem);      // [KT][RS]
  float* sc = reinterpret_cast<float*>(cs + KT * RS);    // [32][SROW]

  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int split = blockIdx.x;
  const bool decode = a.tiles == nullptr;
  int64_t vec0;
  int cnt, seq, first, off;
  if (decode) {
    seq = blockIdx.z;
    off = blockIdx.y * MT * 16;
    vec0 = int64_t(seq) * a.heads + off;
    cnt = min(MT * 16, a.heads - off);
    first = a.positions[seq];
  } else {
    const int t = blockIdx.y;
    vec0 = a.tiles[t];
    off = a.tiles[a.n_tiles + t];
    cnt = a.tiles[2 * a.n_tiles + t];
    seq = a.tiles[3 * a.n_tiles + t];
    first = a.pos0[seq];
  }
  auto qpos = [&](int i) {                // position of query vector i
    return decode ? first : first + (off + i) / a.heads;
  };
  // (a padded graph lane's position may run past its table)
  const int len = min(qpos(cnt - 1) + 1, a.max_blocks << a.block_shift);
  const int32_t* bt = a.block_tables + int64_t(seq) * a.max_blocks;
  const elem* cache = reinterpret_cast<const elem*>(a.cache);
  const int bmask = (1 << a.block_shift) - 1;

  // this thread's vectors of a tile; the pages of its two 16-token halves
  // are looked up a tile ahead
  vec8 pf[PF];
  int page[2];
  auto lookup = [&](int t) {
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int p = t * KT + i * 16;
      page[i] = p < len ? bt[p >> a.block_shift] : 0;
    }
  };
  auto fetch = [&](int t) {
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int e = i * 256 + threadIdx.x;
      const int p = t * KT + e / (RP / 8), d = e % (RP / 8) * 8;
      pf[i] = vec8{};
      if (p < len && d < a.rank)
        pf[i] = *reinterpret_cast<const vec8*>(
            cache + ((int64_t(page[2 * i / PF]) << a.block_shift) +
                     (p & bmask)) * a.rank + d);
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < PF; ++i) {
      const int e = i * 256 + threadIdx.x;
      *reinterpret_cast<uint4*>(cs + e / (RP / 8) * RS + e % (RP / 8) * 8) =
          to_bf16x8<KC>(pf[i]);
    }
  };
  int t = split;
  lookup(t);
  fetch(t);
  lookup(t + a.n_split);

  // this wave's queries, as fragments in registers
  const uint16_t* q = reinterpret_cast<const uint16_t*>(a.q);
  const int kg = w & 1, half = w >> 1;    // group of keys, half of the work
  const int q0 = MT == 1 ? 0 : half * 16, d0 = MT == 1 ? half * KW * 32 : 0;
  s16x8_t qf[KW];
#pragma unroll
  for (int kk = 0; kk < KW; ++kk) {
    uint4 raw = {0, 0, 0, 0};
    const int d = d0 + kk * 32 + g * 8;
    if (q0 + lr < cnt && d < a.rank)
      raw = *reinterpret_cast<const uint4*>(q + (vec0 + q0 + lr) * a.rank +
                                            d);
    qf[kk] = __builtin_bit_cast(s16x8_t, raw);
  }
  int qp[MT];                             // of row lr of each tile
#pragma unroll
  for (int m = 0; m < MT; ++m)
    qp[m] = m * 16 + lr < cnt ? qpos(m * 16 + lr) : -1;

  f32x4_t o[MT][NC];
  float ms[MT], ls[MT];                   // of row lr of each tile
#pragma unroll
  for (int m = 0; m < MT; ++m) {
#pragma unroll
    for (int c = 0; c < NC; ++c) o[m][c] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    ms[m] = kNegInf;
    ls[m] = 0.f;
  }

  for (; t * KT < len; t += a.n_split) {
    __syncthreads();                      // the last tile's readers
    stage();
    __syncthreads();
    fetch(t + a.n_split);
    lookup(t + 2 * a.n_split);
    f32x4_t s = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < KW; ++kk) {
      const s16x8_t kf = *reinterpret_cast<const s16x8_t*>(
          cs + (kg * 16 + lr) * RS + d0 + kk * 32 + g * 8);
      s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[kk], kf, s, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
      sc[(half * 16 + g * 4 + r) * SROW + kg * 16 + lr] = s[r];
    __syncthreads();
    s16x8_t pw[MT];                       // row lr, keys g * 8 + j
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      float p[8], mx = kNegInf;
#pragma unroll
      for (int j = 0; j < 8; j += 4) {
        f32x4_t v = *reinterpret_cast<const f32x4_t*>(
            sc + (m * 16 + lr) * SROW + g * 8 + j);
        if constexpr (SP == 2) {
          const f32x4_t u = *reinterpret_cast<const f32x4_t*>(
              sc + (16 + lr) * SROW + g * 8 + j);
#pragma unroll
          for (int i = 0; i < 4; ++i) v[i] += u[i];
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          p[j + i] = t * KT + g * 8 + j + i <= qp[m] ? v[i] * a.scale
                                                     : kNegInf;
          mx = fmaxf(mx, p[j + i]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, kWave));
      mx = fmaxf(mx, __shfl_xor(mx, 32, kWave));
      const float mn = fmaxf(ms[m], mx);
      const float corr = __expf(ms[m] - mn);
      float sum = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        p[i] = __expf(p[i] - mn);
        sum += p[i];
      }
      sum += __shfl_xor(sum, 16, kWave);
      sum += __shfl_xor(sum, 32, kWave);
      ls[m] = ls[m] * corr + sum;
      const uint4 raw = {pack2(p[0], p[1]), pack2(p[2], p[3]),
                         pack2(p[4], p[5]), pack2(p[6], p[7])};
      pw[m] = __builtin_bit_cast(s16x8_t, raw);
      if (!__all(mn == ms[m])) {
        ms[m] = mn;
        float cr[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) cr[r] = __shfl(corr, g * 4 + r, kWave);
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[m][c][r] *= cr[r];
      }
    }
    // columns in pairs: a dword of a row holds two of them, so eight rows'
    // dwords make the fragments of the even and of the odd columns
#pragma unroll
    for (int cp = 0; cp < NC / 2; ++cp) {
      uint32_t d[8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        d[j] = *reinterpret_cast<const uint32_t*>(
            cs + (g * 8 + j) * RS + w * NC * 16 + cp * 32 + lr * 2);
      uint4 ev, od;
      ev.x = __builtin_amdgcn_perm(d[1], d[0], 0x05040100);
      ev.y = __builtin_amdgcn_perm(d[3], d[2], 0x05040100);
      ev.z = __builtin_amdgcn_perm(d[5], d[4], 0x05040100);
      ev.w = __builtin_amdgcn_perm(d[7], d[6], 0x05040100);
      od.x = __builtin_amdgcn_perm(d[1], d[0], 0x07060302);
      od.y = __builtin_amdgcn_perm(d[3], d[2], 0x07060302);
      od.z = __builtin_amdgcn_perm(d[5], d[4], 0x07060302);
      od.w = __builtin_amdgcn_perm(d[7], d[6], 0x07060302);
      const s16x8_t fe = __builtin_bit_cast(s16x8_t, ev);
      const s16x8_t fo = __builtin_bit_cast(s16x8_t, od);
#pragma unroll
      for (int m = 0; m < MT; ++m) {
        o[m][2 * cp] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            pw[m], fe, o[m][2 * cp], 0, 0, 0);
        o[m][2 * cp + 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            pw[m], fo, o[m][2 * cp + 1], 0, 0, 0);
      }
    }
  }

#pragma unroll
  for (int m = 0; m < MT; ++m) {
    float l[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) l[r] = __shfl(ls[m], g * 4 + r, kWave);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = m * 16 + g * 4 + r;
      if (i >= cnt) continue;
#pragma unroll
      for (int cp = 0; cp < NC / 2; ++cp) {
        const int col = w * NC * 16 + cp * 32 + lr * 2;
        if (col >= a.rank) continue;
        const float v0 = o[m][2 * cp][r], v1 = o[m][2 * cp + 1][r];
        if (a.n_split == 1) {
          *reinterpret_cast<uint32_t*>(reinterpret_cast<uint16_t*>(a.out) +
                                       (vec0 + i) * a.rank + col) =
              pack2(v0 / l[r], v1 / l[r]);
        } else {
          *reinterpret_cast<f32x2_t*>(
              a.part_acc + ((vec0 + i) * a.n_split + split) * a.rank + col) =
              f32x2_t{v0, v1};
        }
      }
    }
    if (a.n_split > 1 && w == 0 && g == 0 && m * 16 + lr < cnt) {
      float* ml = a.part_ml + ((vec0 + m * 16 + lr) * a.n_split + split) * 2;
      ml[0] = ms[m];
      ml[1] = ls[m];
    }
  }
}

__global__ __launch_bounds__(128)
void latent_combine_kernel(LatentAttnArgs a) {
  const int64_t v = blockIdx.x;
  const float* ml = a.part_ml + v * a.n_split * 2;
  float mm = kNegInf, ll = 0.f;
  for (int s = 0; s < a.n_split; ++s) mm = fmaxf(mm, ml[2 * s]);
  for (int s = 0; s < a.n_split; ++s)
    ll += ml[2 * s + 1] * __expf(ml[2 * s] - mm);
  const float* acc = a.part_acc + v * a.n_split * a.rank;
  for (int c = threadIdx.x * 4; c < a.rank; c += 512) {
    f32x4_t o = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < a.n_split; ++s) {
      const float f = __expf(ml[2 * s] - mm);
      const f32x4_t p =
          *reinterpret_cast<const f32x4_t*>(acc + int64_t(s) * a.rank + c);
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] += f * p[j];
    }
    const uint2 out = {pack2(o[0] / ll, o[1] / ll),
                       pack2(o[2] / ll, o[3] / ll)};
    *reinterpret_cast<uint2*>(reinterpret_cast<uint16_t*>(a.out) +
                              v * a.rank + c) = out;
  }
}

// ------------------------------------------------------------ gather
template <typename KC>
__global__ __launch_bounds__(256)
void latent_gather_kernel(GatherArgs a) {
  using vec8 = typename KC::vec8;
  const int b = blockIdx.x;
  const int seq = a.blocks[b], tok0 = a.blocks[a.n + b];
  const int cnt = a.blocks[2 * a.n + b];
  const int64_t dst = a.blocks[3 * a.n + b];
  const int32_t* bt = a.block_tables + int64_t(seq) * a.max_blocks;
  const typename KC::elem* cache =
      reinterpret_cast<const typename KC::elem*>(a.cache);
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  const int nv = a.rank / 8;
  constexpr int kPart = kGatherRows / 8;  // rows of one workgroup
  for (int e = threadIdx.x; e < kPart * nv; e += 256) {
    const int r = blockIdx.y * kPart + e / nv, d = e % nv * 8;
    uint4 v = {0, 0, 0, 0};               // rows past the end are zeros
    if (r < cnt) {
      const int p = tok0 + r;
      const int64_t tok =
          int64_t(bt[p / a.block_size]) * a.block_size + p % a.block_size;
      v = to_bf16x8<KC>(
          *reinterpret_cast<const vec8*>(cache + tok * a.rank + d));
    }
    *reinterpret_cast<uint4*>(out + (dst + r) * a.rank + d) = v;
  }
}

template <int MT, int NC, typename KC>
void attn(const LatentAttnArgs& a, hipStream_t st) {
  constexpr int RS = NC * 64 + 8;
  constexpr size_t smem = size_t(KT) * RS * 2 + 32 * SROW * 4;
  auto* k = latent_attn_kernel<MT, NC, KC>;
  const dim3 grid = a.tiles ? dim3(a.n_split, a.n_tiles, 1)
                            : dim3(a.n_split,
                                   (a.heads + MT * 16 - 1) / (MT * 16),
                                   a.rows);
  hipLaunchKernelGGL(k, grid, dim3(256), smem, st, a);
}

template <int MT, typename KC>
void attn_rank(const LatentAttnArgs& a, hipStream_t st) {
  if (a.rank <= 128) attn<MT, 2, KC>(a, st);
  else if (a.rank <= 256) attn<MT, 4, KC>(a, st);
  else if (a.rank <= 384) attn<MT, 6, KC>(a, st);
  else attn<MT, 8, KC>(a, st);
}

template <typename KC>
void attn_tile(const LatentAttnArgs& a, hipStream_t st) {
  if (latent_tile(a.heads, a.tiles == nullptr) == 16) attn_rank<1, KC>(a, st);
  else attn_rank<2, KC>(a, st);
}

template <typename T, int KS>
void head_linear_rows(const HeadLinearArgs& a, hipStream_t st) {
  const bool vw = a.k % 8 == 0;
  const bool vx = vw && a.x_stride % 8 == 0 &&
                  reinterpret_cast<uintptr_t>(a.x) % 16 == 0;
  const int cols = KS > 1 ? 16 : 64;
  auto run = [&](auto* k, int rows) {
    hipLaunchKernelGGL(k, dim3((a.n + cols - 1) / cols, a.heads,
                               (a.rows + rows - 1) / rows),
                       dim3(256), 0, st, a, vw, vx);
  };
  if (a.rows <= 16) run(head_linear_kernel<T, 1, KS>, 16);
  else if (a.rows <= 32) run(head_linear_kernel<T, 2, KS>, 32);
  else run(head_linear_kernel<T, 4, KS>, 64);
}

template <typename T>
void head_linear(const HeadLinearArgs& a, hipStream_t st) {
  if (a.k >= 256) head_linear_rows<T, 4>(a, st);
  else head_linear_rows<T, 1>(a, st);
}

}  // namespace

void launch_latent_prep(const LatentPrepArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  const bool vec = a.q_rank % 8 == 0 && a.kv_rank % 8 == 0 &&
                   a.stride % 8 == 0;
  auto go = [&](auto t, auto c) {
    using T = decltype(t);
    using CE = decltype(c);
    if (vec)
      hipLaunchKernelGGL((latent_prep_kernel<T, CE, 8>), dim3(a.rows),
                         dim3(128), 0, st, a);
    else
      hipLaunchKernelGGL((latent_prep_kernel<T, CE, 1>), dim3(a.rows),
                         dim3(128), 0, st, a);
  };
  if (a.cache_kind == kCacheFP8) go(uint16_t{}, uint8_t{});
  else if (a.f32) go(float{}, float{});
  else go(uint16_t{}, uint16_t{});
}

void launch_head_linear(const HeadLinearArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  if (a.f32) head_linear<float>(a, st);
  else head_linear<uint16_t>(a, st);
}

bool latent_fast_ok(int rank, int block_size, bool f32) {
  return !f32 && rank % 8 == 0 && rank <= 512 && block_size >= 16 &&
         (block_size & (block_size - 1)) == 0;
}

int latent_tile(int heads, bool decode) {
  return decode && heads <= 16 ? 16 : kLatentVectors;
}

void launch_latent_attn(const LatentAttnArgs& a, hipStream_t st) {
  if (a.rows == 0 || (a.tiles && a.n_tiles == 0)) return;
  if (a.cache_kind == kCacheFP8) attn_tile<CacheFP8>(a, st);
  else attn_tile<CacheBF16>(a, st);
  if (a.n_split > 1)
    hipLaunchKernelGGL(latent_combine_kernel, dim3(a.rows * a.heads),
                       dim3(128), 0, st, a);
}

void launch_latent_rows(const WindowAttnArgs& a, bool decode,
                        hipStream_t st) {
  if (a.cache == kCacheFP8)
    run_window_rows<uint16_t, uint8_t, 16>(a, decode, st);
  else if (a.f32) run_window_rows<float, float, 16>(a, decode, st);
  else run_window_rows<uint16_t, uint16_t, 16>(a, decode, st);
}

void launch_latent_gather(const GatherArgs& a, hipStream_t st) {
  if (a.n == 0) return;
  if (a.cache_kind == kCacheFP8)
    hipLaunchKernelGGL(latent_gather_kernel<CacheFP8>, dim3(a.n, 8),
                       dim3(256), 0, st, a);
  else
    hipLaunchKernelGGL(latent_gather_kernel<CacheBF16>, dim3(a.n, 8),
                       dim3(256), 0, st, a);
}

}  // namespace rlli
