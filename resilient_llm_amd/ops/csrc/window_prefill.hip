// Tiled prompt attention over the paged cache for the windowed, sinked
// softmax of window_attn.hip (bf16 matrix cores, f32 softmax).
//
// A workgroup owns one tile of 32 * SUB prompt rows of a sequence and up
// to eight (query head, 32-row sub-tile) units of one kv head, one wave
// per unit, so every staged K/V tile is shared by all of them.  Only the
// 64-token K/V tiles that the window or the kept first tokens reach are
// walked.  Rows were rotated and cached by window_rope_append before.
// P is the larger of the key and value widths, rounded up; the unused
// columns are zeros.

#include "attn.h"

#include <type_traits>

namespace rlli {
namespace {

constexpr float kNegInf = -1e30f;
constexpr int KVBLK = 64;
constexpr int PPAD = KVBLK + 8;

template <int P, typename KC>
__global__ __launch_bounds__(512)
void window_prefill_kernel(WindowAttnArgs a, int heads_per_wg, int n_sub) {
  constexpr int DC = P / 32;             // contraction chunks of QK^T
  constexpr int CT = P / 16;             // output column tiles
  constexpr int KROW = P + 8;
  using elem = typename KC::elem;
  using vec8 = typename KC::vec8;
  const int group = a.n_q / a.n_kv;
  const int n_hw = (group + heads_per_wg - 1) / heads_per_wg;
  const int tile = blockIdx.x;
  const int kvh = blockIdx.y / n_hw;
  const int hw = blockIdx.y % n_hw;
  const int row0 = a.tiles[tile];
  const int pos0 = a.tiles[a.n_tiles + tile];
  const int nrows = a.tiles[2 * a.n_tiles + tile];
  const int32_t* bt =
      a.block_tables + int64_t(a.tiles[3 * a.n_tiles + tile]) * a.max_blocks;

  const int lane = threadIdx.x & 63;
  const int wave = threadIdx.x >> 6;
  const int jcol = lane & 15;
  const int koct = lane >> 4;
  const int hl = hw * heads_per_wg + wave / n_sub;   // head in the group
  const int sub0 = (wave % n_sub) * 32;              // first tile row
  const bool active = hl < group && sub0 < nrows;
  const int head = kvh * group + hl;

  extern __shared__ __attribute__((aligned(16))) char smem_raw[];
  uint16_t* vt = reinterpret_cast<uint16_t*>(smem_raw);     // [P][PPAD]
  uint16_t* ks = vt + P * PPAD;                             // [64][KROW]
  uint16_t* p_lds = ks + KVBLK * KROW + wave * 32 * PPAD;

  const uint16_t* qkv = reinterpret_cast<const uint16_t*>(a.qkv);
  s16x8_t qf[2][DC];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt)
#pragma unroll
    for (int dc = 0; dc < DC; ++dc) {
      const int r = sub0 + qt * 16 + jcol;
      const int d = dc * 32 + koct * 8;
      uint4 raw = {0, 0, 0, 0};
      if (active && r < nrows && d < a.dim)
        raw = *reinterpret_cast<const uint4*>(
            qkv + int64_t(row0 + r) * a.stride + head * a.dim + d);
      qf[qt][dc] = *reinterpret_cast<s16x8_t*>(&raw);
    }

  f32x4_t o_acc[2][CT];
  float m_st[2][4], l_st[2][4];
#pragma unroll
  for (int qt = 0; qt < 2; ++qt) {
#pragma unroll
    for (int ct = 0; ct < CT; ++ct) o_acc[qt][ct] = f32x4_t{0, 0, 0, 0};
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      m_st[qt][r] = kNegInf;
      l_st[qt][r] = 0.f;
    }
  }

  const elem* kc = reinterpret_cast<const elem*>(a.k_cache);
  const elem* vc = reinterpret_cast<const elem*>(a.v_cache);
  const int hi = pos0 + nrows;
  const int lo = max(0, pos0 - a.window + 1);        // tile-wide bound
  const int keep = min(a.keep_first, hi);
  int kv0 = (lo / KVBLK) * KVBLK;
  const int w_start = kv0;
  if (keep > 0) kv0 = 0;
  while (kv0 < hi) {
    // tiles between the kept tokens and the window hold nothing visible
    if (kv0 >= keep && kv0 < w_start) kv0 = w_start;
    __syncthreads();
    for (int idx = threadIdx.x; idx < KVBLK * (P / 8); idx += blockDim.x) {
      const int kv = idx / (P / 8);
      const int d8 = (idx % (P / 8)) * 8;
      const int p = kv0 + kv;
      vec8 vraw = {}, kraw = {};
      if (p < hi) {
        const int64_t rowi =
            (int64_t(bt[p / a.block_size]) * a.n_kv + kvh) * a.block_size +
            p % a.block_size;
        if (d8 < a.dim)
          kraw = *reinterpret_cast<const vec8*>(kc + rowi * a.dim + d8);
        if (d8 < a.vdim)
          vraw = *reinterpret_cast<const vec8*>(vc + rowi * a.vdim + d8);
      }
      float vf[8], kf[8];
      KC::to_f32(vraw, vf);
      KC::to_f32(kraw, kf);
      bf16x8 kp;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        kp.s[j] = f32_to_bf16(kf[j]);
        vt[(d8 + j) * PPAD + kv] = f32_to_bf16(vf[j]);
      }
      *reinterpret_cast<uint4*>(ks + kv * KROW + d8) = kp.u;
    }
    __syncthreads();

    const int rlast = pos0 + min(sub0 + 31, nrows - 1);
    const bool sees = active && kv0 <= rlast &&
                      (kv0 < keep ||
                       pos0 + sub0 - (kv0 + KVBLK - 1) < a.window);
    if (sees) {
      constexpr int KT = KVBLK / 16;
      f32x4_t s_acc[2][KT];
#pragma unroll
      for (int qt = 0; qt < 2; ++qt)
#pragma unroll
        for (int kt = 0; kt < KT; ++kt) s_acc[qt][kt] = f32x4_t{0, 0, 0, 0};
#pragma unroll
      for (int kt = 0; kt < KT; ++kt)
#pragma unroll
        for (int dc = 0; dc < DC; ++dc) {
          const s16x8_t kf = *reinterpret_cast<const s16x8_t*>(
              ks + (kt * 16 + jcol) * KROW + dc * 32 + koct * 8);
#pragma unroll
          for (int qt = 0; qt < 2; ++qt)
            s_acc[qt][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                qf[qt][dc], kf, s_acc[qt][kt], 0, 0, 0);
        }
#pragma unroll
      for (int qt = 0; qt < 2; ++qt) {
        float corr[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int trow = qt * 16 + koct * 4 + r;
          const int qpos = pos0 + sub0 + trow;
          float sv[KT], mx = kNegInf;
#pragma unroll
          for (int kt = 0; kt < KT; ++kt) {
            const int c = kv0 + kt * 16 + jcol;
            const bool ok = c <= qpos &&
                            (qpos - c < a.window || c < a.keep_first);
            sv[kt] = ok ? s_acc[qt][kt][r] * a.scale : kNegInf;
            mx = fmaxf(mx, sv[kt]);
          }
#pragma unroll
          for (int off = 8; off > 0; off >>= 1)
            mx = fmaxf(mx, __shfl_xor(mx, off, kWave));
          const float m_new = fmaxf(m_st[qt][r], mx);
          corr[r] = __expf(m_st[qt][r] - m_new);
          m_st[qt][r] = m_new;
          float rs = 0.f;
#pragma unroll
          for (int kt = 0; kt < KT; ++kt) {
            const float p = __expf(sv[kt] - m_new);
            rs += p;
            p_lds[trow * PPAD + kt * 16 + jcol] = f32_to_bf16(p);
          }
#pragma unroll
          for (int off = 8; off > 0; off >>= 1)
            rs += __shfl_xor(rs, off, kWave);
          l_st[qt][r] = l_st[qt][r] * corr[r] + rs;
        }
#pragma unroll
        for (int ct = 0; ct < CT; ++ct)
#pragma unroll
          for (int r = 0; r < 4; ++r) o_acc[qt][ct][r] *= corr[r];
      }
#pragma unroll
      for (int kb = 0; kb < KVBLK / 32; ++kb) {
        s16x8_t pf[2];
#pragma unroll
        for (int qt = 0; qt < 2; ++qt)
          pf[qt] = *reinterpret_cast<const s16x8_t*>(
              p_lds + (qt * 16 + jcol) * PPAD + kb * 32 + koct * 8);
#pragma unroll
        for (int ct = 0; ct < CT; ++ct) {
          const s16x8_t vf = *reinterpret_cast<const s16x8_t*>(
              vt + (ct * 16 + jcol) * PPAD + kb * 32 + koct * 8);
#pragma unroll
          for (int qt = 0; qt < 2; ++qt)
            o_acc[qt][ct] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                pf[qt], vf, o_acc[qt][ct], 0, 0, 0);
        }
      }
    }
    kv0 += KVBLK;
  }

  if (!active) return;
  uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
  const float snk = a.sink ? a.sink[head] : kNegInf;
#pragma unroll
  for (int qt = 0; qt < 2; ++qt)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int rr = sub0 + qt * 16 + koct * 4 + r;
      if (rr >= nrows) continue;
      const float m_new = fmaxf(m_st[qt][r], snk);
      const float corr = __expf(m_st[qt][r] - m_new);
      const float l = l_st[qt][r] * corr +
                      (a.sink ? __expf(snk - m_new) : 0.f);
      const float f = corr / l;
#pragma unroll
      for (int ct = 0; ct < CT; ++ct) {
        const int d = ct * 16 + jcol;
        if (d < a.vdim)
          out[(int64_t(row0 + rr) * a.n_q + head) * a.vdim + d] =
              f32_to_bf16(o_acc[qt][ct][r] * f);
      }
    }
}

template <int P, typename KC>
void go(const WindowAttnArgs& a, hipStream_t st) {
  const int group = a.n_q / a.n_kv;
  const int sub = window_prefill_sub_tiles(group);
  const int hpw = 8 / sub < group ? 8 / sub : group;
  const int waves = hpw * sub;
  const size_t smem = size_t(P) * PPAD * 2 + size_t(KVBLK) * (P + 8) * 2 +
                      size_t(waves) * 32 * PPAD * 2;
  auto* k = window_prefill_kernel<P, KC>;
  if (smem > 65536)
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              int(smem));
  hipLaunchKernelGGL(k, dim3(a.n_tiles, a.n_kv * ((group + hpw - 1) / hpw)),
                     dim3(waves * 64), smem, st, a, hpw, sub);
}

template <int P>
void by_cache(const WindowAttnArgs& a, hipStream_t st) {
  if (a.cache == kCacheFP8) go<P, CacheFP8>(a, st);
  else go<P, CacheBF16>(a, st);
}

}  // namespace

// 32-row sub-tiles per tile: fills up to eight waves with (head, rows)
int window_prefill_sub_tiles(int group) {
  return group == 1 ? 8 : group == 2 ? 4 : group <= 4 ? 2 : 1;
}

void launch_window_prefill(const WindowAttnArgs& a, hipStream_t st) {
  if (a.n_tiles == 0) return;
  const int d = a.dim > a.vdim ? a.dim : a.vdim;
  if (d <= 32) by_cache<32>(a, st);
  else if (d <= 64) by_cache<64>(a, st);
  else if (d <= 96) by_cache<96>(a, st);
  else if (d <= 128) by_cache<128>(a, st);
  else if (d <= 192) by_cache<192>(a, st);
  else by_cache<256>(a, st);
}

}  // namespace rlli
