// The sequential half of the recurrences' prompt kernels: chunk after chunk
// of a sequence with the state in MFMA accumulators, and the norm and gate
// that follow.
//
// A workgroup owns one (sequence, head, slice of value columns); a wave the
// 16 output rows of a sub-chunk and every fourth key tile of the state.  All
// products are f32 MFMA.  A chunk's operands travel in registers, loaded
// while the chunk before it computes.  A sequence's chunks follow one
// another and only the last is short, so no table is on the path of a load.
// Loads and stores are unconditional where sizes allow (what has no place
// goes to spare rows), since a branch around one makes later waits drain
// everything in flight.
//
// kScanMax: with F the chunk's running log-decay, a = i - F and the maximum
// M_t = max(m, max_{s <= t} a_s), m what the chunk started with,
//     m_t = F_t + M_t,   O_t = e^{m - M_t} q_t S + sum_s q_t k_s e^{a_s - M_t} v_s
//     S   = e^{m - M_C} S + sum_s k_s e^{a_s - M_C} v_s^T
// A holds e^{a_s - max_{r <= t} a_r}; the rest of the exponent is a row
// factor <= 1.
// kScanDelta: U = Ub - W S takes the place of the values, two waves of
// barriers per chunk.

#include "rec_math.h"

#include <type_traits>

namespace rlli {
namespace {

constexpr int C = kRecChunk;

// VT value tiles of 16 columns per workgroup, MD key tiles per wave.  FULL:
// dim is 64 MD, values come in whole slices and rows are aligned, so that no
// load is conditional (a branch around a load ends in a wait for it): rows
// behind the last one are loaded from the last one instead.
template <typename T, int MODE, int VT, int MD, bool FULL>
__global__ __launch_bounds__(256, FULL && VT == 1 && MD <= 2 ? 2 : 1)
void rec_scan_kernel(ScanArgs a, bool vec_q, bool vec_v) {
  constexpr bool MAX = MODE == kScanMax, DELTA = MODE == kScanDelta;
  constexpr bool RAW = MODE != kScanPlain;      // operands as they are
  using KE = std::conditional_t<RAW, T, float>;
  using QE = KE;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  constexpr int VS = VT * 16, SR = VS + 4;
  const int DP = FULL ? 64 * MD : a.dpad, ndt = DP / 16;
  float* Sl = sm;                         // [DP][SR]
  float* Vl = Sl + DP * SR;               // [64][SR]
  float* Vk = RAW ? Vl + C * SR : Vl;     // [64][SR] with the key factors
  const int seq = blockIdx.x / a.heads, h = blockIdx.x % a.heads;
  const int v0 = blockIdx.y * VS;
  const int lane = threadIdx.x & 63;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lr = lane & 15, g = lane >> 4;
  const int first = a.seqs[seq], count = a.seqs[a.n_seqs + seq];
  if (count <= 0) return;
  const bool fresh = a.seqs[2 * a.n_seqs + seq] == 0;
  const int64_t slot_h =
      int64_t(a.seqs[3 * a.n_seqs + seq]) * a.heads + h;
  float* state = a.state + slot_h * a.dim * a.vpad;
  float m = 0.f;
  if constexpr (MAX) m = fresh ? 0.f : a.m[slot_h];

  f32x4_t S[MD][VT];
#pragma unroll
  for (int i = 0; i < MD; ++i)
#pragma unroll
    for (int nt = 0; nt < VT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (i * 4 + w) * 16 + g * 4 + r;
        const int c = v0 + nt * 16 + lr;
        S[i][nt][r] = (!fresh && d < a.dim && c < a.cols)
                          ? state[int64_t(d) * a.vpad + c] : 0.f;
      }

  // A chunk's operands are loaded into registers as soon as those of the
  // chunk before it are used up, and not touched before they are needed.
  constexpr int NQ = 4 * MD, NV = VT, VQ = VS / 4;
  const int trow = w * 16 + lr;
  const int last = first + count - 1;
  const int row_first = a.tiles[first];
  const int n_last = a.tiles[2 * a.n_tiles + last];
  Raw4<QE> qr[NQ];
  Raw4<KE> kr[MD][4];
  f32x4_t ar[4], wr[DELTA ? NQ : 1], ur[DELTA ? VT : 1];
  Raw4<T> vr[DELTA ? 1 : NV];             // four columns of a row
  // row factors: of four output rows, of this lane's operand row, of the
  // staged value rows, of the chunk
  f32x4_t f_row, f_key;
  float f_lane = 0.f, av[MAX ? NV : 1], F_row = 0.f, F_end = 0.f, end = 0.f;
  const T* vb = reinterpret_cast<const T*>(a.v) + h * a.vdim;
  const int hk = h / a.group, kv_heads = a.heads / a.group;
  auto row_of = [&](int t) { return row_first + (t - first) * C; };
  auto rows_of = [&](int t) { return t == last ? n_last : C; };
  auto chunk = [&](int t) { return int64_t(t) * a.heads + h; };
  auto load_q = [&](int t) {
    if constexpr (RAW) {
      const T* q = reinterpret_cast<const T*>(a.q) +
                   int64_t(row_of(t) + trow) * a.q_stride + hk * a.dim;
      const bool ok = trow < rows_of(t);
      if constexpr (FULL) q -= int64_t(ok ? 0 : trow - n_last + 1) * a.q_stride;
#pragma unroll
      for (int i = 0; i < NQ; ++i) {
        if constexpr (FULL) qr[i].load(q + i * 16 + g * 4);
        else if (i < ndt)
          qr[i] = raw_guard(q, i * 16 + g * 4, a.dim, ok, vec_q);
      }
    } else {
      const float* qd = a.qd + chunk(t) * C * DP + trow * DP + g * 4;
#pragma unroll
      for (int i = 0; i < NQ; ++i)
        if (i < ndt) qr[i].load(qd + i * 16);
    }
    if constexpr (DELTA) {
      const float* wp = a.w + chunk(t) * C * DP + trow * DP + g * 4;
#pragma unroll
      for (int i = 0; i < NQ; ++i)
        if (i < ndt) wr[i] = *reinterpret_cast<const f32x4_t*>(wp + i * 16);
    }
  };
  auto load_a = [&](int t) {
    const float* sc = a.sc + chunk(t) * C * C + trow * C + g * 4;
#pragma unroll
    for (int J = 0; J < 4; ++J)            // (blocks behind w: not used)
      ar[J] = *reinterpret_cast<const f32x4_t*>(sc + min(J, w) * 16);
  };
  auto load_v = [&](int t) {
    const float* rf = a.rows + chunk(t) * 3 * C;
    if constexpr (DELTA) {
      const float* ub =
          a.ub + (chunk(t) * C + w * 16 + g * 4) * a.ubp + v0 + lr;
#pragma unroll
      for (int nt = 0; nt < VT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          ur[nt][r] = v0 + nt * 16 < a.ubp ? ub[r * a.ubp + nt * 16] : 0.f;
    } else {
      const int row0 = row_of(t), n = rows_of(t);
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int e = i * 256 + threadIdx.x;
        const int r = e / VQ, c = v0 + e % VQ * 4;
        if constexpr (FULL)
          vr[i].load(vb + int64_t(row0 + min(r, n - 1)) * a.v_stride +
                     (c < a.vdim ? c : 0));
        else
          vr[i] = raw_guard(vb + int64_t(row0 + r) * a.v_stride, c, a.vdim,
                            r < n, vec_v);
        if constexpr (MAX) av[i] = rf[C + r];
      }
    }
  };
  auto load_rows = [&](int t) {
    const float* rf = a.rows + chunk(t) * 3 * C;
    if constexpr (DELTA) {
      f_row = *reinterpret_cast<const f32x4_t*>(rf + w * 16 + g * 4);
      f_key = *reinterpret_cast<const f32x4_t*>(rf + C + w * 16 + g * 4);
      end = a.dec[chunk(t)];
    }
    if constexpr (MAX) {
      f_row = *reinterpret_cast<const f32x4_t*>(rf + 2 * C + w * 16 + g * 4);
      f_lane = rf[2 * C + trow];
      F_row = rf[trow];
      F_end = rf[C - 1];
      end = rf[3 * C - 1];
    }
  };
  auto load_k = [&](int t) {
    const KE* kt = reinterpret_cast<const KE*>(a.kt) +
                   (int64_t(t) * kv_heads + hk) * DP * C;
#pragma unroll
    for (int i = 0; i < MD; ++i)
      if (FULL || i * 4 + w < ndt)
#pragma unroll
        for (int s = 0; s < 4; ++s)
          kr[i][s].load(kt + ((i * 4 + w) * 16 + lr) * C + s * 16 + g * 4);
  };
  load_v(first);
  load_rows(first);
  load_q(first);
  load_a(first);
  load_k(first);
  for (int t = first; t <= last; ++t) {
    const int next = min(t + 1, last);     // (no load is conditional)
    const int row0 = row_of(t), n = rows_of(t);
    f32x4_t dv[RAW ? 1 : MD];
    float keep = 1.f;
    if constexpr (!RAW) {
      const float* dec = a.dec + chunk(t) * DP;
#pragma unroll
      for (int i = 0; i < MD; ++i)
        if (FULL || i * 4 + w < ndt)
          dv[i] = *reinterpret_cast<const f32x4_t*>(
              dec + (i * 4 + w) * 16 + g * 4);
    }
    f32x4_t f_out = f_row, f_k = f_key;
    float f_a = 1.f, M_end = 0.f;
    if constexpr (DELTA) keep = end;
    if constexpr (MAX) {
      M_end = fmaxf(m, end);
      keep = gexp<T>(m - M_end);
      a.mrow[int64_t(trow < n ? row0 + trow : a.n_rows + trow) * a.heads + h] =
          F_row + fmaxf(m, f_lane);       // (every slice, the same value)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        f_out[r] = a.qscale * gexp<T>(m - fmaxf(m, f_row[r]));
      f_a = gexp<T>(f_lane - fmaxf(m, f_lane));
      m = F_end + M_end;
    }
#pragma unroll
    for (int i = 0; i < MD; ++i)
      if (FULL || i * 4 + w < ndt)
#pragma unroll
        for (int nt = 0; nt < VT; ++nt)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            Sl[((i * 4 + w) * 16 + g * 4 + r) * SR + nt * 16 + lr] =
                S[i][nt][r];
    if constexpr (!DELTA) {
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        const int e = i * 256 + threadIdx.x;
        const int r = e / VQ, c = e % VQ * 4;
        f32x4_t v;
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          v[k] = vr[i].get(k);
          if constexpr (MAX)              // the normalizer's column of ones
            if (v0 + c + k >= a.vdim) v[k] = v0 + c + k == a.vdim ? 1.f : 0.f;
          if (r >= n) v[k] = 0.f;
        }
        *reinterpret_cast<f32x4_t*>(Vl + r * SR + c) = v;
        if constexpr (MAX)
          *reinterpret_cast<f32x4_t*>(Vk + r * SR + c) =
              v * gexp<T>(av[i] - M_end);
      }
      load_v(next);
    }
    load_rows(next);
    __syncthreads();
    f32x4_t o[VT], x[DELTA ? VT : 1];
#pragma unroll
    for (int nt = 0; nt < VT; ++nt) {
      o[nt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if constexpr (DELTA) x[nt] = o[nt];
    }
    // LDS operands are asked for in batches ahead of the products
    constexpr int GI = NQ < 8 / VT ? NQ : 8 / VT;
#pragma unroll
    for (int i0 = 0; i0 < NQ; i0 += GI) {
      float s[GI][4][VT];
#pragma unroll
      for (int i = 0; i < GI; ++i)
        if (FULL || i0 + i < ndt)
#pragma unroll
          for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int nt = 0; nt < VT; ++nt)
              s[i][j][nt] =
                  Sl[((i0 + i) * 16 + g * 4 + j) * SR + nt * 16 + lr];
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int i = 0; i < GI; ++i)
        if (FULL || i0 + i < ndt)
#pragma unroll
          for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int nt = 0; nt < VT; ++nt) {
              o[nt] = mma4(qr[i0 + i].get(j), s[i][j][nt], o[nt]);
              if constexpr (DELTA)
                x[nt] = mma4(wr[i0 + i][j], s[i][j][nt], x[nt]);
            }
    }
    load_q(next);
    if constexpr (RAW)
#pragma unroll
      for (int nt = 0; nt < VT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[nt][r] *= f_out[r];
    if constexpr (DELTA) {
#pragma unroll
      for (int nt = 0; nt < VT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int at = (w * 16 + g * 4 + r) * SR + nt * 16 + lr;
          const float u = ur[nt][r] - x[nt][r];
          Vl[at] = u;
          Vk[at] = u * f_k[r];
        }
      load_v(next);
      __syncthreads();
    }
    float vv[16][VT];
    auto values = [&](const float* from) {
#pragma unroll
      for (int k = 0; k < 16; ++k)
#pragma unroll
        for (int nt = 0; nt < VT; ++nt)
          vv[k][nt] =
              from[(k / 4 * 16 + g * 4 + k % 4) * SR + nt * 16 + lr];
      __builtin_amdgcn_sched_barrier(0);
    };
    values(Vl);
#pragma unroll
    for (int k = 0; k < 16; ++k) {         // (the last wave needs all four)
      const float e = ar[k / 4][k % 4];
      const float p = k / 4 > w ? 0.f : MAX ? e * f_a : e;
#pragma unroll
      for (int nt = 0; nt < VT; ++nt) o[nt] = mma4(p, vv[k][nt], o[nt]);
    }
    load_a(next);
    if constexpr (RAW) values(Vk);
#pragma unroll
    for (int nt = 0; nt < VT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tr = w * 16 + g * 4 + r, c = v0 + nt * 16 + lr;
        const bool ok = tr < n && (!(MAX || !FULL) || c < a.cols);
        a.o[(int64_t(ok ? row0 + tr : a.n_rows + tr) * a.heads + h) * a.opad +
            (ok ? c : 0)] = o[nt][r];
      }
#pragma unroll
    for (int i = 0; i < MD; ++i) {
      if (!FULL && i * 4 + w >= ndt) continue;
#pragma unroll
      for (int nt = 0; nt < VT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          S[i][nt][r] *= RAW ? keep : dv[RAW ? 0 : i][r];
#pragma unroll
      for (int k = 0; k < 16; ++k)
#pragma unroll
        for (int nt = 0; nt < VT; ++nt)
          S[i][nt] = mma4(kr[i][k / 4].get(k % 4), vv[k][nt], S[i][nt]);
    }
    load_k(next);
    // (delta: the next chunk's first barrier comes before its first write
    // to the value tiles, and Sl was last read before the second)
    if constexpr (!DELTA) __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < MD; ++i)
#pragma unroll
    for (int nt = 0; nt < VT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (i * 4 + w) * 16 + g * 4 + r;
        const int c = v0 + nt * 16 + lr;
        if (d < a.dim && c < a.cols) state[int64_t(d) * a.vpad + c] = S[i][nt][r];
      }
  // other slices of this head may yet read the old maximum: it returns to
  // its slot in the launch that follows
  if constexpr (MAX)
    if (blockIdx.y == 0 && threadIdx.x == 0)
      a.m_new[int64_t(seq) * a.heads + h] = m;
}

template <typename T, int MODE, int VT>
void scan_md(const ScanArgs& a, hipStream_t st) {
  constexpr int VS = VT * 16;
  const size_t smem = size_t(a.dpad + (MODE == kScanPlain ? 1 : 2) * C) *
                      (VS + 4) * sizeof(float);
  auto aligned = [](const void* p, int64_t stride, int width) {
    return stride % 4 == 0 && width % 4 == 0 &&
           reinterpret_cast<uintptr_t>(p) % (4 * sizeof(T)) == 0;
  };
  const bool vec_q = aligned(a.q, a.q_stride, a.dim);
  const bool vec_v = aligned(a.v, a.v_stride, a.vdim);
  auto run = [&](auto* k) {
    if (smem > 65536)
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                                hipFuncAttributeMaxDynamicSharedMemorySize,
                                int(smem));
    hipLaunchKernelGGL(k, dim3(a.n_seqs * a.heads, (a.cols + VS - 1) / VS),
                       dim3(256), smem, st, a, vec_q, vec_v);
  };
  const bool full = (a.dim == 64 || a.dim == 128) && a.vdim % VS == 0 &&
                    (MODE == kScanPlain || vec_q) &&
                    (MODE == kScanDelta || vec_v);
  if constexpr (sizeof(T) == 2) {
    if (full) {
      if (a.dim == 64) run(rec_scan_kernel<T, MODE, VT, 1, true>);
      else run(rec_scan_kernel<T, MODE, VT, 2, true>);
      return;
    }
  }
  if (a.dpad <= 64) run(rec_scan_kernel<T, MODE, VT, 1, false>);
  else if (a.dpad <= 128) run(rec_scan_kernel<T, MODE, VT, 2, false>);
  else run(rec_scan_kernel<T, MODE, VT, 4, false>);
}

template <typename T, int MODE>
void scan(const ScanArgs& a, hipStream_t st) {
  // a scan step is latency-bound: narrow value slices, several
  // workgroups per CU, until there are plenty anyway
  const int64_t sh = int64_t(a.n_seqs) * a.heads;
  if (a.vdim > 32 && sh * ((a.vdim + 63) / 64) >= 512)
    scan_md<T, MODE, 4>(a, st);
  else if (a.vdim > 16 && sh * ((a.vdim + 31) / 32) >= 1024)
    scan_md<T, MODE, 2>(a, st);
  else
    scan_md<T, MODE, 1>(a, st);
}

// GL lanes per (row, head); V4 float4 columns per lane when the width and
// its offsets allow vectors (V4 = 0: one column at a time)
template <typename T, int KIND, int V4, int GL>
__global__ __launch_bounds__(256)
void rec_gate_kernel(RecGateArgs a) {
  if (a.m_new) {                          // (a few values, any thread)
    const int64_t i = int64_t(blockIdx.x) * 256 + threadIdx.x;
    if (i < int64_t(a.n_seqs) * a.heads)
      a.m[int64_t(a.seqs[3 * a.n_seqs + i / a.heads]) * a.heads +
          i % a.heads] = a.m_new[i];
  }
  const int lane = threadIdx.x % GL;
  const int64_t rh = int64_t(blockIdx.x) * (256 / GL) + threadIdx.x / GL;
  if (rh >= int64_t(a.rows) * a.heads) return;
  const int64_t row = rh / a.heads;
  const int h = int(rh % a.heads);
  const float* o = a.o + rh * a.opad;
  const T* gate = reinterpret_cast<const T*>(a.gate) + row * a.gate_stride +
                  h * a.vdim;
  const float* norm = a.norm + h * a.norm_stride;
  T* out = reinterpret_cast<T*>(a.out) + row * a.out_stride + h * a.vdim;
  float pre = 1.f;
  if (a.mrow)
    pre = 1.f / (fmaxf(fabsf(o[a.vdim]), gexp<T>(-a.mrow[rh])) + 1e-6f);
  auto gated = [](float r, float g) {
    return KIND == kGateSilu ? r * (g / (1.f + gexp<T>(-g)))
                             : r / (1.f + gexp<T>(-g));
  };
  float ss = 0.f;
  if constexpr (V4 > 0) {
    f32x4_t ov[V4], gv[V4];
#pragma unroll
    for (int i = 0; i < V4; ++i) {
      const int c = (i * GL + lane) * 4;
      ov[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (c < a.vdim) {
        ov[i] = *reinterpret_cast<const f32x4_t*>(o + c);
        if constexpr (KIND != kGateNone) gv[i] = act_load4(gate + c);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        ov[i][j] *= pre;
        ss += ov[i][j] * ov[i][j];
      }
    }
    const float inv = 1.f / sqrtf(group_sum<GL>(ss) / a.vdim + a.eps);
#pragma unroll
    for (int i = 0; i < V4; ++i) {
      const int c = (i * GL + lane) * 4;
      if (c >= a.vdim) break;
      const f32x4_t nv = *reinterpret_cast<const f32x4_t*>(norm + c);
      f32x4_t r;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        r[j] = ov[i][j] * inv * nv[j];
        if constexpr (KIND != kGateNone) r[j] = gated(r[j], gv[i][j]);
      }
      act_store4(out + c, r);
    }
  } else {
    for (int e = lane; e < a.vdim; e += GL) ss += o[e] * o[e] * pre * pre;
    const float inv = pre / sqrtf(group_sum<GL>(ss) / a.vdim + a.eps);
    for (int e = lane; e < a.vdim; e += GL) {
      float r = o[e] * inv * norm[e];
      if constexpr (KIND != kGateNone) r = gated(r, act_load(gate + e));
      act_store(out + e, r);
    }
  }
}

template <typename T, int KIND>
void gate(const RecGateArgs& a, hipStream_t st) {
  auto go = [&](auto* kg, int per_wg = 4) {
    const int64_t rh = int64_t(a.rows) * a.heads;
    hipLaunchKernelGGL(kg, dim3(uint32_t((rh + per_wg - 1) / per_wg)),
                       dim3(256), 0, st, a);
  };
  const bool vec_g =
      KIND == kGateNone ||
      (a.gate_stride % 4 == 0 &&
       reinterpret_cast<uintptr_t>(a.gate) % (4 * sizeof(T)) == 0);
  if (a.vdim % 4 || a.opad % 4 || !vec_g || a.out_stride % 4 ||
      reinterpret_cast<uintptr_t>(a.out) % 16)
    go(rec_gate_kernel<T, KIND, 0, 64>);
  else if (a.vdim <= 64)
    go(rec_gate_kernel<T, KIND, 1, 16>, 16);
  else if (a.vdim <= 128)
    go(rec_gate_kernel<T, KIND, 1, 32>, 8);
  else if (a.vdim <= 256)
    go(rec_gate_kernel<T, KIND, 1, 64>);
  else
    go(rec_gate_kernel<T, KIND, 4, 64>);
}

}  // namespace

void launch_rec_scan(const ScanArgs& a, hipStream_t st) {
  if (a.n_seqs == 0) return;
  auto go = [&](auto t) {
    using T = decltype(t);
    if (a.mode == kScanMax) scan<T, kScanMax>(a, st);
    else if (a.mode == kScanDelta) scan<T, kScanDelta>(a, st);
    else scan<T, kScanPlain>(a, st);
  };
  if (a.f32) go(float{});
  else go(uint16_t{});
}

void launch_rec_gate(const RecGateArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  auto go = [&](auto t) {
    using T = decltype(t);
    if (a.kind == kGateSilu) gate<T, kGateSilu>(a, st);
    else if (a.kind == kGateSigmoid) gate<T, kGateSigmoid>(a, st);
    else gate<T, kGateNone>(a, st);
  };
  if (a.f32) go(float{});
  else go(uint16_t{});
}

}  // namespace rlli
