// mLSTM: per head, with log gates i_t = cap tanh(z_i / cap) and
// f_t = log sigmoid(cap tanh(z_f / cap)) and a running maximum m from 0,
//     m' = max(f + m, i),  S <- e^{f+m-m'} S + e^{i-m'} k v^T,  n likewise,
//     o = S^T q / (max(|n . q|, e^{-m'}) + 1e-6)
// then RMS norm over the value width and a sigmoid gate.  The normalizer n
// is one more value column, of ones.
//
// Decode is one kernel per layer.  Prompts: per (chunk, head) the products
// q_t . k_s (as they are: 16-bit products are exact in f32 accumulators) and
// their decays relative to the chunk's own running maximum; the scan and the
// gate of rec_scan.hip do the rest.

#include "rec_math.h"

namespace rlli {
namespace {

constexpr int C = kRecChunk;
constexpr float kNoGate = -1e30f;

DEV_INLINE float soft_cap(float x, float cap) {
  return cap * tanhf(x / cap);
}

// NT threads: many when there are few heads to fill the chip with
template <typename T, int NT>
__global__ __launch_bounds__(NT)
void mlstm_decode_kernel(MlstmArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seq = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  float* qs = sm;                         // [dim]
  float* ks = qs + a.dpad;                // [dim]
  float* red = ks + a.dpad;               // [rows][vpad] then sums
  const T* row = reinterpret_cast<const T*>(a.proj) + int64_t(seq) * a.stride;
  const bool fresh = a.positions[seq] == 0;
  const int64_t slot_h = int64_t(a.slots[seq]) * a.heads + h;
  const float i =
      soft_cap(act_load(row + a.off_i + h) + a.i_bias[h], a.cap);
  const float f = log_sigmoid<float>(
      soft_cap(act_load(row + a.off_f + h) + a.f_bias[h], a.cap));
  const float fm = f + (fresh ? 0.f : a.m[slot_h]);
  const float m = fmaxf(fm, i);
  const float keep = expf(fm - m), take = expf(i - m);
  const float qscale = 1.f / sqrtf(float(a.dim));
  for (int d = tid; d < a.dim; d += NT) {
    qs[d] = act_load(row + h * a.dim + d) * qscale;
    ks[d] = act_load(row + a.off_k + h * a.dim + d) * take;
  }
  const int v4n = a.vpad / 4, n_rows = NT / v4n;
  const int vr = tid / v4n, vc = tid % v4n;
  const bool live = vr < n_rows;
  f32x4_t v = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int c = vc * 4 + j;
    if (c < a.vdim) v[j] = act_load(row + a.off_v + h * a.vdim + c);
    else if (c == a.vdim) v[j] = 1.f;
  }
  __syncthreads();
  if (tid == 0) a.m[slot_h] = m;
  float* S = a.state + slot_h * a.dim * a.vpad + vc * 4;
  f32x4_t o = f32x4_t{0.f, 0.f, 0.f, 0.f};
  if (live) {
    constexpr int U = 8;
    for (int d0 = vr; d0 < a.dim; d0 += U * n_rows) {
      f32x4_t s[U];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int d = d0 + u * n_rows;
        s[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
        if (d < a.dim && !fresh)
          s[u] = *reinterpret_cast<const f32x4_t*>(S + int64_t(d) * a.vpad);
      }
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int d = d0 + u * n_rows;
        if (d >= a.dim) break;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          s[u][j] = keep * s[u][j] + ks[d] * v[j];
          o[j] += qs[d] * s[u][j];
        }
        *reinterpret_cast<f32x4_t*>(S + int64_t(d) * a.vpad) = s[u];
      }
    }
    *reinterpret_cast<f32x4_t*>(red + vr * a.vpad + vc * 4) = o;
  }
  __syncthreads();
  float nq = 0.f;                         // every thread, for the divisor
  for (int r = 0; r < n_rows; ++r) nq += red[r * a.vpad + a.vdim];
  const float pre = 1.f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
  float ss = 0.f;
  for (int e = tid; e < a.vdim; e += NT) {
    float t = 0.f;
    for (int r = 0; r < n_rows; ++r) t += red[r * a.vpad + e];
    t *= pre;
    red[e] = t;                           // column e is this thread's alone
    ss += t * t;
  }
  __shared__ float ws[NT / 64];
  ss = wave_sum(ss);
  if ((tid & 63) == 0) ws[tid >> 6] = ss;
  __syncthreads();
  ss = 0.f;
#pragma unroll
  for (int k = 0; k < NT / 64; ++k) ss += ws[k];
  const float inv = 1.f / sqrtf(ss / a.vdim + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + int64_t(seq) * a.out_stride +
           h * a.vdim;
  for (int e = tid; e < a.vdim; e += NT)
    act_store(out + e, red[e] * inv * a.norm[h * a.vdim + e] *
                           sigm<T>(act_load(row + a.off_g + h * a.vdim + e)));
}

template <typename T, bool VEC>
__global__ __launch_bounds__(256)
void mlstm_intra_kernel(MlstmArgs a) {
  __shared__ float A[C], M[C];            // a = i - F and its running maximum
  const int tile = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lr = lane & 15, g = lane >> 4;
  const int row0 = a.tiles[tile], n = a.tiles[2 * a.n_tiles + tile];
  const T* qb = reinterpret_cast<const T*>(a.proj) +
                int64_t(row0) * a.stride + h * a.dim;
  const T* kb = qb + a.off_k;
  const int64_t ch = int64_t(tile) * a.heads + h;
  f32x4_t qk[4];
#pragma unroll
  for (int J = 0; J < 4; ++J) qk[J] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int d0 = 0; d0 < a.dim; d0 += 32) {
    const int d = d0 + g * 8;             // rows behind the last repeat it
    const auto qf = frag_at<VEC>(qb + min(w * 16 + lr, n - 1) * a.stride, d,
                                 a.dim);
    Frag8<T> kf[4];
#pragma unroll
    for (int J = 0; J < 4; ++J)
      kf[J] = frag_at<VEC>(kb + min(min(J, w) * 16 + lr, n - 1) * a.stride, d,
                           a.dim);
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J <= w) qk[J] = Frag8<T>::mma(qf, kf[J], qk[J]);
  }
  if (tid < C) {
    float f = 0.f, i = kNoGate;
    if (tid < n) {
      const T* row = reinterpret_cast<const T*>(a.proj) +
                     int64_t(row0 + tid) * a.stride;
      i = soft_cap(act_load(row + a.off_i + h) + a.i_bias[h], a.cap);
      f = log_sigmoid<float>(
          soft_cap(act_load(row + a.off_f + h) + a.f_bias[h], a.cap));
    }
    const float F = wave_prefix_sum(f);
    const float av = tid < n ? i - F : kNoGate;
    const float mv = wave_prefix_max(av);
    A[tid] = av;
    M[tid] = mv;
    float* rf = a.row_f + ch * 3 * C;
    rf[tid] = F;
    rf[C + tid] = av;
    rf[2 * C + tid] = mv;
  }
  keys_down<VEC>(kb, a.stride, n, a.dim, a.dpad,
                 reinterpret_cast<T*>(a.kt) + ch * a.dpad * C);
  __syncthreads();
  const float qscale = 1.f / sqrtf(float(a.dim));
  float* sc = a.sc + ch * C * C;
#pragma unroll
  for (int J = 0; J < 4; ++J) {
    if (J > w) break;
    const int s = J * 16 + lr;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = w * 16 + g * 4 + r;
      sc[t * C + s] =
          s <= t ? qk[J][r] * qscale * gexp<T>(fminf(A[s] - M[t], 0.f)) : 0.f;
    }
  }
}

template <typename T>
void prefill(const MlstmArgs& a, hipStream_t st) {
  const T* p = reinterpret_cast<const T*>(a.proj);
  const bool vec = a.dim % 8 == 0 && a.stride % 8 == 0 && a.off_k % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(p) % 16 == 0;
  auto intra = [&](auto* k) {
    hipLaunchKernelGGL(k, dim3(a.n_tiles, a.heads), dim3(256), 0, st, a);
  };
  if (vec) intra(mlstm_intra_kernel<T, true>);
  else intra(mlstm_intra_kernel<T, false>);
  ScanArgs sa{};
  sa.v = p + a.off_v;
  sa.v_stride = a.stride;
  sa.q = p;
  sa.q_stride = a.stride;
  sa.kt = a.kt;
  sa.sc = a.sc;
  sa.rows = a.row_f;
  sa.state = a.state;
  sa.m = a.m;
  sa.m_new = a.m_new;
  sa.o = a.o;
  sa.mrow = a.mrow;
  sa.tiles = a.tiles;
  sa.seqs = a.seqs;
  sa.n_rows = a.rows;
  sa.n_tiles = a.n_tiles;
  sa.n_seqs = a.n_seqs;
  sa.heads = a.heads;
  sa.group = 1;
  sa.dim = a.dim;
  sa.dpad = a.dpad;
  sa.vdim = a.vdim;
  sa.cols = a.vdim + 1;
  sa.vpad = a.vpad;
  sa.opad = a.opad;
  sa.qscale = 1.f / sqrtf(float(a.dim));
  sa.mode = kScanMax;
  sa.f32 = a.f32;
  launch_rec_scan(sa, st);
  RecGateArgs ga{};
  ga.o = a.o;
  ga.mrow = a.mrow;
  ga.gate = p + a.off_g;
  ga.gate_stride = a.stride;
  ga.norm = a.norm;
  ga.norm_stride = a.vdim;
  ga.out = a.out;
  ga.out_stride = a.out_stride;
  ga.m_new = a.m_new;
  ga.m = a.m;
  ga.seqs = a.seqs;
  ga.n_seqs = a.n_seqs;
  ga.rows = a.rows;
  ga.heads = a.heads;
  ga.vdim = a.vdim;
  ga.opad = a.opad;
  ga.kind = kGateSigmoid;
  ga.eps = a.eps;
  ga.f32 = a.f32;
  launch_rec_gate(ga, st);
}

}  // namespace

void launch_mlstm_decode(const MlstmArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  auto go = [&](auto* k, int nt) {
    const int n_rows = nt / (a.vpad / 4);
    const size_t smem = size_t(2 * a.dpad + n_rows * a.vpad) * sizeof(float);
    hipLaunchKernelGGL(k, dim3(a.rows, a.heads), dim3(nt), smem, st, a);
  };
  const bool few = int64_t(a.rows) * a.heads < 256;
  if (a.f32) {
    go(mlstm_decode_kernel<float, 256>, 256);
  } else if (few) {
    go(mlstm_decode_kernel<uint16_t, 1024>, 1024);
  } else {
    go(mlstm_decode_kernel<uint16_t, 256>, 256);
  }
}

void launch_mlstm_prefill(const MlstmArgs& a, hipStream_t st) {
  if (a.rows == 0 || a.n_seqs == 0) return;
  if (a.f32) prefill<float>(a, st);
  else prefill<uint16_t>(a, st);
}

}  // namespace rlli
