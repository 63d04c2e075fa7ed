// Gated delta rule: per head, with one decay g_t and unit keys,
//     S <- g_t S,  u_t = beta_t (v_t - S^T k_t),  S <- S + k_t u_t^T,
//     o_t = S^T q_t
// then RMS norm over the value width and a silu gate.  q, k, v went through
// a short causal convolution and silu; query/key heads may serve several
// value heads.
//
// Decode is one kernel per layer, the convolution and its ring included.
// S^T k and S^T q are formed in one pass over the state,
//     o = g S^T q + (q . k) u,
// and the new state is written from the registers that hold the old one.
// The ring has at least one row more than the convolution looks back, so
// that heads which share a key head never read the row another one writes.
//
// Prompts, per (chunk, head), with G the running log-decay in the chunk:
//     T[t,s] = beta_t k_t.k_s e^{G_t - G_s} (s < t)
//     (I + T) [Ub | W] = [beta v | beta e^{G} k]
//     A[t,s] = q_t.k_s e^{G_t - G_s} (s <= t)
// so that U = Ub - W S with the state S at the chunk's start; rec_scan.hip
// does the rest.  Dot products run on the convolved rows as they are (16-bit
// products are exact in f32 accumulators), their norms and decays are
// factors.  The triangular system is solved by blocks of 16 rows: diagonal
// blocks are inverted in registers, and solved blocks serve as the next
// product's operand straight from the accumulators.

#include "rec_math.h"

#include <type_traits>

namespace rlli {
namespace {

constexpr int C = kRecChunk;
constexpr int TR = C + 4;
constexpr int DR = 20;

DEV_INLINE float delta_log_decay(float a, float bias, float rate) {
  return fmaxf(-rate * softplus(a + bias), -80.f);
}

// REG: a thread's part of the state fits its registers
// (U rows); NT threads: many when there are few heads to fill the chip with
template <typename T, bool REG, int NT, int U>
__global__ __launch_bounds__(NT)
void delta_decode_kernel(DeltaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seq = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int group = a.heads / a.kv_heads, kvh = h / group;
  const int v4n = a.vpad / 4, n_rows = NT / v4n;
  float* qs = sm;                         // [dim]
  float* ks = qs + a.dpad;                // [dim]
  float* vs = ks + a.dpad;                // [vdim]
  float* rk = vs + a.vpad;                // [n_rows][vpad] S^T k, then u
  float* rq = rk + n_rows * a.vpad;       // [n_rows][vpad] S^T q, then o
  const T* row = reinterpret_cast<const T*>(a.proj) + int64_t(seq) * a.stride;
  const int pos = a.positions[seq];
  const int slot = a.slots[seq];
  const bool fresh = pos == 0;
  float* S = a.state + (int64_t(slot) * a.heads + h) * a.dim * a.vpad;
  const int vr = tid / v4n, vc = tid % v4n;
  const bool live = vr < n_rows;
  f32x4_t s[REG ? U : 1];
  auto load_s = [&](int d) {
    return fresh || d >= a.dim || !live
               ? f32x4_t{0.f, 0.f, 0.f, 0.f}
               : *reinterpret_cast<const f32x4_t*>(
                     S + int64_t(d) * a.vpad + vc * 4);
  };
  if constexpr (REG)
#pragma unroll
    for (int u = 0; u < U; ++u) s[u] = load_s(vr + u * n_rows);

  const int back = a.n_taps - 1, CH = a.channels;
  T* ring = reinterpret_cast<T*>(a.tail) + int64_t(slot) * a.ring * CH;
  for (int e = tid; e < 2 * a.dim + a.vdim; e += NT) {
    const int part = e < a.dim ? 0 : e < 2 * a.dim ? 1 : 2;
    const int c = part == 0 ? kvh * a.dim + e
                  : part == 1
                      ? (a.kv_heads + kvh) * a.dim + e - a.dim
                      : 2 * a.kv_heads * a.dim + h * a.vdim + e - 2 * a.dim;
    const T x0 = row[c];
    float y = a.taps[int64_t(back) * CH + c] * act_load(&x0);
    for (int k = 1; k <= back && k <= pos; ++k)
      y += a.taps[int64_t(back - k) * CH + c] *
           act_load(ring + int64_t((pos - k) % a.ring) * CH + c);
    if (back > 0 && (part == 2 || h % group == 0))
      ring[int64_t(pos % a.ring) * CH + c] = x0;
    sm[part == 0   ? e
       : part == 1 ? a.dpad + e - a.dim
                   : 2 * a.dpad + e - 2 * a.dim] = round_act(T{}, silu<T>(y));
  }
  for (int e = a.vdim + tid; e < a.vpad; e += NT) vs[e] = 0.f;
  __syncthreads();
  float qq = 0.f, kk = 0.f, qk = 0.f;
  for (int d = tid; d < a.dim; d += NT) {
    qq += qs[d] * qs[d];
    kk += ks[d] * ks[d];
    qk += qs[d] * ks[d];
  }
  __shared__ float part[4][NT / 64];
  qq = wave_sum(qq);
  kk = wave_sum(kk);
  qk = wave_sum(qk);
  if ((tid & 63) == 0) {
    part[0][tid >> 6] = qq;
    part[1][tid >> 6] = kk;
    part[2][tid >> 6] = qk;
  }
  const float g = expf(delta_log_decay(act_load(row + a.off_a + h),
                                       a.dt_bias[h], a.a_rate[h]));
  const float beta = 1.f / (1.f + expf(-act_load(row + a.off_b + h)));
  f32x4_t pk = f32x4_t{0.f, 0.f, 0.f, 0.f}, pq = pk;
  auto take = [&](int d, const f32x4_t& sv) {
    const float kd = ks[d], qd = qs[d];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      pk[j] += kd * sv[j];
      pq[j] += qd * sv[j];
    }
  };
  if constexpr (REG) {
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (live && vr + u * n_rows < a.dim) take(vr + u * n_rows, s[u]);
  } else if (live) {
    for (int d = vr; d < a.dim; d += n_rows) take(d, load_s(d));
  }
  if (live) {
    *reinterpret_cast<f32x4_t*>(rk + vr * a.vpad + vc * 4) = pk;
    *reinterpret_cast<f32x4_t*>(rq + vr * a.vpad + vc * 4) = pq;
  }
  __syncthreads();
  auto total = [&](int i) {
    float s = 0.f;
#pragma unroll
    for (int k = 0; k < NT / 64; ++k) s += part[i][k];
    return s;
  };
  const float kn = 1.f / sqrtf(total(1) + 1e-6f);
  const float qn = 1.f / sqrtf(total(0) + 1e-6f) / sqrtf(float(a.dim));
  const float dot = total(2) * qn * kn;
  float ss = 0.f;
  for (int e = tid; e < a.vpad; e += NT) {
    float sk = 0.f, sq = 0.f;
    for (int r = 0; r < n_rows; ++r) {
      sk += rk[r * a.vpad + e];
      sq += rq[r * a.vpad + e];
    }
    const float u = beta * (vs[e] - g * kn * sk);
    const float o = g * qn * sq + dot * u;
    rk[e] = e < a.vdim ? u : 0.f;         // column e is this thread's alone
    rq[e] = o;
    if (e < a.vdim) ss += o * o;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) part[3][tid >> 6] = ss;
  __syncthreads();
  if (live) {
    const f32x4_t u4 = *reinterpret_cast<const f32x4_t*>(rk + vc * 4);
    auto put = [&](int d, const f32x4_t& sv) {
      f32x4_t n;
      const float kd = ks[d] * kn;
#pragma unroll
      for (int j = 0; j < 4; ++j) n[j] = g * sv[j] + kd * u4[j];
      *reinterpret_cast<f32x4_t*>(S + int64_t(d) * a.vpad + vc * 4) = n;
    };
    if constexpr (REG) {
#pragma unroll
      for (int u = 0; u < U; ++u)
        if (vr + u * n_rows < a.dim) put(vr + u * n_rows, s[u]);
    } else {
      for (int d = vr; d < a.dim; d += n_rows) put(d, load_s(d));
    }
  }
  const float inv = 1.f / sqrtf(total(3) / a.vdim + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + int64_t(seq) * a.out_stride +
           h * a.vdim;
  for (int e = tid; e < a.vdim; e += NT)
    act_store(out + e, rq[e] * inv * a.norm[e] *
                           silu<T>(act_load(row + a.off_g + h * a.vdim + e)));
}

// ND: 32-column steps of a key (0: any)
template <typename T, bool VEC, int ND>
__global__ __launch_bounds__(256)
void delta_intra_kernel(DeltaArgs a) {
  __shared__ __attribute__((aligned(16))) float Tm[C * TR];   // [64][TR] below the diagonal
  __shared__ __attribute__((aligned(16))) float Dv[4 * 16 * DR];   // inverted diagonal blocks
  __shared__ float qn[C], kn[C], be[C], G[C];
  const int tile = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int group = a.heads / a.kv_heads, kvh = h / group;
  const int lane = tid & 63;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lr = lane & 15, g = lane >> 4;
  const int row0 = a.tiles[tile], n = a.tiles[2 * a.n_tiles + tile];
  const T* xb = reinterpret_cast<const T*>(a.x) + int64_t(row0) * a.x_stride;
  const T* qb = xb + kvh * a.dim;
  const T* kb = qb + a.kv_heads * a.dim;
  const T* vb = xb + 2 * a.kv_heads * a.dim + h * a.vdim;
  const int64_t ch = int64_t(tile) * a.heads + h;

  // Products of the rows as they are: own rows down, block J's rows across.
  // Rows behind the last one repeat it; their beta is zero.
  f32x4_t qk[4], kk[4];
#pragma unroll
  for (int J = 0; J < 4; ++J) qk[J] = kk[J] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  float sq = 0.f, sk = 0.f;               // squares of row w * 16 + lr
  const int steps = ND > 0 ? ND : (a.dim + 31) / 32;
  constexpr int SU = ND > 0 ? ND : 1;
  for (int st = 0; st < steps; st += SU) {
    Frag8<T> qf[SU], kf[SU][4];
#pragma unroll
    for (int u = 0; u < SU; ++u) {
      const int d = (st + u) * 32 + g * 8;
      qf[u] = frag_at<VEC>(qb + min(w * 16 + lr, n - 1) * a.x_stride, d,
                           a.dim);
#pragma unroll
      for (int J = 0; J < 4; ++J)         // (blocks behind w: not used)
        kf[u][J] = frag_at<VEC>(
            kb + min(min(J, w) * 16 + lr, n - 1) * a.x_stride, d, a.dim);
    }
#pragma unroll
    for (int u = 0; u < SU; ++u) {
      const Frag8<T> own = kf[u][3];      // min(3, w) = w
      sq += frag_sq(qf[u]);
      sk += frag_sq(own);
#pragma unroll
      for (int J = 0; J < 4; ++J)
        if (J <= w) {
          qk[J] = Frag8<T>::mma(qf[u], kf[u][J], qk[J]);
          kk[J] = Frag8<T>::mma(own, kf[u][J], kk[J]);
        }
    }
  }
  sq += __shfl_xor(sq, 16, kWave);
  sk += __shfl_xor(sk, 16, kWave);
  sq += __shfl_xor(sq, 32, kWave);
  sk += __shfl_xor(sk, 32, kWave);
  if (g == 0) {
    qn[w * 16 + lr] = 1.f / sqrtf(sq + 1e-6f) / sqrtf(float(a.dim));
    kn[w * 16 + lr] = 1.f / sqrtf(sk + 1e-6f);
  }
  if (tid < C) {
    float lg = 0.f, b = 0.f;
    if (tid < n) {
      const T* row = reinterpret_cast<const T*>(a.proj) +
                     int64_t(row0 + tid) * a.stride;
      lg = delta_log_decay(act_load(row + a.off_a + h), a.dt_bias[h],
                           a.a_rate[h]);
      b = 1.f / (1.f + expf(-act_load(row + a.off_b + h)));
    }
    G[tid] = wave_prefix_sum(lg);
    be[tid] = b;
  }
  __syncthreads();
  if (tid < C) {
    float* rf = a.row_f + ch * 3 * C;
    rf[tid] = qn[tid] * expf(G[tid]);
    rf[C + tid] = kn[tid] * expf(G[C - 1] - G[tid]);
    if (tid == 0) a.dec[ch] = expf(G[C - 1]);
  }
  float* sc = a.sc + ch * C * C;
#pragma unroll
  for (int J = 0; J < 4; ++J) {
    if (J > w) break;
    const int s = J * 16 + lr;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = w * 16 + g * 4 + r;
      const float e = kn[s] * gexp<T>(fminf(G[t] - G[s], 0.f));
      sc[t * C + s] = s <= t ? qk[J][r] * qn[t] * e : 0.f;
      Tm[t * TR + s] = s < t ? kk[J][r] * be[t] * kn[t] * e : 0.f;
    }
  }
  __syncthreads();
  // (I + T_ww)^-1, one column per lane
  {
    float x[16];
    const float* td = Tm + w * 16 * TR + w * 16;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float v = t == lr ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) v -= td[t * TR + s] * x[s];
      x[t] = v;
      if (g == 0) Dv[(w * 16 + t) * DR + lr] = v;
    }
  }
  if (h % group == 0)
    keys_down<VEC>(kb, a.x_stride, n, a.dim, a.dpad,
                   reinterpret_cast<T*>(a.kt) +
                       (int64_t(tile) * a.kv_heads + kvh) * a.dpad * C);
  __syncthreads();
  f32x4_t tf[6], df[4];                   // blocks 10 20 21 30 31 32
#pragma unroll
  for (int I = 0; I < 4; ++I) {
    df[I] = *reinterpret_cast<const f32x4_t*>(Dv + (I * 16 + lr) * DR + g * 4);
#pragma unroll
    for (int K = 0; K < I; ++K) {
      const f32x4_t v = *reinterpret_cast<const f32x4_t*>(
          Tm + (I * 16 + lr) * TR + K * 16 + g * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) tf[I * (I - 1) / 2 + K][j] = -v[j];
    }
  }
  const int nv = a.ubp / 16, nk = a.dpad / 16;
  for (int ct = w; ct < nv + nk; ct += 4) {
    const bool val = ct < nv;
    const int c = (val ? ct : ct - nv) * 16 + lr;
    // (columns behind the last one meet zeros of the state, or nothing)
    const T* src = (val ? vb : kb) + min(c, (val ? a.vdim : a.dim) - 1);
    T raw[16];
#pragma unroll
    for (int k = 0; k < 16; ++k)
      raw[k] = src[min(k / 4 * 16 + g * 4 + k % 4, n - 1) * a.x_stride];
    f32x4_t u[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      f32x4_t acc;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = I * 16 + g * 4 + r;
        acc[r] = act_load(&raw[I * 4 + r]) * be[t] *
                 (val ? 1.f : kn[t] * gexp<T>(G[t]));
      }
#pragma unroll
      for (int K = 0; K < I; ++K)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc = mma4(tf[I * (I - 1) / 2 + K][j], u[K][j], acc);
      u[I] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < 4; ++j) u[I] = mma4(df[I][j], acc[j], u[I]);
    }
    float* dst = val ? a.ub + ch * C * a.ubp + c : a.w + ch * C * a.dpad + c;
    const int ds = val ? a.ubp : a.dpad;
#pragma unroll
    for (int I = 0; I < 4; ++I)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        dst[(I * 16 + g * 4 + r) * ds] = u[I][r];
  }
}

// VEC and the number of 32-column steps (0: any) of a chunk kernel
template <typename F>
void by_dim(int dim, bool vec, F f) {
  using std::integral_constant;
  if (!vec) f(std::false_type{}, integral_constant<int, 0>{});
  else if (dim == 64) f(std::true_type{}, integral_constant<int, 2>{});
  else if (dim == 128) f(std::true_type{}, integral_constant<int, 4>{});
  else f(std::true_type{}, integral_constant<int, 0>{});
}

template <typename T>
void prefill(const DeltaArgs& a, hipStream_t st) {
  const bool vec = a.dim % 8 == 0 && a.x_stride % 8 == 0 &&
                   reinterpret_cast<uintptr_t>(a.x) % 16 == 0;
  by_dim(a.dim, vec, [&](auto v, auto nd) {
    hipLaunchKernelGGL(
        (delta_intra_kernel<T, decltype(v)::value, decltype(nd)::value>),
        dim3(a.n_tiles, a.heads), dim3(256), 0, st, a);
  });
  ScanArgs sa{};
  sa.q = a.x;
  sa.q_stride = a.x_stride;
  sa.kt = a.kt;
  sa.sc = a.sc;
  sa.dec = a.dec;
  sa.rows = a.row_f;
  sa.w = a.w;
  sa.ub = a.ub;
  sa.state = a.state;
  sa.o = a.o;
  sa.tiles = a.tiles;
  sa.seqs = a.seqs;
  sa.n_rows = a.rows;
  sa.n_tiles = a.n_tiles;
  sa.n_seqs = a.n_seqs;
  sa.heads = a.heads;
  sa.group = a.heads / a.kv_heads;
  sa.dim = a.dim;
  sa.dpad = a.dpad;
  sa.vdim = sa.cols = sa.opad = a.vdim;
  sa.vpad = a.vpad;
  sa.ubp = a.ubp;
  sa.mode = kScanDelta;
  sa.f32 = a.f32;
  launch_rec_scan(sa, st);
  RecGateArgs ga{};
  ga.o = a.o;
  ga.gate = reinterpret_cast<const T*>(a.proj) + a.off_g;
  ga.gate_stride = a.stride;
  ga.norm = a.norm;
  ga.out = a.out;
  ga.out_stride = a.out_stride;
  ga.rows = a.rows;
  ga.heads = a.heads;
  ga.vdim = ga.opad = a.vdim;
  ga.kind = kGateSilu;
  ga.eps = a.eps;
  ga.f32 = a.f32;
  launch_rec_gate(ga, st);
}

}  // namespace

void launch_delta_decode(const DeltaArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  auto go = [&](auto* k, int nt) {
    const int n_rows = nt / (a.vpad / 4);
    const size_t smem =
        size_t(2 * a.dpad + a.vpad + 2 * n_rows * a.vpad) * sizeof(float);
    hipLaunchKernelGGL(k, dim3(a.rows, a.heads), dim3(nt), smem, st, a);
  };
  const bool few = int64_t(a.rows) * a.heads < 256;
  const bool reg = a.dim <= 16 * (256 / (a.vpad / 4));
  if (a.f32) {
    if (reg) go(delta_decode_kernel<float, true, 256, 16>, 256);
    else go(delta_decode_kernel<float, false, 256, 16>, 256);
  } else if (few && a.dim <= 4 * (1024 / (a.vpad / 4))) {
    go(delta_decode_kernel<uint16_t, true, 1024, 4>, 1024);
  } else {
    if (reg) go(delta_decode_kernel<uint16_t, true, 256, 16>, 256);
    else go(delta_decode_kernel<uint16_t, false, 256, 16>, 256);
  }
}

void launch_delta_prefill(const DeltaArgs& a, hipStream_t st) {
  if (a.rows == 0 || a.n_seqs == 0) return;
  if (a.f32) prefill<float>(a, st);
  else prefill<uint16_t>(a, st);
}

}  // namespace rlli
