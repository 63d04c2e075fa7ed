// Gated linear recurrences: S_t = diag(alpha_t) S_{t-1} + k_t v_t^T,
// o_t = S_t^T q_t per head, alpha a decay per key channel, then RMS norm
// over the value width.  Two ways to make q, k and alpha from the
// projections:
//   GLA     q | k | v | gate | A1 h:  alpha = sigmoid(z)^(1/tau) with
//           z = A2 (A1 h) + b, q scaled by dim^-1/2, silu output gate
//   HGRN2   q | z | v:  alpha = l + (1 - l) sigmoid(z + b) with a lower
//           bound l per channel, k = 1 - alpha, q = silu(q), no gate
//
// The projections arrive as one GEMM output row; everything from z on is
// 32-bit, matrix products included (the f32 MFMA forms), and so are the
// states.
//
// Decode is one fused kernel per layer: decay, state update, readout,
// norm and gate; a state is read and written exactly once.
//
// Prompts run in chunks of 64 tokens whose four 16-token sub-chunks bound
// every exponent: with L the running log-decay inside a sub-chunk, tot its
// last row and B_I the running log-decay at the start of sub-chunk I,
//     A[t,s] = sum_d (q_t e^{L_t} e^{B_I - B_{J+1}}) * (k_s e^{tot_J - L_s})
// for J < I has only exponents <= 0, whatever the decay.  Inside a
// sub-chunk the factors are e^{L_t - m} and e^{m - L_s} with m the middle
// row's log-decay, as long as either half decays by less than e^40; beyond
// that four-row blocks do the same once more.
//   gla_intra   per (chunk, head): A, q e^{b_t}, k e^{b_C - b_s}, e^{b_C}
//   gla_scan    per (sequence, head, value slice): chunk after chunk,
//               O = (q e^{b}) S + A V, S = e^{b_C} S + (k e^{b_C-b})^T V,
//               S in MFMA accumulators
//   gla_gate    per (row, head): norm and gate

#include "mix.h"

namespace rlli {
namespace {

constexpr int C = kGlaChunk;
constexpr float kSafeLog = 40.f;

// the hardware exponential is good to a few ulp at these exponents; the
// 32-bit mode takes the exact one
template <typename T> DEV_INLINE float gexp(float x);
template <> DEV_INLINE float gexp<uint16_t>(float x) { return __expf(x); }
template <> DEV_INLINE float gexp<float>(float x) { return expf(x); }

template <typename T>
DEV_INLINE float log_sigmoid(float x) {
  // absolute error is what counts: it enters a sum of logarithms
  if constexpr (sizeof(T) == 2)
    return fminf(x, 0.f) - __logf(1.f + __expf(-fabsf(x)));
  return fminf(x, 0.f) - log1pf(expf(-fabsf(x)));
}

// 1 / x for x >= 1, good to an ulp where activations are 16-bit
template <typename T> DEV_INLINE float grcp(float x);
template <> DEV_INLINE float grcp<uint16_t>(float x) {
  return __builtin_amdgcn_rcpf(x);
}
template <> DEV_INLINE float grcp<float>(float x) { return 1.f / x; }

template <typename T>
DEV_INLINE float silu(float x) {
  // (the exponent is bounded so that the reciprocal stays finite)
  return x * grcp<T>(1.f + gexp<T>(fminf(-x, 80.f)));
}

// HGRN2: alpha = low + (1 - low) sigmoid(z), k = 1 - alpha without the
// cancellation
template <typename T>
DEV_INLINE float forget_key(float z, float low, float* alpha) {
  const float e = gexp<T>(-fabsf(z));
  const float r = grcp<T>(1.f + e), er = e * r;
  *alpha = low + (1.f - low) * (z >= 0.f ? r : er);
  return (1.f - low) * (z >= 0.f ? er : r);
}

// log alpha; e^-80 and less is nothing beside a key of order one
template <typename T>
DEV_INLINE float log_forget(float alpha, float k) {
  if constexpr (sizeof(T) == 2) return fmaxf(__logf(alpha), -80.f);
  return alpha > 0.5f ? log1pf(-k) : fmaxf(logf(alpha), -80.f);
}

// running sum over the 16 lanes of a row
DEV_INLINE float row_prefix(float v) {
  v += dpp_mov_f32<0x111>(v);             // row_shr 1, 2, 4, 8: zeros enter
  v += dpp_mov_f32<0x112>(v);
  v += dpp_mov_f32<0x114>(v);
  v += dpp_mov_f32<0x118>(v);
  return v;
}

DEV_INLINE f32x4_t mma4(float a, float b, f32x4_t c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

template <typename T>
DEV_INLINE f32x4_t load4_guard(const T* p, int d, int dim, bool row_ok,
                               bool vec) {
  f32x4_t v = f32x4_t{0.f, 0.f, 0.f, 0.f};
  if (!row_ok) return v;
  if (vec && d + 4 <= dim) return act_load4(p + d);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (d + j < dim) v[j] = act_load(p + d + j);
  return v;
}

// ------------------------------------------------------------- decode
template <typename T, bool FG>
__global__ __launch_bounds__(256)
void gla_decode_kernel(GlaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seq = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x;
  float* al = sm;                       // [dim]
  float* ks = al + a.dpad;              // [dim]
  float* qs = ks + a.dpad;              // [dim]
  float* a1 = qs + a.dpad;              // [rank, padded to 4]
  float* red = a1 + (a.rank + 3) / 4 * 4;   // [rows][vpad] then sums
  const T* row = reinterpret_cast<const T*>(a.proj) + int64_t(seq) * a.stride;
  const int hv = a.heads * a.vdim;
  if constexpr (FG) {
    for (int d = tid; d < a.dim; d += 256) {
      const int hc = h * a.dim + d;
      qs[d] = silu<T>(act_load(row + hc));
      ks[d] = forget_key<T>(act_load(row + a.off_k + hc) + a.a2_bias[hc],
                            a.lower[hc], al + d);
    }
  } else {
    for (int r = tid; r < a.rank; r += 256) a1[r] = act_load(row + a.off_a + r);
    const float qscale = 1.f / sqrtf(float(a.dim));
    for (int d = tid; d < a.dim; d += 256) {
      qs[d] = act_load(row + h * a.dim + d) * qscale;
      ks[d] = act_load(row + a.off_k + h * a.dim + d);
    }
  }
  const int v4n = a.vpad / 4;
  const int n_rows = 256 / v4n;
  const int vr = tid / v4n, vc = tid % v4n;
  const bool live = vr < n_rows;
  f32x4_t v = f32x4_t{0.f, 0.f, 0.f, 0.f};
  if (live) {
    const T* vp = row + a.off_v + h * a.vdim;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (vc * 4 + j < a.vdim) v[j] = act_load(vp + vc * 4 + j);
  }
  __syncthreads();
  if constexpr (!FG) {
    for (int d = tid; d < a.dim; d += 256) {
      const T* w = reinterpret_cast<const T*>(a.a2) +
                   int64_t(h * a.dim + d) * a.rank;
      float z = a.a2_bias[h * a.dim + d];
      for (int r = 0; r < a.rank; ++r) z += act_load(w + r) * a1[r];
      al[d] = expf(log_sigmoid<T>(z) / a.tau);
    }
    __syncthreads();
  }

  const bool fresh = a.positions[seq] == 0;
  float* S = a.state +
             (int64_t(a.slots[seq]) * a.heads + h) * a.dim * a.vpad + vc * 4;
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
          s[u][j] = al[d] * s[u][j] + ks[d] * v[j];
          o[j] += qs[d] * s[u][j];
        }
        *reinterpret_cast<f32x4_t*>(S + int64_t(d) * a.vpad) = s[u];
      }
    }
    *reinterpret_cast<f32x4_t*>(red + vr * a.vpad + vc * 4) = o;
  }
  __syncthreads();
  float ss = 0.f;
  for (int e = tid; e < a.vdim; e += 256) {
    float t = 0.f;
    for (int r = 0; r < n_rows; ++r) t += red[r * a.vpad + e];
    red[e] = t;                         // column e is this thread's alone
    ss += t * t;
  }
  __shared__ float ws[4];
  ss = wave_sum(ss);
  if ((tid & 63) == 0) ws[tid >> 6] = ss;
  __syncthreads();
  const float inv =
      1.f / sqrtf((ws[0] + ws[1] + ws[2] + ws[3]) / a.vdim + a.eps);
  T* out = reinterpret_cast<T*>(a.out) + int64_t(seq) * a.out_stride +
           h * a.vdim;
  for (int e = tid; e < a.vdim; e += 256) {
    float o2 = red[e] * inv * a.norm[e];
    if constexpr (!FG)
      o2 *= silu<T>(act_load(row + a.off_g + h * a.vdim + e));
    act_store(out + e, o2);
  }
}

// -------------------------------------------------------------- intra
// Wave w owns sub-chunk w, lane l its row l & 15 and four neighbouring key
// columns of every 16; MD bounds the key tiles (dpad <= 64 * MD).
template <typename T, bool FG, int MD>
__global__ __launch_bounds__(256)
void gla_intra_kernel(GlaArgs a, bool vec, bool vec_a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  constexpr int NT = 4 * MD;
  const int tile = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int DP = a.dpad, LR = DP + 4, ndt = DP / 16;
  float* kl = sm;                        // [64][LR] keys, then decayed keys
  float* tot = kl + C * LR;              // [4][DP] log-decays of sub-chunks
  float* EB = tot + 4 * DP;              // [3][DP] e^{B_w}, w = 1 .. 3
  float* ED = EB + 3 * DP;               // [3][DP] e^{B_4 - B_{w+1}}, w < 3
  float* EJ = ED + 3 * DP;               // [3][DP] sub-chunks in between
  const int row0 = a.tiles[tile];
  const int n = a.tiles[2 * a.n_tiles + tile];
  const int trow = w * 16 + lr;          // this lane's row
  const bool row_ok = trow < n;
  const T* qrow = reinterpret_cast<const T*>(a.proj) +
                  int64_t(row0 + trow) * a.stride + h * a.dim;
  const T* krow = qrow + a.off_k;
  const float* bias = a.a2_bias + h * a.dim;
  const float* low = FG ? a.lower + h * a.dim : nullptr;
  const float qscale = 1.f / sqrtf(float(a.dim));

  // queries and the running log-decay stay in registers, keys in LDS
  f32x4_t q[NT], L[NT];
  float wmin = 0.f;
  // (raw keys wait in the registers of the log-decays)
#pragma unroll
  for (int dt = 0; dt < NT; ++dt) {
    if (dt >= ndt) continue;
    const int d = dt * 16 + g * 4;
    q[dt] = load4_guard(qrow, d, a.dim, row_ok, vec);
    L[dt] = load4_guard(krow, d, a.dim, row_ok, vec);
  }
#pragma unroll
  for (int dt = 0; dt < NT; ++dt) {
    if (dt >= ndt) continue;
    const int d = dt * 16 + g * 4;
    f32x4_t k = L[dt];
    const f32x4_t bv = load4_guard(bias, d, a.dim, true, a.dim % 4 == 0);
    if constexpr (FG) {
      const f32x4_t lv = load4_guard(low, d, a.dim, true, a.dim % 4 == 0);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool ok = row_ok && d + j < a.dim;
        float alpha;
        const float kk = forget_key<T>(k[j] + bv[j], lv[j], &alpha);
        k[j] = ok ? kk : 0.f;
        L[dt][j] = ok ? log_forget<T>(alpha, kk) : 0.f;
        q[dt][j] = silu<T>(q[dt][j]);
      }
    } else {
      // z transposed: columns down, rows across the lanes
      f32x4_t z = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const T* a1 = qrow - h * a.dim + a.off_a;
      const T* a2 = reinterpret_cast<const T*>(a.a2) +
                    int64_t(h * a.dim + dt * 16 + lr) * a.rank;
      for (int k0 = 0; k0 < a.rank; k0 += 16) {
        const f32x4_t av = load4_guard(a1, k0 + g * 4, a.rank, row_ok, vec_a);
        const f32x4_t wv = load4_guard(a2, k0 + g * 4, a.rank,
                                       dt * 16 + lr < a.dim, vec_a);
#pragma unroll
        for (int j = 0; j < 4; ++j) z = mma4(wv[j], av[j], z);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool ok = row_ok && d + j < a.dim;
        L[dt][j] = ok ? log_sigmoid<T>(z[j] + bv[j]) / a.tau : 0.f;
        q[dt][j] *= qscale;
      }
    }
    *reinterpret_cast<f32x4_t*>(kl + trow * LR + d) = k;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      L[dt][j] = row_prefix(L[dt][j]);
      const float mid = __shfl(L[dt][j], g * 16 + 7, kWave);
      if (lr == 15) {
        tot[w * DP + d + j] = L[dt][j];
        wmin = fminf(wmin, fminf(mid, L[dt][j] - mid));
      }
    }
  }
  const bool safe = __all(wmin > -kSafeLog);
  __syncthreads();
  for (int d = threadIdx.x; d < DP; d += 256) {
    float t[4], b = 0.f;
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      t[s] = tot[s * DP + d];
      if (s > 0) EB[(s - 1) * DP + d] = gexp<T>(b);
      b += t[s];
    }
    a.dec[(int64_t(tile) * a.heads + h) * DP + d] = expf(b);
    float after = 0.f;
#pragma unroll
    for (int s = 3; s >= 0; --s) {
      if (s < 3) ED[s * DP + d] = gexp<T>(after);
      after += t[s];
    }
    EJ[d] = gexp<T>(t[1]);                // from 0 to 2
    EJ[DP + d] = gexp<T>(t[1] + t[2]);    // from 0 to 3
    EJ[2 * DP + d] = gexp<T>(t[2]);       // from 1 to 3
  }
  f32x4_t acc[4];
#pragma unroll
  for (int J = 0; J < 4; ++J) acc[J] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  if (!safe) {
    // steep decay: four-row blocks.  Block pairs a > b factor around the
    // row before a, so every exponent is <= 0; inside a block the three
    // distances are summed lane by lane.
    float near[4] = {0.f, 0.f, 0.f, 0.f};  // row lr and the row so far back
    f32x4_t far = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int dt = 0; dt < NT; ++dt) {
      if (dt >= ndt) continue;
      const f32x4_t k = *reinterpret_cast<const f32x4_t*>(
          kl + trow * LR + dt * 16 + g * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float Lt = L[dt][j], qv = q[dt][j], kv = k[j];
        float ref[4];
#pragma unroll
        for (int b = 1; b < 4; ++b)
          ref[b] = __shfl(Lt, g * 16 + 4 * b - 1, kWave);
        const int own = lr >> 2;
        const float mine = own == 3 ? ref[3] : own == 2 ? ref[2] : ref[1];
        const float qa = own > 0 ? qv * gexp<T>(Lt - mine) : 0.f;
#pragma unroll
        for (int b = 1; b < 4; ++b)
          far = mma4(own == b ? qa : 0.f,
                     lr < 4 * b ? kv * gexp<T>(ref[b] - Lt) : 0.f, far);
        near[0] += qv * kv;
        near[1] += qv * dpp_mov_f32<0x111>(kv) *
                   gexp<T>(fminf(Lt - dpp_mov_f32<0x111>(Lt), 0.f));
        near[2] += qv * dpp_mov_f32<0x112>(kv) *
                   gexp<T>(fminf(Lt - dpp_mov_f32<0x112>(Lt), 0.f));
        near[3] += qv * dpp_mov_f32<0x113>(kv) *
                   gexp<T>(fminf(Lt - dpp_mov_f32<0x113>(Lt), 0.f));
      }
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      near[x] += __shfl_xor(near[x], 16, kWave);
      near[x] += __shfl_xor(near[x], 32, kWave);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const float v = __shfl(near[x], g * 4 + r, kWave);
        if (lr >> 2 == g && g * 4 + r - lr == x) far[r] = v;
      }
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J == w) acc[J] = far;
  }
  __syncthreads();

  // this wave's own rows: q e^{L}, k e^{tot - L} and the diagonal block
  const int64_t ch = int64_t(tile) * a.heads + h;
  float* qd = a.qd + ch * C * DP;
  float* kd = a.kd + ch * DP * C;
  f32x4_t diag = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int dt = 0; dt < NT; ++dt) {
    if (dt >= ndt) continue;
    const int d = dt * 16 + g * 4;
    const f32x4_t tw = *reinterpret_cast<const f32x4_t*>(tot + w * DP + d);
    f32x4_t eb = f32x4_t{1.f, 1.f, 1.f, 1.f}, ed = eb;
    if (w > 0) eb = *reinterpret_cast<const f32x4_t*>(EB + (w - 1) * DP + d);
    if (w < 3) ed = *reinterpret_cast<const f32x4_t*>(ED + w * DP + d);
    f32x4_t kt = *reinterpret_cast<const f32x4_t*>(kl + trow * LR + d), qo;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float Lt = L[dt][j];
      if (safe) {
        const float Lm = __shfl(Lt, g * 16 + 7, kWave);
        diag = mma4(q[dt][j] * gexp<T>(Lt - Lm), kt[j] * gexp<T>(Lm - Lt),
                    diag);
      }
      q[dt][j] *= gexp<T>(Lt);
      qo[j] = q[dt][j] * eb[j];
      kt[j] *= gexp<T>(tw[j] - Lt);
      kd[int64_t(d + j) * C + trow] = kt[j] * ed[j];
    }
    *reinterpret_cast<f32x4_t*>(qd + trow * DP + d) = qo;
    *reinterpret_cast<f32x4_t*>(kl + trow * LR + d) = kt;
  }
  if (safe) {
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J == w) acc[J] = diag;
  }
  __syncthreads();
  // rows of the sub-chunks before
#pragma unroll
  for (int dt = 0; dt < NT; ++dt) {
    if (dt >= ndt) continue;
    const int d = dt * 16 + g * 4;
#pragma unroll
    for (int J = 0; J < 3; ++J) {
      if (J >= w) break;
      f32x4_t qe = q[dt];
      if (J + 1 < w) {
        const f32x4_t e = *reinterpret_cast<const f32x4_t*>(
            EJ + (J == 1 ? 2 : w - 2) * DP + d);
#pragma unroll
        for (int j = 0; j < 4; ++j) qe[j] *= e[j];
      }
      const f32x4_t kt =
          *reinterpret_cast<const f32x4_t*>(kl + (J * 16 + lr) * LR + d);
#pragma unroll
      for (int j = 0; j < 4; ++j) acc[J] = mma4(qe[j], kt[j], acc[J]);
    }
  }
  float* sc = a.sc + ch * C * C;
#pragma unroll
  for (int J = 0; J < 4; ++J) {
    if (J > w) break;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = g * 4 + r;
      float v = acc[J][r];
      if (J == w && lr > t) v = 0.f;
      sc[(w * 16 + t) * C + J * 16 + lr] = v;
    }
  }
}

// --------------------------------------------------------------- scan
// VT value tiles of 16 columns per workgroup, MD key tiles per wave
template <typename T, int VT, int MD>
__global__ __launch_bounds__(256)
void gla_scan_kernel(GlaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  constexpr int VS = VT * 16, SR = VS + 4;
  const int DP = a.dpad, ndt = DP / 16;
  float* Sl = sm;                         // [DP][SR]
  float* Vl = Sl + DP * SR;               // [64][SR]
  const int seq = blockIdx.x / a.heads, h = blockIdx.x % a.heads;
  const int v0 = blockIdx.y * VS;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int lr = lane & 15, g = lane >> 4;
  const int first = a.seqs[seq], count = a.seqs[a.n_seqs + seq];
  const bool fresh = a.seqs[2 * a.n_seqs + seq] == 0;
  float* state = a.state +
                 (int64_t(a.seqs[3 * a.n_seqs + seq]) * a.heads + h) *
                     a.dim * a.vpad;
  const int hv = a.heads * a.vdim;

  f32x4_t S[MD][VT];
#pragma unroll
  for (int i = 0; i < MD; ++i)
#pragma unroll
    for (int nt = 0; nt < VT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (i * 4 + w) * 16 + g * 4 + r;
        const int c = v0 + nt * 16 + lr;
        S[i][nt][r] = (!fresh && d < a.dim && c < a.vdim)
                          ? state[int64_t(d) * a.vpad + c] : 0.f;
      }

  // A chunk's operands travel in registers, loaded while the chunk
  // before it computes: q e^b and A rows and V until its outputs are
  // done, the key side until its state update is.
  constexpr int NQ = 4 * MD, NV = VT * 16 * C / 256;
  const int trow = w * 16 + lr;
  f32x4_t qr[NQ], ar[4], kr[MD][4];
  float vr[NV];
  const T* vb = reinterpret_cast<const T*>(a.proj) + a.off_v + h * a.vdim;
  auto load_q = [&](int t) {
    const int64_t ch = int64_t(t) * a.heads + h;
    const float* qd = a.qd + ch * C * DP + trow * DP + g * 4;
    const float* sc = a.sc + ch * C * C + trow * C + g * 4;
#pragma unroll
    for (int i = 0; i < NQ; ++i)
      if (i < ndt) qr[i] = *reinterpret_cast<const f32x4_t*>(qd + i * 16);
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J <= w) ar[J] = *reinterpret_cast<const f32x4_t*>(sc + J * 16);
    const int row0 = a.tiles[t], n = a.tiles[2 * a.n_tiles + t];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = i * 256 + threadIdx.x;
      const int r = e / VS, c = v0 + e % VS;
      vr[i] = (r < n && c < a.vdim)
                  ? act_load(vb + int64_t(row0 + r) * a.stride + c) : 0.f;
    }
  };
  auto load_k = [&](int t) {
    const float* kd = a.kd + (int64_t(t) * a.heads + h) * DP * C;
#pragma unroll
    for (int i = 0; i < MD; ++i)
      if (i * 4 + w < ndt)
#pragma unroll
        for (int s = 0; s < 4; ++s)
          kr[i][s] = *reinterpret_cast<const f32x4_t*>(
              kd + int64_t((i * 4 + w) * 16 + lr) * C + s * 16 + g * 4);
  };
  if (count > 0) {
    load_q(first);
    load_k(first);
  }
  for (int t = first; t < first + count; ++t) {
    const bool more = t + 1 < first + count;
    const int row0 = a.tiles[t];
    const int n = a.tiles[2 * a.n_tiles + t];
    const float* dec = a.dec + (int64_t(t) * a.heads + h) * DP;
    f32x4_t dv[MD];
#pragma unroll
    for (int i = 0; i < MD; ++i)
      if (i * 4 + w < ndt)
        dv[i] = *reinterpret_cast<const f32x4_t*>(
            dec + (i * 4 + w) * 16 + g * 4);
#pragma unroll
    for (int i = 0; i < MD; ++i)
      if (i * 4 + w < ndt)
#pragma unroll
        for (int nt = 0; nt < VT; ++nt)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            Sl[((i * 4 + w) * 16 + g * 4 + r) * SR + nt * 16 + lr] =
                S[i][nt][r];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int e = i * 256 + threadIdx.x;
      Vl[(e / VS) * SR + e % VS] = vr[i];
    }
    __syncthreads();
    f32x4_t o[VT];
#pragma unroll
    for (int nt = 0; nt < VT; ++nt) o[nt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NQ; ++i) {
      if (i < ndt)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nt = 0; nt < VT; ++nt)
          o[nt] = mma4(qr[i][j], Sl[(i * 16 + g * 4 + j) * SR + nt * 16 + lr],
                       o[nt]);
    }
#pragma unroll
    for (int J = 0; J < 4; ++J) {
      if (J <= w)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int nt = 0; nt < VT; ++nt)
          o[nt] = mma4(ar[J][j], Vl[(J * 16 + g * 4 + j) * SR + nt * 16 + lr],
                       o[nt]);
    }
    if (more) load_q(t + 1);
#pragma unroll
    for (int nt = 0; nt < VT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tr = w * 16 + g * 4 + r, c = v0 + nt * 16 + lr;
        if (tr < n && c < a.vdim)
          a.o[int64_t(row0 + tr) * hv + h * a.vdim + c] = o[nt][r];
      }
#pragma unroll
    for (int i = 0; i < MD; ++i) {
      if (i * 4 + w >= ndt) continue;
#pragma unroll
      for (int nt = 0; nt < VT; ++nt)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][nt][r] *= dv[i][r];
#pragma unroll
      for (int s = 0; s < 4; ++s)
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int nt = 0; nt < VT; ++nt)
            S[i][nt] = mma4(kr[i][s][j],
                            Vl[(s * 16 + g * 4 + j) * SR + nt * 16 + lr],
                            S[i][nt]);
    }
    if (more) load_k(t + 1);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < MD; ++i)
#pragma unroll
    for (int nt = 0; nt < VT; ++nt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int d = (i * 4 + w) * 16 + g * 4 + r;
        const int c = v0 + nt * 16 + lr;
        if (d < a.dim && c < a.vdim) state[int64_t(d) * a.vpad + c] = S[i][nt][r];
      }
}

// GL lanes per (row, head); V4 float4 columns per lane when the width and
// its offsets allow vectors (V4 = 0: one column at a time)
template <typename T, bool FG, int V4, int GL>
__global__ __launch_bounds__(256)
void gla_gate_kernel(GlaArgs a) {
  const int lane = threadIdx.x % GL;
  const int64_t rh = int64_t(blockIdx.x) * (256 / GL) + threadIdx.x / GL;
  if (rh >= int64_t(a.rows) * a.heads) return;
  const int64_t row = rh / a.heads;
  const int h = int(rh % a.heads);
  const int hv = a.heads * a.vdim;
  const float* o = a.o + row * hv + h * a.vdim;
  const T* gate = reinterpret_cast<const T*>(a.proj) + row * a.stride +
                  a.off_g + h * a.vdim;
  T* out = reinterpret_cast<T*>(a.out) + row * a.out_stride + h * a.vdim;
  float ss = 0.f;
  if constexpr (V4 > 0) {
    f32x4_t ov[V4], gv[V4];
#pragma unroll
    for (int i = 0; i < V4; ++i) {
      const int c = (i * GL + lane) * 4;
      ov[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (c < a.vdim) {
        ov[i] = *reinterpret_cast<const f32x4_t*>(o + c);
        if constexpr (!FG) gv[i] = act_load4(gate + c);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) ss += ov[i][j] * ov[i][j];
    }
    const float inv = 1.f / sqrtf(group_sum<GL>(ss) / a.vdim + a.eps);
#pragma unroll
    for (int i = 0; i < V4; ++i) {
      const int c = (i * GL + lane) * 4;
      if (c >= a.vdim) break;
      const f32x4_t nv = *reinterpret_cast<const f32x4_t*>(a.norm + c);
      f32x4_t r;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        r[j] = ov[i][j] * inv * nv[j];
        if constexpr (!FG) r[j] *= gv[i][j] / (1.f + gexp<T>(-gv[i][j]));
      }
      act_store4(out + c, r);
    }
  } else {
    for (int e = lane; e < a.vdim; e += GL) ss += o[e] * o[e];
    const float inv = 1.f / sqrtf(group_sum<GL>(ss) / a.vdim + a.eps);
    for (int e = lane; e < a.vdim; e += GL) {
      float r = o[e] * inv * a.norm[e];
      if constexpr (!FG) {
        const float g = act_load(gate + e);
        r *= g / (1.f + gexp<T>(-g));
      }
      act_store(out + e, r);
    }
  }
}

template <typename T, int VT>
void scan_md(const GlaArgs& a, hipStream_t st) {
  constexpr int VS = VT * 16;
  const size_t smem = size_t(a.dpad + C) * (VS + 4) * sizeof(float);
  auto run = [&](auto* k) {
    if (smem > 65536)
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                                hipFuncAttributeMaxDynamicSharedMemorySize,
                                int(smem));
    hipLaunchKernelGGL(k, dim3(a.n_seqs * a.heads, (a.vdim + VS - 1) / VS),
                       dim3(256), smem, st, a);
  };
  if (a.dpad <= 64) run(gla_scan_kernel<T, VT, 1>);
  else if (a.dpad <= 128) run(gla_scan_kernel<T, VT, 2>);
  else run(gla_scan_kernel<T, VT, 4>);
}

template <typename T, bool FG>
void prefill(const GlaArgs& a, hipStream_t st) {
  const bool vec = a.dim % 4 == 0 && a.stride % 4 == 0;
  const bool vec_a = a.rank % 4 == 0 && a.off_a % 4 == 0 && a.stride % 4 == 0;
  const size_t smem =
      size_t(C * (a.dpad + 4) + 13 * a.dpad) * sizeof(float);
  auto intra = [&](auto* k) {
    if (smem > 65536)
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(k),
                                hipFuncAttributeMaxDynamicSharedMemorySize,
                                int(smem));
    hipLaunchKernelGGL(k, dim3(a.n_tiles, a.heads), dim3(256), smem, st, a,
                       vec, vec_a);
  };
  if (a.dpad <= 64) intra(gla_intra_kernel<T, FG, 1>);
  else if (a.dpad <= 128) intra(gla_intra_kernel<T, FG, 2>);
  else intra(gla_intra_kernel<T, FG, 4>);
  // a scan step is latency-bound: narrow value slices, several
  // workgroups per CU, until there are plenty anyway
  const int64_t sh = int64_t(a.n_seqs) * a.heads;
  if (a.vdim > 32 && sh * ((a.vdim + 63) / 64) >= 512) scan_md<T, 4>(a, st);
  else if (a.vdim > 16 && sh * ((a.vdim + 31) / 32) >= 1024)
    scan_md<T, 2>(a, st);
  else scan_md<T, 1>(a, st);
  auto gate = [&](auto* kg, int per_wg = 4) {
    const int64_t rh = int64_t(a.rows) * a.heads;
    hipLaunchKernelGGL(kg, dim3(uint32_t((rh + per_wg - 1) / per_wg)),
                       dim3(256), 0, st, a);
  };
  if (a.vdim % 4 || a.stride % 4 || a.off_g % 4 || a.out_stride % 4 ||
      reinterpret_cast<uintptr_t>(a.out) % 16)
    gate(gla_gate_kernel<T, FG, 0, 64>);
  else if (a.vdim <= 64)
    gate(gla_gate_kernel<T, FG, 1, 16>, 16);
  else if (a.vdim <= 128)
    gate(gla_gate_kernel<T, FG, 1, 32>, 8);
  else if (a.vdim <= 256)
    gate(gla_gate_kernel<T, FG, 1, 64>);
  else
    gate(gla_gate_kernel<T, FG, 4, 64>);
}

}  // namespace

void launch_gla_decode(const GlaArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  const int n_rows = 256 / (a.vpad / 4);
  const size_t smem =
      size_t(3 * a.dpad + (a.rank + 3) / 4 * 4 + n_rows * a.vpad) *
      sizeof(float);
  const dim3 grid(a.rows, a.heads);
  auto go = [&](auto* k) {
    hipLaunchKernelGGL(k, grid, dim3(256), smem, st, a);
  };
  if (a.forget) {
    if (a.f32) go(gla_decode_kernel<float, true>);
    else go(gla_decode_kernel<uint16_t, true>);
  } else {
    if (a.f32) go(gla_decode_kernel<float, false>);
    else go(gla_decode_kernel<uint16_t, false>);
  }
}

void launch_gla_prefill(const GlaArgs& a, hipStream_t st) {
  if (a.rows == 0 || a.n_seqs == 0) return;
  if (a.forget) {
    if (a.f32) prefill<float, true>(a, st);
    else prefill<uint16_t, true>(a, st);
  } else {
    if (a.f32) prefill<float, false>(a, st);
    else prefill<uint16_t, false>(a, st);
  }
}

}  // namespace rlli
