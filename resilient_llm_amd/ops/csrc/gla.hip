// Gated linear recurrences: S_t = diag(alpha_t) S_{t-1} + k_t v_t^T,
// o_t = S_t^T q_t per head, alpha a decay per key channel, then RMS norm
// over the value width.  Three ways to make q, k and alpha from the
// projections:
//   GLA     q | k | v | gate | A1 h:  alpha = sigmoid(z)^(1/tau) with
//           z = A2 (A1 h) + b, q scaled by dim^-1/2, silu output gate
//   HGRN2   q | z | v:  alpha = l + (1 - l) sigmoid(z + b) with a lower
//           bound l per channel, k = 1 - alpha, q = silu(q), no gate
//   RWKV    alpha = e^(-e^z) with z = A2 tanh(A1 h) + b, silu output gate,
//           and o_t = S_{t-1}^T q_t + (q_t . u k_t) v_t: the past, and the
//           present through a bonus u per channel
//
// Projections arrive as GEMM output rows; everything from z on is
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
// that four-row blocks do the same once more.  RWKV's queries take the
// log-decay of the row before theirs, its diagonal is the bonus.
//   gla_intra   per (chunk, head): A, q e^{b_t}, k e^{b_C - b_s}, e^{b_C}
// then the scan and the gate of rec_scan.hip.

#include "rec_math.h"

#include <type_traits>

namespace rlli {
namespace {

constexpr int C = kRecChunk;
constexpr float kSafeLog = 40.f;

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

// RWKV: log alpha; e^-80 is nothing
template <typename T>
DEV_INLINE float log_rwkv(float z) {
  return -fminf(gexp<T>(z), 80.f);
}

// ------------------------------------------------------------- decode
template <typename T, int KIND>
__global__ __launch_bounds__(256)
void gla_decode_kernel(GlaArgs a) {
  constexpr bool FG = KIND == kHgrn2, BONUS = KIND == kRwkv;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int seq = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x;
  float* al = sm;                       // [dim]
  float* ks = al + a.dpad;              // [dim]
  float* qs = ks + a.dpad;              // [dim]
  float* uk = qs + a.dpad;              // [dim] bonus times key (RWKV)
  float* a1 = uk + (BONUS ? a.dpad : 0);    // [rank, padded to 4]
  float* red = a1 + (a.rank + 3) / 4 * 4;   // [rows][vpad] then sums
  const T* row = reinterpret_cast<const T*>(a.proj) + int64_t(seq) * a.stride;
  if constexpr (FG) {
    for (int d = tid; d < a.dim; d += 256) {
      const int hc = h * a.dim + d;
      qs[d] = silu<T>(act_load(row + hc));
      ks[d] = forget_key<T>(act_load(row + a.off_k + hc) + a.a2_bias[hc],
                            a.lower[hc], al + d);
    }
  } else {
    const T* low =
        reinterpret_cast<const T*>(a.a1) + int64_t(seq) * a.a1_stride;
    for (int r = tid; r < a.rank; r += 256)
      a1[r] = BONUS ? gtanh<T>(act_load(low + r)) : act_load(low + r);
    const float qscale = BONUS ? 1.f : 1.f / sqrtf(float(a.dim));
    for (int d = tid; d < a.dim; d += 256) {
      qs[d] = act_load(row + h * a.dim + d) * qscale;
      ks[d] = act_load(row + a.off_k + h * a.dim + d);
      if constexpr (BONUS) uk[d] = a.bonus[h * a.dim + d] * ks[d];
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
      al[d] = BONUS ? expf(log_rwkv<T>(z))
                    : expf(log_sigmoid<T>(z) / a.tau);
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
          if constexpr (BONUS) o[j] += qs[d] * (s[u][j] + uk[d] * v[j]);
          s[u][j] = al[d] * s[u][j] + ks[d] * v[j];
          if constexpr (!BONUS) o[j] += qs[d] * s[u][j];
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
    float o2 = red[e] * inv * a.norm[h * a.norm_stride + e];
    if constexpr (!FG)
      o2 *= silu<T>(act_load(row + a.off_g + h * a.vdim + e));
    act_store(out + e, o2);
  }
}

// -------------------------------------------------------------- intra
// the running log-decay that a query sees: its own row's or, before the
// present row counts, the last one's (rows are lanes)
template <bool BEFORE>
DEV_INLINE float seen_log(float L) {
  if constexpr (BEFORE) return dpp_mov_f32<0x111>(L);
  return L;
}

// Wave w owns sub-chunk w, lane l its row l & 15 and four neighbouring key
// columns of every 16; MD bounds the key tiles (dpad <= 64 * MD).  FULL: dim
// is 64 MD, the rank a multiple of 16 and rows are aligned, so that no load
// is conditional (rows behind the last one are loaded from it).
template <typename T, int KIND, int MD, bool FULL>
__global__ __launch_bounds__(256)
void gla_intra_kernel(GlaArgs a, bool vec, bool vec_a) {
  constexpr bool FG = KIND == kHgrn2, BONUS = KIND == kRwkv;
  extern __shared__ __attribute__((aligned(16))) float sm[];
  constexpr int NT = 4 * MD;
  const int tile = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x & 63;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int lr = lane & 15, g = lane >> 4;
  const int DP = FULL ? 64 * MD : a.dpad, LR = DP + 4, ndt = DP / 16;
  float* kl = sm;                        // [64][LR] keys, then decayed keys
  float* tot = kl + C * LR;              // [4][DP] log-decays of sub-chunks
  float* EB = tot + 4 * DP;              // [3][DP] e^{B_w}, w = 1 .. 3
  float* ED = EB + 3 * DP;               // [3][DP] e^{B_4 - B_{w+1}}, w < 3
  float* EJ = ED + 3 * DP;               // [3][DP] sub-chunks in between
  const int row0 = a.tiles[tile];
  const int n = a.tiles[2 * a.n_tiles + tile];
  const int trow = w * 16 + lr;          // this lane's row
  const bool row_ok = trow < n;
  const int64_t at = row0 + (FULL ? min(trow, n - 1) : trow);
  const T* qrow = reinterpret_cast<const T*>(a.proj) + at * a.stride +
                  h * a.dim;
  auto row4 = [&](const T* p, int d, int width, bool v) {
    if constexpr (FULL) return act_load4(p + d);
    else return load4_guard(p, d, width, row_ok, v);
  };
  auto vec4 = [&](const float* p, int d) {
    if constexpr (FULL) return *reinterpret_cast<const f32x4_t*>(p + d);
    else return load4_guard(p, d, a.dim, true, a.dim % 4 == 0);
  };
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
    if (!FULL && dt >= ndt) continue;
    const int d = dt * 16 + g * 4;
    q[dt] = row4(qrow, d, a.dim, vec);
    L[dt] = row4(krow, d, a.dim, vec);
  }
#pragma unroll
  for (int dt = 0; dt < NT; ++dt) {
    if (!FULL && dt >= ndt) continue;
    const int d = dt * 16 + g * 4;
    f32x4_t k = L[dt];
    if constexpr (FULL && !FG)
      if (!row_ok) k = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const f32x4_t bv = vec4(bias, d);
    if constexpr (FG) {
      const f32x4_t lv = vec4(low, d);
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
      const T* a1 = reinterpret_cast<const T*>(a.a1) + at * a.a1_stride;
      const T* a2 = reinterpret_cast<const T*>(a.a2) +
                    int64_t(h * a.dim + dt * 16 + lr) * a.rank;
      for (int k0 = 0; k0 < a.rank; k0 += 16) {
        f32x4_t av = row4(a1, k0 + g * 4, a.rank, vec_a);
        if constexpr (BONUS)
#pragma unroll
          for (int j = 0; j < 4; ++j) av[j] = gtanh<T>(av[j]);
        f32x4_t wv;
        if constexpr (FULL) wv = act_load4(a2 + k0 + g * 4);
        else wv = load4_guard(a2, k0 + g * 4, a.rank, dt * 16 + lr < a.dim,
                              vec_a);
#pragma unroll
        for (int j = 0; j < 4; ++j) z = mma4(wv[j], av[j], z);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool ok = row_ok && d + j < a.dim;
        const float lw = BONUS ? log_rwkv<T>(z[j] + bv[j])
                               : log_sigmoid<T>(z[j] + bv[j]) / a.tau;
        L[dt][j] = ok ? lw : 0.f;
        if constexpr (!BONUS) q[dt][j] *= qscale;
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
  auto seen = [&](float Lt) { return seen_log<BONUS>(Lt); };
  float own = 0.f;                       // this row's diagonal
  if constexpr (BONUS) {
#pragma unroll
    for (int dt = 0; dt < NT; ++dt) {
      if (!FULL && dt >= ndt) continue;
      const int d = dt * 16 + g * 4;
      const f32x4_t kv = *reinterpret_cast<const f32x4_t*>(kl + trow * LR + d);
      const f32x4_t uv = vec4(a.bonus + h * a.dim, d);
#pragma unroll
      for (int j = 0; j < 4; ++j) own += q[dt][j] * uv[j] * kv[j];
    }
    own += __shfl_xor(own, 16, kWave);
    own += __shfl_xor(own, 32, kWave);
  }
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
      if (!FULL && dt >= ndt) continue;
      const f32x4_t k = *reinterpret_cast<const f32x4_t*>(
          kl + trow * LR + dt * 16 + g * 4);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float Lt = L[dt][j], Lq = seen(Lt), qv = q[dt][j], kv = k[j];
        float ref[4];
#pragma unroll
        for (int b = 1; b < 4; ++b)
          ref[b] = __shfl(Lt, g * 16 + 4 * b - 1, kWave);
        const int blk = lr >> 2;
        const float mine = blk == 3 ? ref[3] : blk == 2 ? ref[2] : ref[1];
        const float qa = blk > 0 ? qv * gexp<T>(Lq - mine) : 0.f;
#pragma unroll
        for (int b = 1; b < 4; ++b)
          far = mma4(blk == b ? qa : 0.f,
                     lr < 4 * b ? kv * gexp<T>(ref[b] - Lt) : 0.f, far);
        if constexpr (!BONUS) near[0] += qv * kv;
        near[1] += qv * dpp_mov_f32<0x111>(kv) *
                   gexp<T>(fminf(Lq - dpp_mov_f32<0x111>(Lt), 0.f));
        near[2] += qv * dpp_mov_f32<0x112>(kv) *
                   gexp<T>(fminf(Lq - dpp_mov_f32<0x112>(Lt), 0.f));
        near[3] += qv * dpp_mov_f32<0x113>(kv) *
                   gexp<T>(fminf(Lq - dpp_mov_f32<0x113>(Lt), 0.f));
      }
    }
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      near[x] += __shfl_xor(near[x], 16, kWave);
      near[x] += __shfl_xor(near[x], 32, kWave);
    }
    if constexpr (BONUS) near[0] = own;
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
    if (!FULL && dt >= ndt) continue;
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
        diag = mma4(q[dt][j] * gexp<T>(seen(Lt) - Lm),
                    kt[j] * gexp<T>(Lm - Lt), diag);
      }
      q[dt][j] *= gexp<T>(seen(Lt));
      qo[j] = q[dt][j] * eb[j];
      kt[j] *= gexp<T>(tw[j] - Lt);
      kd[int64_t(d + j) * C + trow] = kt[j] * ed[j];
    }
    *reinterpret_cast<f32x4_t*>(qd + trow * DP + d) = qo;
    *reinterpret_cast<f32x4_t*>(kl + trow * LR + d) = kt;
  }
  if (safe) {
    if constexpr (BONUS)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float v = __shfl(own, g * 4 + r, kWave);
        if (g * 4 + r == lr) diag[r] = v;
      }
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J == w) acc[J] = diag;
  }
  __syncthreads();
  // rows of the sub-chunks before
#pragma unroll
  for (int dt = 0; dt < NT; ++dt) {
    if (!FULL && dt >= ndt) continue;
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

template <typename T, int KIND>
void prefill(const GlaArgs& a, hipStream_t st) {
  const bool vec = a.dim % 4 == 0 && a.stride % 4 == 0 && a.off_k % 4 == 0 &&
                   reinterpret_cast<uintptr_t>(a.proj) % (4 * sizeof(T)) == 0;
  const bool vec_a = a.rank % 4 == 0 && a.a1_stride % 4 == 0 &&
                     reinterpret_cast<uintptr_t>(a.a1) % (4 * sizeof(T)) == 0;
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
  bool done = false;                      // (gains nothing for the others)
  if constexpr (sizeof(T) == 2 && KIND == kRwkv) {
    done = vec && vec_a && a.rank % 16 == 0 && (a.dim == 64 || a.dim == 128) &&
           reinterpret_cast<uintptr_t>(a.a2) % 8 == 0;
    if (done && a.dim == 64) intra(gla_intra_kernel<T, KIND, 1, true>);
    else if (done) intra(gla_intra_kernel<T, KIND, 2, true>);
  }
  if (done) {
  } else if (a.dpad <= 64) {
    intra(gla_intra_kernel<T, KIND, 1, false>);
  } else if (a.dpad <= 128) {
    intra(gla_intra_kernel<T, KIND, 2, false>);
  } else {
    intra(gla_intra_kernel<T, KIND, 4, false>);
  }
  ScanArgs sa{};
  sa.v = reinterpret_cast<const T*>(a.proj) + a.off_v;
  sa.v_stride = a.stride;
  sa.qd = a.qd;
  sa.kt = a.kd;
  sa.sc = a.sc;
  sa.dec = a.dec;
  sa.state = a.state;
  sa.o = a.o;
  sa.tiles = a.tiles;
  sa.seqs = a.seqs;
  sa.n_rows = a.rows;
  sa.n_tiles = a.n_tiles;
  sa.n_seqs = a.n_seqs;
  sa.heads = a.heads;
  sa.group = 1;
  sa.dim = a.dim;
  sa.dpad = a.dpad;
  sa.vdim = sa.cols = sa.opad = a.vdim;
  sa.vpad = a.vpad;
  sa.mode = kScanPlain;
  sa.f32 = a.f32;
  launch_rec_scan(sa, st);
  RecGateArgs ga{};
  ga.o = a.o;
  ga.gate = reinterpret_cast<const T*>(a.proj) + a.off_g;
  ga.gate_stride = a.stride;
  ga.norm = a.norm;
  ga.norm_stride = a.norm_stride;
  ga.out = a.out;
  ga.out_stride = a.out_stride;
  ga.rows = a.rows;
  ga.heads = a.heads;
  ga.vdim = ga.opad = a.vdim;
  ga.kind = KIND == kHgrn2 ? kGateNone : kGateSilu;
  ga.eps = a.eps;
  ga.f32 = a.f32;
  launch_rec_gate(ga, st);
}

template <typename F>
void by_kind(const GlaArgs& a, F f) {
  auto go = [&](auto t) {
    if (a.kind == kHgrn2) f(t, std::integral_constant<int, kHgrn2>{});
    else if (a.kind == kRwkv) f(t, std::integral_constant<int, kRwkv>{});
    else f(t, std::integral_constant<int, kGla>{});
  };
  if (a.f32) go(float{});
  else go(uint16_t{});
}

}  // namespace

void launch_gla_decode(const GlaArgs& a, hipStream_t st) {
  if (a.rows == 0) return;
  const int n_rows = 256 / (a.vpad / 4);
  const size_t smem =
      size_t((a.kind == kRwkv ? 4 : 3) * a.dpad + (a.rank + 3) / 4 * 4 +
             n_rows * a.vpad) * sizeof(float);
  by_kind(a, [&](auto t, auto kind) {
    hipLaunchKernelGGL((gla_decode_kernel<decltype(t), decltype(kind)::value>),
                       dim3(a.rows, a.heads), dim3(256), smem, st, a);
  });
}

void launch_gla_prefill(const GlaArgs& a, hipStream_t st) {
  if (a.rows == 0 || a.n_seqs == 0) return;
  by_kind(a, [&](auto t, auto kind) {
    prefill<decltype(t), decltype(kind)::value>(a, st);
  });
}

}  // namespace rlli
