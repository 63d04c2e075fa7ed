// Torch bindings (torch.ops.rlli_rec.*) of the linear recurrences.

#include "ext_common.h"
#include "rec.h"

namespace {

using namespace rlli_ext;

// state, norm and output, as all recurrences have them; ``cols`` value
// columns are carried
template <typename A>
void carry_args(A& a, const Tensor& state, int64_t vdim, int64_t cols,
                double eps) {
  TORCH_CHECK(state.is_cuda() && state.is_contiguous() && state.dim() == 4 &&
              state.scalar_type() == at::kFloat,
              "state must be f32 [slots, heads, dim, columns padded to 4]");
  a.heads = int(state.size(1));
  a.dim = int(state.size(2));
  a.vpad = int(state.size(3));
  a.vdim = int(vdim);
  TORCH_CHECK(a.vpad % 4 == 0 && a.vpad >= cols && a.vpad < cols + 4,
              "state width does not fit the value width");
  TORCH_CHECK(a.dim >= 1 && a.dim <= 256 && vdim >= 1 && cols <= 1024,
              "recurrent head sizes out of range");
  a.dpad = (a.dim + 15) / 16 * 16;
  a.state = state.data_ptr<float>();
  a.eps = float(eps);
}

template <typename A>
void decode_args(A& a, const Tensor& slots, const Tensor& positions) {
  a.slots = i32(slots, "slots");
  a.positions = i32(positions, "positions");
  TORCH_CHECK(slots.numel() == a.rows && positions.numel() == a.rows,
              "one state slot and position per row");
}

template <typename A>
void prompt_args(A& a, const Tensor& tiles, const Tensor& seqs) {
  a.tiles = i32(tiles, "tiles");
  a.seqs = i32(seqs, "seqs");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4 && seqs.dim() == 2 &&
              seqs.size(0) == 4);
  a.n_tiles = int(tiles.size(1));
  a.n_seqs = int(seqs.size(1));
}

// projections, state, norm and output of the per-channel decays
rlli::GlaArgs rec_args(const Tensor& proj, const Tensor& bias,
                       const Tensor& norm, const Tensor& state, int64_t vdim,
                       double eps, const Tensor& out) {
  rlli::GlaArgs a{};
  a.f32 = act_f32(proj, "proj");
  TORCH_CHECK(proj.dim() == 2, "proj must be [rows, columns]");
  carry_args(a, state, vdim, vdim, eps);
  a.rows = int(proj.size(0));
  a.stride = int(proj.size(1));
  a.n_slots = int(state.size(0));
  a.proj = proj.data_ptr();
  a.a2_bias = f32_vec(bias, int64_t(a.heads) * a.dim, "bias");
  a.norm = f32_vec(norm, a.vdim, "norm");
  a.out_stride = int(row_stride(out, proj, a.rows,
                                int64_t(a.heads) * a.vdim, "out"));
  a.out = out.data_ptr();
  a.off_k = a.heads * a.dim;
  a.off_v = 2 * a.off_k;
  return a;
}

void gla_fill(rlli::GlaArgs& a, const Tensor& proj, const Tensor& a2,
              double tau) {
  same_act(a2, proj, "a2");
  TORCH_CHECK(a2.dim() == 2 && a2.size(0) == a.heads * a.dim);
  a.rank = int(a2.size(1));
  TORCH_CHECK(a.rank <= 1024, "decay rank out of range");
  TORCH_CHECK(a.stride == 2 * a.heads * (a.dim + a.vdim) + a.rank,
              "gla projection width mismatch");
  a.kind = rlli::kGla;
  a.a2 = a2.data_ptr();
  a.off_g = a.off_v + a.heads * a.vdim;
  a.a1 = static_cast<const char*>(proj.data_ptr()) +
         (a.off_g + a.heads * a.vdim) * proj.element_size();
  a.a1_stride = a.stride;
  a.tau = float(tau);
}

void hgrn2_fill(rlli::GlaArgs& a, const Tensor& lower) {
  a.kind = rlli::kHgrn2;
  a.lower = f32_vec(lower, int64_t(a.heads) * a.dim, "lower");
  TORCH_CHECK(a.stride == a.heads * (2 * a.dim + a.vdim),
              "hgrn2 projection width mismatch");
}

// r, k, v and gate are four matrices [rows, heads * dim]
rlli::GlaArgs rwkv_args(const Tensor& rkvg, const Tensor& low,
                        const Tensor& w2, const Tensor& w0,
                        const Tensor& bonus, const Tensor& norm,
                        const Tensor& state, double eps, const Tensor& out) {
  rlli::GlaArgs a{};
  TORCH_CHECK(rkvg.dim() == 3 && rkvg.size(0) == 4 && rkvg.is_cuda(),
              "rkvg must be [4, rows, columns]");
  a.f32 = rkvg.scalar_type() == at::kFloat;
  TORCH_CHECK(a.f32 || rkvg.scalar_type() == at::kBFloat16,
              "rkvg must be bf16 or f32");
  TORCH_CHECK(state.dim() == 4);
  carry_args(a, state, state.size(2), state.size(2), eps);
  const int64_t n = int64_t(a.heads) * a.dim;
  a.rows = int(rkvg.size(1));
  a.stride = row_stride(rkvg.select(0, 0), rkvg, a.rows, n, "rkvg");
  a.off_k = rkvg.stride(0);
  a.off_v = 2 * a.off_k;
  a.off_g = 3 * a.off_k;
  a.n_slots = int(state.size(0));
  a.kind = rlli::kRwkv;
  a.proj = rkvg.data_ptr();
  TORCH_CHECK(w2.dim() == 2 && w2.size(0) == n && w2.is_cuda() &&
              w2.is_contiguous() && w2.scalar_type() == rkvg.scalar_type(),
              "w2 must be [heads * dim, rank] of the activation dtype");
  a.rank = int(w2.size(1));
  TORCH_CHECK(a.rank <= 1024, "decay rank out of range");
  a.a2 = w2.data_ptr();
  a.a1_stride = row_stride(low, rkvg, a.rows, a.rank, "low");
  a.a1 = low.data_ptr();
  a.a2_bias = f32_vec(w0, n, "w0");
  a.bonus = f32_vec(bonus, n, "bonus");
  a.norm = f32_vec(norm, n, "norm");
  a.norm_stride = a.dim;
  a.out_stride = int(row_stride(out, rkvg, a.rows, n, "out"));
  a.out = out.data_ptr();
  return a;
}

void decode(rlli::GlaArgs& a, const Tensor& proj, const Tensor& slots,
            const Tensor& positions) {
  decode_args(a, slots, positions);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_gla_decode(a, stream_of(proj));
  check_launch("recurrent decode");
}

void prefill(rlli::GlaArgs& a, const Tensor& proj, const Tensor& tiles,
             const Tensor& seqs) {
  prompt_args(a, tiles, seqs);
  const int64_t C = rlli::kRecChunk;
  const int64_t nh = int64_t(a.n_tiles) * a.heads;
  auto fo = proj.options().dtype(at::kFloat);
  Tensor qd = at::empty({nh, C, a.dpad}, fo);
  Tensor kd = at::empty({nh, a.dpad, C}, fo);
  Tensor sc = at::empty({nh, C, C}, fo);
  Tensor dec = at::empty({nh, a.dpad}, fo);
  Tensor o = at::empty({a.rows + C, int64_t(a.heads) * a.vdim}, fo);
  a.qd = qd.data_ptr<float>();
  a.kd = kd.data_ptr<float>();
  a.sc = sc.data_ptr<float>();
  a.dec = dec.data_ptr<float>();
  a.o = o.data_ptr<float>();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_gla_prefill(a, stream_of(proj));
  check_launch("recurrent prefill");
}

void gla_decode(const Tensor& proj, const Tensor& a2, const Tensor& a2_bias,
                const Tensor& norm, Tensor state, const Tensor& slots,
                const Tensor& positions, int64_t vdim, double tau,
                double eps, Tensor out) {
  auto a = rec_args(proj, a2_bias, norm, state, vdim, eps, out);
  gla_fill(a, proj, a2, tau);
  decode(a, proj, slots, positions);
}

void gla_prefill(const Tensor& proj, const Tensor& a2, const Tensor& a2_bias,
                 const Tensor& norm, Tensor state, const Tensor& tiles,
                 const Tensor& seqs, int64_t vdim, double tau, double eps,
                 Tensor out) {
  auto a = rec_args(proj, a2_bias, norm, state, vdim, eps, out);
  gla_fill(a, proj, a2, tau);
  prefill(a, proj, tiles, seqs);
}

void hgrn2_decode(const Tensor& proj, const Tensor& bias, const Tensor& lower,
                  const Tensor& norm, Tensor state, const Tensor& slots,
                  const Tensor& positions, int64_t vdim, double eps,
                  Tensor out) {
  auto a = rec_args(proj, bias, norm, state, vdim, eps, out);
  hgrn2_fill(a, lower);
  decode(a, proj, slots, positions);
}

void hgrn2_prefill(const Tensor& proj, const Tensor& bias,
                   const Tensor& lower, const Tensor& norm, Tensor state,
                   const Tensor& tiles, const Tensor& seqs, int64_t vdim,
                   double eps, Tensor out) {
  auto a = rec_args(proj, bias, norm, state, vdim, eps, out);
  hgrn2_fill(a, lower);
  prefill(a, proj, tiles, seqs);
}

void rwkv_decode(const Tensor& rkvg, const Tensor& low, const Tensor& w2,
                 const Tensor& w0, const Tensor& bonus, const Tensor& norm,
                 Tensor state, const Tensor& slots, const Tensor& positions,
                 double eps, Tensor out) {
  auto a = rwkv_args(rkvg, low, w2, w0, bonus, norm, state, eps, out);
  decode(a, rkvg, slots, positions);
}

void rwkv_prefill(const Tensor& rkvg, const Tensor& low, const Tensor& w2,
                  const Tensor& w0, const Tensor& bonus, const Tensor& norm,
                  Tensor state, const Tensor& tiles, const Tensor& seqs,
                  double eps, Tensor out) {
  auto a = rwkv_args(rkvg, low, w2, w0, bonus, norm, state, eps, out);
  prefill(a, rkvg, tiles, seqs);
}

// ---------------------------------------------------------------- delta
// columns of proj: q | k | v | gate | beta | decay, anything behind them
rlli::DeltaArgs delta_args(const Tensor& proj, const Tensor& a_rate,
                           const Tensor& dt_bias, const Tensor& norm,
                           const Tensor& state, int64_t kv_heads,
                           int64_t vdim, double eps, const Tensor& out) {
  rlli::DeltaArgs a{};
  a.f32 = act_f32(proj, "proj");
  TORCH_CHECK(proj.dim() == 2, "proj must be [rows, columns]");
  carry_args(a, state, vdim, vdim, eps);
  TORCH_CHECK(kv_heads >= 1 && a.heads % kv_heads == 0,
              "heads must be a multiple of kv heads");
  a.kv_heads = int(kv_heads);
  a.rows = int(proj.size(0));
  a.stride = proj.size(1);
  a.channels = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
  a.off_g = a.channels;
  a.off_b = a.off_g + a.heads * a.vdim;
  a.off_a = a.off_b + a.heads;
  TORCH_CHECK(a.stride >= a.off_a + a.heads, "delta projection too narrow");
  a.ubp = (a.vdim + 15) / 16 * 16;
  a.proj = proj.data_ptr();
  a.a_rate = f32_vec(a_rate, a.heads, "a_rate");
  a.dt_bias = f32_vec(dt_bias, a.heads, "dt_bias");
  a.norm = f32_vec(norm, a.vdim, "norm");
  a.out_stride = row_stride(out, proj, a.rows,
                            int64_t(a.heads) * a.vdim, "out");
  a.out = out.data_ptr();
  return a;
}

void delta_decode(const Tensor& proj, const Tensor& taps,
                  const OptTensor& tail, const Tensor& a_rate,
                  const Tensor& dt_bias, const Tensor& norm, Tensor state,
                  const Tensor& slots, const Tensor& positions,
                  int64_t kv_heads, int64_t vdim, double eps, Tensor out) {
  auto a = delta_args(proj, a_rate, dt_bias, norm, state, kv_heads, vdim, eps,
                      out);
  decode_args(a, slots, positions);
  TORCH_CHECK(taps.dim() == 2);
  a.n_taps = int(taps.size(0));
  a.taps = f32_vec(taps, int64_t(a.n_taps) * a.channels, "taps");
  a.ring = 1;
  if (a.n_taps > 1) {
    TORCH_CHECK(tail.has_value(), "a convolution over time needs its state");
    same_act(*tail, proj, "tail");
    // heads that share a key head read its ring while one of them writes
    TORCH_CHECK(tail->dim() == 3 && tail->size(0) == state.size(0) &&
                tail->size(1) >= a.n_taps && tail->size(2) == a.channels,
                "tail must be [slots, taps or more, channels]");
    a.tail = tail->data_ptr();
    a.ring = int(tail->size(1));
  }
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_delta_decode(a, stream_of(proj));
  check_launch("delta_decode");
}

void delta_prefill(const Tensor& proj, const Tensor& x, const Tensor& a_rate,
                   const Tensor& dt_bias, const Tensor& norm, Tensor state,
                   const Tensor& tiles, const Tensor& seqs, int64_t kv_heads,
                   int64_t vdim, double eps, Tensor out) {
  auto a = delta_args(proj, a_rate, dt_bias, norm, state, kv_heads, vdim, eps,
                      out);
  prompt_args(a, tiles, seqs);
  same_act(x, proj, "x");
  TORCH_CHECK(x.dim() == 2 && x.size(0) == a.rows && x.size(1) >= a.channels,
              "x must be [rows, channels]");
  a.x = x.data_ptr();
  a.x_stride = x.size(1);
  const int64_t C = rlli::kRecChunk;
  const int64_t nh = int64_t(a.n_tiles) * a.heads;
  auto fo = proj.options().dtype(at::kFloat);
  Tensor kt = at::empty({int64_t(a.n_tiles) * a.kv_heads, a.dpad, C},
                        proj.options());
  Tensor sc = at::empty({nh, C, C}, fo);
  Tensor dec = at::empty({nh}, fo);
  Tensor row_f = at::empty({nh, 3, C}, fo);
  Tensor w = at::empty({nh, C, a.dpad}, fo);
  Tensor ub = at::empty({nh, C, a.ubp}, fo);
  Tensor o = at::empty({a.rows + C, int64_t(a.heads) * a.vdim}, fo);
  a.kt = kt.data_ptr();
  a.sc = sc.data_ptr<float>();
  a.dec = dec.data_ptr<float>();
  a.row_f = row_f.data_ptr<float>();
  a.w = w.data_ptr<float>();
  a.ub = ub.data_ptr<float>();
  a.o = o.data_ptr<float>();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_delta_prefill(a, stream_of(proj));
  check_launch("delta_prefill");
}

// ---------------------------------------------------------------- mlstm
// columns of proj: q | k | v | gate | i | f, anything behind them
rlli::MlstmArgs mlstm_args(const Tensor& proj, const Tensor& i_bias,
                           const Tensor& f_bias, const Tensor& norm,
                           const Tensor& state, const Tensor& m, int64_t vdim,
                           double cap, double eps, const Tensor& out) {
  rlli::MlstmArgs a{};
  a.f32 = act_f32(proj, "proj");
  TORCH_CHECK(proj.dim() == 2, "proj must be [rows, columns]");
  carry_args(a, state, vdim, vdim + 1, eps);
  a.rows = int(proj.size(0));
  a.stride = proj.size(1);
  a.off_k = a.heads * a.dim;
  a.off_v = 2 * a.off_k;
  a.off_g = a.off_v + a.heads * a.vdim;
  a.off_i = a.off_g + a.heads * a.vdim;
  a.off_f = a.off_i + a.heads;
  TORCH_CHECK(a.stride >= a.off_f + a.heads, "mlstm projection too narrow");
  a.opad = (a.vdim + 4) / 4 * 4;
  a.proj = proj.data_ptr();
  a.i_bias = f32_vec(i_bias, a.heads, "i_bias");
  a.f_bias = f32_vec(f_bias, a.heads, "f_bias");
  a.norm = f32_vec(norm, int64_t(a.heads) * a.vdim, "norm");
  f32_vec(m, state.size(0) * a.heads, "m");
  a.m = m.data_ptr<float>();
  TORCH_CHECK(cap > 0, "the gates' cap must be positive");
  a.cap = float(cap);
  a.out_stride = row_stride(out, proj, a.rows,
                            int64_t(a.heads) * a.vdim, "out");
  a.out = out.data_ptr();
  return a;
}

void mlstm_decode(const Tensor& proj, const Tensor& i_bias,
                  const Tensor& f_bias, const Tensor& norm, Tensor state,
                  Tensor m, const Tensor& slots, const Tensor& positions,
                  int64_t vdim, double cap, double eps, Tensor out) {
  auto a = mlstm_args(proj, i_bias, f_bias, norm, state, m, vdim, cap, eps,
                      out);
  decode_args(a, slots, positions);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_mlstm_decode(a, stream_of(proj));
  check_launch("mlstm_decode");
}

void mlstm_prefill(const Tensor& proj, const Tensor& i_bias,
                   const Tensor& f_bias, const Tensor& norm, Tensor state,
                   Tensor m, const Tensor& tiles, const Tensor& seqs,
                   int64_t vdim, double cap, double eps, Tensor out) {
  auto a = mlstm_args(proj, i_bias, f_bias, norm, state, m, vdim, cap, eps,
                      out);
  prompt_args(a, tiles, seqs);
  const int64_t C = rlli::kRecChunk;
  const int64_t nh = int64_t(a.n_tiles) * a.heads;
  auto fo = proj.options().dtype(at::kFloat);
  Tensor kt = at::empty({nh, a.dpad, C}, proj.options());
  Tensor sc = at::empty({nh, C, C}, fo);
  Tensor row_f = at::empty({nh, 3, C}, fo);
  Tensor o = at::empty({a.rows + C, a.heads, a.opad}, fo);
  Tensor mrow = at::empty({a.rows + C, a.heads}, fo);
  Tensor m_new = at::empty({a.n_seqs, a.heads}, fo);
  a.kt = kt.data_ptr();
  a.sc = sc.data_ptr<float>();
  a.row_f = row_f.data_ptr<float>();
  a.o = o.data_ptr<float>();
  a.mrow = mrow.data_ptr<float>();
  a.m_new = m_new.data_ptr<float>();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_mlstm_prefill(a, stream_of(proj));
  check_launch("mlstm_prefill");
}

}  // namespace

TORCH_LIBRARY(rlli_rec, m) {
  m.def("gla_decode(Tensor proj, Tensor a2, Tensor a2_bias, Tensor norm, "
        "Tensor(a!) state, Tensor slots, Tensor positions, int vdim, "
        "float tau, float eps, Tensor(b!) out) -> ()");
  m.def("gla_prefill(Tensor proj, Tensor a2, Tensor a2_bias, Tensor norm, "
        "Tensor(a!) state, Tensor tiles, Tensor seqs, int vdim, float tau, "
        "float eps, Tensor(b!) out) -> ()");
  m.def("hgrn2_decode(Tensor proj, Tensor bias, Tensor lower, Tensor norm, "
        "Tensor(a!) state, Tensor slots, Tensor positions, int vdim, "
        "float eps, Tensor(b!) out) -> ()");
  m.def("hgrn2_prefill(Tensor proj, Tensor bias, Tensor lower, Tensor norm, "
        "Tensor(a!) state, Tensor tiles, Tensor seqs, int vdim, float eps, "
        "Tensor(b!) out) -> ()");
  m.def("rwkv_decode(Tensor rkvg, Tensor low, Tensor w2, Tensor w0, "
        "Tensor bonus, Tensor norm, Tensor(a!) state, Tensor slots, "
        "Tensor positions, float eps, Tensor(b!) out) -> ()");
  m.def("rwkv_prefill(Tensor rkvg, Tensor low, Tensor w2, Tensor w0, "
        "Tensor bonus, Tensor norm, Tensor(a!) state, Tensor tiles, "
        "Tensor seqs, float eps, Tensor(b!) out) -> ()");
  m.def("delta_decode(Tensor proj, Tensor taps, Tensor(a!)? tail, "
        "Tensor a_rate, Tensor dt_bias, Tensor norm, Tensor(b!) state, "
        "Tensor slots, Tensor positions, int kv_heads, int vdim, float eps, "
        "Tensor(c!) out) -> ()");
  m.def("delta_prefill(Tensor proj, Tensor x, Tensor a_rate, Tensor dt_bias, "
        "Tensor norm, Tensor(a!) state, Tensor tiles, Tensor seqs, "
        "int kv_heads, int vdim, float eps, Tensor(b!) out) -> ()");
  m.def("mlstm_decode(Tensor proj, Tensor i_bias, Tensor f_bias, "
        "Tensor norm, Tensor(a!) state, Tensor(b!) m, Tensor slots, "
        "Tensor positions, int vdim, float cap, float eps, Tensor(c!) out) "
        "-> ()");
  m.def("mlstm_prefill(Tensor proj, Tensor i_bias, Tensor f_bias, "
        "Tensor norm, Tensor(a!) state, Tensor(b!) m, Tensor tiles, "
        "Tensor seqs, int vdim, float cap, float eps, Tensor(c!) out) "
        "-> ()");
}

TORCH_LIBRARY_IMPL(rlli_rec, CUDA, m) {
  m.impl("gla_decode", &gla_decode);
  m.impl("gla_prefill", &gla_prefill);
  m.impl("hgrn2_decode", &hgrn2_decode);
  m.impl("hgrn2_prefill", &hgrn2_prefill);
  m.impl("rwkv_decode", &rwkv_decode);
  m.impl("rwkv_prefill", &rwkv_prefill);
  m.impl("delta_decode", &delta_decode);
  m.impl("delta_prefill", &delta_prefill);
  m.impl("mlstm_decode", &mlstm_decode);
  m.impl("mlstm_prefill", &mlstm_prefill);
}
