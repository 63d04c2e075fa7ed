// Torch bindings (torch.ops.rlli_rec.*) of the gated linear recurrences.

#include "ext_common.h"
#include "mix.h"

namespace {

using namespace rlli_ext;

// what both recurrences share: projections, state, norm, output
rlli::GlaArgs rec_args(const Tensor& proj, const Tensor& bias,
                       const Tensor& norm, const Tensor& state, int64_t vdim,
                       double eps, const Tensor& out) {
  rlli::GlaArgs a{};
  a.f32 = act_f32(proj, "proj");
  TORCH_CHECK(proj.dim() == 2, "proj must be [rows, columns]");
  TORCH_CHECK(state.is_cuda() && state.is_contiguous() && state.dim() == 4 &&
              state.scalar_type() == at::kFloat,
              "state must be f32 [slots, heads, dim, vdim padded to 4]");
  a.rows = int(proj.size(0));
  a.stride = int(proj.size(1));
  a.n_slots = int(state.size(0));
  a.heads = int(state.size(1));
  a.dim = int(state.size(2));
  a.vpad = int(state.size(3));
  a.vdim = int(vdim);
  TORCH_CHECK(a.vpad % 4 == 0 && a.vpad >= a.vdim && a.vpad < a.vdim + 4);
  TORCH_CHECK(a.dim >= 1 && a.dim <= 256 && a.vdim >= 1 && a.vdim <= 1024,
              "recurrent head sizes out of range");
  a.dpad = (a.dim + 15) / 16 * 16;
  a.proj = proj.data_ptr();
  a.a2_bias = f32_vec(bias, int64_t(a.heads) * a.dim, "bias");
  a.norm = f32_vec(norm, a.vdim, "norm");
  a.state = state.data_ptr<float>();
  a.eps = float(eps);
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
  a.a2 = a2.data_ptr();
  a.off_g = a.off_v + a.heads * a.vdim;
  a.off_a = a.off_g + a.heads * a.vdim;
  a.tau = float(tau);
}

void hgrn2_fill(rlli::GlaArgs& a, const Tensor& lower) {
  a.forget = true;
  a.lower = f32_vec(lower, int64_t(a.heads) * a.dim, "lower");
  TORCH_CHECK(a.stride == a.heads * (2 * a.dim + a.vdim),
              "hgrn2 projection width mismatch");
}

void decode(rlli::GlaArgs& a, const Tensor& proj, const Tensor& slots,
            const Tensor& positions) {
  a.slots = i32(slots, "slots");
  a.positions = i32(positions, "positions");
  TORCH_CHECK(slots.numel() == a.rows && positions.numel() == a.rows,
              "one state slot and position per row");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_gla_decode(a, stream_of(proj));
  check_launch("recurrent decode");
}

void prefill(rlli::GlaArgs& a, const Tensor& proj, const Tensor& tiles,
             const Tensor& seqs) {
  a.tiles = i32(tiles, "tiles");
  a.seqs = i32(seqs, "seqs");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4 && seqs.dim() == 2 &&
              seqs.size(0) == 4);
  a.n_tiles = int(tiles.size(1));
  a.n_seqs = int(seqs.size(1));
  const int64_t C = rlli::kGlaChunk;
  const int64_t nh = int64_t(a.n_tiles) * a.heads;
  auto fo = proj.options().dtype(at::kFloat);
  Tensor qd = at::empty({nh, C, a.dpad}, fo);
  Tensor kd = at::empty({nh, a.dpad, C}, fo);
  Tensor sc = at::empty({nh, C, C}, fo);
  Tensor dec = at::empty({nh, a.dpad}, fo);
  Tensor o = at::empty({a.rows, int64_t(a.heads) * a.vdim}, fo);
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
}

TORCH_LIBRARY_IMPL(rlli_rec, CUDA, m) {
  m.impl("gla_decode", &gla_decode);
  m.impl("gla_prefill", &gla_prefill);
  m.impl("hgrn2_decode", &hgrn2_decode);
  m.impl("hgrn2_prefill", &hgrn2_prefill);
}
