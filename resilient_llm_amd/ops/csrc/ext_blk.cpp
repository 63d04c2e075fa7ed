// Torch bindings (torch.ops.rlli_blk.*) of the residual-block kernels.

#include "ext_common.h"
#include "blk.h"

namespace {

using namespace rlli_ext;

void check_tail(const OptTensor& tail, const Tensor& like, int n_taps,
                int width) {
  if (n_taps == 1) return;
  TORCH_CHECK(tail.has_value(), "a convolution over time needs its state");
  TORCH_CHECK(tail->is_cuda() && tail->is_contiguous() &&
              tail->scalar_type() == like.scalar_type(),
              "tail must be contiguous, on the GPU and of the activation "
              "dtype");
  TORCH_CHECK(tail->dim() == 3 && tail->size(1) >= n_taps - 1 &&
              tail->size(2) == width,
              "tail must be [slots, taps - 1 or more, width]");
}

std::tuple<Tensor, Tensor> block_run(rlli::BlockArgs& a, const Tensor& act,
                                     Tensor x, const Tensor& gain,
                                     int64_t groups, double eps,
                                     const Tensor& positions,
                                     const OptTensor& taps,
                                     const OptTensor& tail,
                                     const OptTensor& slots,
                                     int64_t n_decode) {
  TORCH_CHECK(x.dim() == 2 && x.is_cuda() && x.is_contiguous() &&
              x.scalar_type() == at::kFloat, "residual must be f32 [T, W]");
  a.width = int(x.size(1));
  TORCH_CHECK(a.width <= 16000, "width out of range");
  a.groups = int(groups);
  TORCH_CHECK(groups >= 1 && a.width % groups == 0,
              "norm groups must divide the width");
  a.x = x.data_ptr<float>();
  a.gain = f32_vec(gain, a.width, "gain");
  a.eps = float(eps);
  a.positions = i32(positions, "positions");
  TORCH_CHECK(positions.numel() == x.size(0), "one position per row");
  Tensor h = at::empty({a.n, a.width}, act.options());
  Tensor hc;
  a.h = h.data_ptr();
  a.branches = 1;
  a.ring = 1;
  if (taps) {
    TORCH_CHECK((taps->dim() == 2 || taps->dim() == 3) && !a.rows,
                "taps must be [taps, width] or [branches, taps, width]");
    if (taps->dim() == 3) a.branches = int(taps->size(0));
    a.n_taps = int(taps->size(-2));
    a.taps = f32_vec(*taps, int64_t(a.branches) * a.n_taps * a.width, "taps");
    check_tail(tail, act, a.n_taps, a.width);
    if (a.n_taps > 1) a.ring = int(tail->size(1));
    a.n_decode = int(n_decode);
    TORCH_CHECK(n_decode >= 0 && n_decode <= a.n);
    if (a.n_taps > 1) {
      a.tail = tail->data_ptr();
      if (a.n_decode) {
        TORCH_CHECK(slots.has_value());
        a.slots = i32(*slots, "slots");
        TORCH_CHECK(slots->numel() == a.n_decode, "one slot per decode row");
      }
    }
    hc = taps->dim() == 3
             ? at::empty({a.branches, a.n, a.width}, act.options())
             : at::empty({a.n, a.width}, act.options());
    a.hc = hc.data_ptr();
  } else {
    a.n_taps = 1;
    hc = at::empty({0}, act.options());
  }
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  rlli::launch_block_step(a, stream_of(x));
  check_launch("block_step");
  return {h, hc};
}

std::tuple<Tensor, Tensor> block_embed(
    const Tensor& ids, const Tensor& table, const OptTensor& pos_table,
    const Tensor& positions, Tensor x, const Tensor& gain, int64_t groups,
    double eps, const OptTensor& taps, const OptTensor& tail,
    const OptTensor& slots, int64_t n_decode, double scale) {
  rlli::BlockArgs a{};
  a.f32 = act_f32(table, "table");
  TORCH_CHECK(table.dim() == 2 && table.size(1) == x.size(-1));
  a.table = table.data_ptr();
  if (pos_table) {
    same_act(*pos_table, table, "pos_table");
    TORCH_CHECK(pos_table->dim() == 2 &&
                pos_table->size(1) == table.size(1));
    a.pos_table = pos_table->data_ptr();
    a.n_positions = int(pos_table->size(0));
    TORCH_CHECK(a.n_positions >= 1, "empty position table");
  }
  a.ids = i32(ids, "ids");
  a.n = int(x.size(0));
  TORCH_CHECK(ids.numel() == a.n, "one id per row");
  a.embed_scale = float(scale);
  a.keep = true;
  return block_run(a, table, x, gain, groups, eps, positions, taps, tail,
                   slots, n_decode);
}

std::tuple<Tensor, Tensor> block_step(
    Tensor x, const Tensor& y, const Tensor& gain, int64_t groups, double eps,
    const Tensor& positions, const OptTensor& taps, const OptTensor& tail,
    const OptTensor& slots, int64_t n_decode, const OptTensor& rows,
    bool keep, const OptTensor& y2, const OptTensor& gain1,
    const OptTensor& gain2, const OptTensor& part_ids,
    const OptTensor& part_w, const OptTensor& part_h, int64_t part_limit,
    const OptTensor& y_bias) {
  rlli::BlockArgs a{};
  a.f32 = act_f32(y, "y");
  TORCH_CHECK(x.dim() == 2 && y.dim() == (part_ids ? 3 : 2) &&
              y.size(0) == x.size(0) && y.size(-1) == x.size(1),
              "y/residual mismatch");
  a.y = y.data_ptr();
  if (y_bias) {
    TORCH_CHECK(!part_ids && !y2, "a bias goes with a single output");
    a.y_bias = f32_vec(*y_bias, x.size(1), "y_bias");
  }
  if (part_ids) {
    TORCH_CHECK(part_w.has_value() && part_h.has_value() && !y2,
                "parts come with weights and the block's input");
    a.parts = int(y.size(1));
    a.part_limit = int(part_limit);
    a.part_ids = i32(*part_ids, "part_ids");
    TORCH_CHECK(part_ids->numel() == y.size(0) * y.size(1),
                "one id per part");
    a.part_w = f32_vec(*part_w, part_ids->numel(), "part_w");
    same_act(*part_h, y, "part_h");
    TORCH_CHECK(part_h->sizes() == x.sizes(), "part_h/residual mismatch");
    a.part_h = part_h->data_ptr();
  }
  if (y2) {
    same_act(*y2, y, "y2");
    TORCH_CHECK(y2->sizes() == y.sizes() && gain1.has_value() &&
                gain2.has_value(), "two outputs have a norm each");
    a.y2 = y2->data_ptr();
    a.gain1 = f32_vec(*gain1, x.size(1), "gain1");
    a.gain2 = f32_vec(*gain2, x.size(1), "gain2");
  }
  a.n = int(x.size(0));
  a.keep = keep;
  if (rows) {
    TORCH_CHECK(rows->is_cuda() && rows->is_contiguous() &&
                rows->scalar_type() == at::kLong && !keep);
    a.rows = rows->data_ptr<int64_t>();
    a.n = int(rows->numel());
  }
  return block_run(a, y, x, gain, groups, eps, positions, taps, tail, slots,
                   n_decode);
}

void conv_prompt(const Tensor& h, const Tensor& taps, const OptTensor& tail,
                 const Tensor& spans, const Tensor& portions, Tensor out,
                 bool silu) {
  rlli::ConvArgs a{};
  TORCH_CHECK(h.dim() == 2 && (taps.dim() == 2 || taps.dim() == 3) &&
              out.dim() == taps.dim());
  const int64_t rows = h.size(0), W = h.size(1);
  a.f32 = h.scalar_type() == at::kFloat;
  TORCH_CHECK(a.f32 || h.scalar_type() == at::kBFloat16,
              "h must be bf16 or f32");
  a.h_stride = row_stride(h, h, rows, W, "h");
  a.branches = 1;
  if (taps.dim() == 3) {
    a.branches = int(taps.size(0));
    TORCH_CHECK(out.size(0) == a.branches && a.branches >= 1,
                "one output per branch");
    a.branch_stride = out.stride(0);
    a.out_stride = row_stride(out.select(0, 0), h, rows, W, "out");
    TORCH_CHECK(a.branches == 1 || a.branch_stride >= rows * a.out_stride,
                "branches of out overlap");
  } else {
    a.out_stride = row_stride(out, h, rows, W, "out");
  }
  a.width = int(W);
  a.n_taps = int(taps.size(-2));
  a.silu = silu;
  a.h = h.data_ptr();
  a.out = out.data_ptr();
  a.taps = f32_vec(taps, int64_t(a.branches) * a.n_taps * a.width, "taps");
  check_tail(tail, h, a.n_taps, a.width);
  a.ring = 1;
  if (a.n_taps > 1) {
    a.tail = tail->data_ptr();
    a.ring = int(tail->size(1));
  }
  a.spans = i32(spans, "spans");
  a.portions = i32(portions, "portions");
  TORCH_CHECK(spans.dim() == 2 && spans.size(0) == 5 &&
              portions.dim() == 2 && portions.size(0) == 5);
  a.n_spans = int(spans.size(1));
  a.n_portions = int(portions.size(1));
  c10::hip::HIPGuardMasqueradingAsCUDA guard(h.device());
  rlli::launch_conv_prompt(a, stream_of(h));
  check_launch("conv_prompt");
}

void gate_act(const Tensor& gate_up, Tensor out, c10::string_view act,
              double limit) {
  const bool f32 = act_f32(gate_up, "gate_up");
  TORCH_CHECK(gate_up.dim() == 2 && gate_up.size(1) % 2 == 0);
  const int64_t rows = gate_up.size(0), ff = gate_up.size(1) / 2;
  const int64_t stride = row_stride(out, gate_up, rows, ff, "out");
  TORCH_CHECK(act == "relu" || act == "silu" || act == "clamp_glu",
              "act must be relu, silu or clamp_glu");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(gate_up.device());
  rlli::launch_gate_act(gate_up.data_ptr(), out.data_ptr(), int(rows),
                        int(ff), stride,
                        act == "relu"   ? rlli::kActRelu
                        : act == "silu" ? rlli::kActSilu
                                        : rlli::kActClampGlu,
                        float(limit), f32, stream_of(gate_up));
  check_launch("gate_act");
}

Tensor soft_cap(const Tensor& x, double cap) {
  const bool f32 = act_f32(x, "x");
  TORCH_CHECK(cap > 0, "cap must be positive");
  Tensor out = at::empty(x.sizes(), x.options().dtype(at::kFloat));
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  rlli::launch_soft_cap(x.data_ptr(), out.data_ptr<float>(), x.numel(),
                        float(cap), f32, stream_of(x));
  check_launch("soft_cap");
  return out;
}

}  // namespace

TORCH_LIBRARY(rlli_blk, m) {
  m.def("block_embed(Tensor ids, Tensor table, Tensor? pos_table, "
        "Tensor positions, Tensor(a!) x, Tensor gain, int groups, float eps, "
        "Tensor? taps, Tensor(b!)? tail, Tensor? slots, int n_decode, "
        "float scale) -> (Tensor, Tensor)");
  m.def("block_step(Tensor(a!) x, Tensor y, Tensor gain, int groups, "
        "float eps, Tensor positions, Tensor? taps, Tensor(b!)? tail, "
        "Tensor? slots, int n_decode, Tensor? rows, bool keep, Tensor? y2, "
        "Tensor? gain1, Tensor? gain2, Tensor? part_ids=None, "
        "Tensor? part_w=None, Tensor? part_h=None, int part_limit=0, "
        "Tensor? y_bias=None) -> (Tensor, Tensor)");
  m.def("conv_prompt(Tensor h, Tensor taps, Tensor(a!)? tail, Tensor spans, "
        "Tensor portions, Tensor(b!) out, bool silu) -> ()");
  m.def("gate_act(Tensor gate_up, Tensor(a!) out, str act, float limit) "
        "-> ()");
  m.def("soft_cap(Tensor x, float cap) -> Tensor");
}

TORCH_LIBRARY_IMPL(rlli_blk, CUDA, m) {
  m.impl("block_embed", &block_embed);
  m.impl("block_step", &block_step);
  m.impl("conv_prompt", &conv_prompt);
  m.impl("gate_act", &gate_act);
  m.impl("soft_cap", &soft_cap);
}
