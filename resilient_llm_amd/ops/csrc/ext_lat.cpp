// Torch bindings (torch.ops.rlli_lat.*) of the parallel-block and latent
// attention kernels.

#include "ext_common.h"
#include "lat.h"

namespace {

using namespace rlli_ext;

int cache_kind(const Tensor& cache, bool f32) {
  TORCH_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 4 &&
              cache.size(1) == 1,
              "latent cache must be [blocks, 1, block, rank]");
  if (cache.scalar_type() == at::kFloat8_e4m3fn) {
    TORCH_CHECK(!f32, "fp8 cache needs bf16 activations");
    return rlli::kCacheFP8;
  }
  TORCH_CHECK(cache.scalar_type() == (f32 ? at::kFloat : at::kBFloat16),
              "cache dtype must match the activations (or be fp8)");
  return f32 ? rlli::kCacheF32 : rlli::kCacheBF16;
}

// ---------------------------------------------------------------- block
void check_tail(const OptTensor& tail, const Tensor& like, int n_taps,
                int width) {
  if (n_taps == 1) return;
  TORCH_CHECK(tail.has_value(), "a convolution over time needs its state");
  same_act(*tail, like, "tail");
  TORCH_CHECK(tail->dim() == 3 && tail->size(1) == n_taps - 1 &&
              tail->size(2) == width, "tail must be [slots, taps - 1, width]");
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
  if (taps) {
    TORCH_CHECK(taps->dim() == 2 && !a.rows, "taps must be [taps, width]");
    a.n_taps = int(taps->size(0));
    a.taps = f32_vec(*taps, int64_t(a.n_taps) * a.width, "taps");
    check_tail(tail, act, a.n_taps, a.width);
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
    hc = at::empty({a.n, a.width}, act.options());
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
    const OptTensor& slots, int64_t n_decode) {
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
  a.keep = true;
  return block_run(a, table, x, gain, groups, eps, positions, taps, tail,
                   slots, n_decode);
}

std::tuple<Tensor, Tensor> block_step(
    Tensor x, const Tensor& y, const Tensor& gain, int64_t groups, double eps,
    const Tensor& positions, const OptTensor& taps, const OptTensor& tail,
    const OptTensor& slots, int64_t n_decode, const OptTensor& rows,
    bool keep) {
  rlli::BlockArgs a{};
  a.f32 = act_f32(y, "y");
  TORCH_CHECK(y.dim() == 2 && y.sizes() == x.sizes(), "y/residual mismatch");
  a.y = y.data_ptr();
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
                 const Tensor& spans, const Tensor& portions, Tensor out) {
  rlli::ConvArgs a{};
  a.f32 = act_f32(h, "h");
  same_act(out, h, "out");
  TORCH_CHECK(h.dim() == 2 && h.sizes() == out.sizes() && taps.dim() == 2);
  a.width = int(h.size(1));
  a.n_taps = int(taps.size(0));
  a.h = h.data_ptr();
  a.out = out.data_ptr();
  a.taps = f32_vec(taps, int64_t(a.n_taps) * a.width, "taps");
  check_tail(tail, h, a.n_taps, a.width);
  if (a.n_taps > 1) a.tail = tail->data_ptr();
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

void gate_act(const Tensor& gate_up, Tensor out, c10::string_view act) {
  const bool f32 = act_f32(gate_up, "gate_up");
  TORCH_CHECK(gate_up.dim() == 2 && gate_up.size(1) % 2 == 0);
  const int64_t rows = gate_up.size(0), ff = gate_up.size(1) / 2;
  const int64_t stride = row_stride(out, gate_up, rows, ff, "out");
  TORCH_CHECK(act == "relu" || act == "silu", "act must be relu or silu");
  c10::hip::HIPGuardMasqueradingAsCUDA guard(gate_up.device());
  rlli::launch_gate_act(gate_up.data_ptr(), out.data_ptr(), int(rows),
                        int(ff), stride,
                        act == "relu" ? rlli::kActRelu : rlli::kActSilu, f32,
                        stream_of(gate_up));
  check_launch("gate_act");
}

// --------------------------------------------------------------- latent
Tensor latent_prep(const Tensor& proj, const Tensor& q_norm,
                   const Tensor& kv_norm, double eps, Tensor cache,
                   const Tensor& slots) {
  rlli::LatentPrepArgs a{};
  a.f32 = act_f32(proj, "proj");
  a.cache_kind = cache_kind(cache, a.f32);
  TORCH_CHECK(proj.dim() == 2);
  a.rows = int(proj.size(0));
  a.stride = int(proj.size(1));
  a.q_rank = int(q_norm.numel());
  a.kv_rank = int(cache.size(3));
  TORCH_CHECK(a.stride >= a.q_rank + a.kv_rank, "projection too narrow");
  a.q_norm = f32_vec(q_norm, a.q_rank, "q_norm");
  a.kv_norm = f32_vec(kv_norm, a.kv_rank, "kv_norm");
  a.slots = i32(slots, "slots");
  TORCH_CHECK(slots.numel() == a.rows, "one slot per row");
  a.proj = proj.data_ptr();
  a.cache = cache.data_ptr();
  a.eps = float(eps);
  Tensor cq = at::empty({a.rows, a.q_rank}, proj.options());
  a.cq = cq.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(proj.device());
  rlli::launch_latent_prep(a, stream_of(proj));
  check_launch("latent_prep");
  return cq;
}

void head_linear(const Tensor& x, const Tensor& w, const OptTensor& gate,
                 Tensor out) {
  rlli::HeadLinearArgs a{};
  a.f32 = act_f32(w, "w");
  TORCH_CHECK(w.dim() == 3, "w must be [heads, n, k]");
  a.heads = int(w.size(0));
  a.n = int(w.size(1));
  a.k = int(w.size(2));
  a.rows = int(x.size(0));
  a.x_stride = row_stride(x, w, a.rows, int64_t(a.heads) * a.k, "x");
  a.y_stride = row_stride(out, w, a.rows, int64_t(a.heads) * a.n, "out");
  if (gate) {
    a.gate_stride = row_stride(*gate, w, a.rows, int64_t(a.heads) * a.n,
                               "gate");
    a.gate = gate->data_ptr();
  }
  a.x = x.data_ptr();
  a.w = w.data_ptr();
  a.y = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(w.device());
  rlli::launch_head_linear(a, stream_of(w));
  check_launch("head_linear");
}

bool latent_fast(const Tensor& cache, bool f32) {
  return rlli::latent_fast_ok(int(cache.size(3)), int(cache.size(2)), f32);
}

// the plain kernel, the latent being key and value
void latent_plain(const Tensor& q, const Tensor& cache, int kind,
                  const Tensor& block_tables, double scale, int64_t heads,
                  const OptTensor& positions, const OptTensor& tiles,
                  Tensor out) {
  rlli::WindowAttnArgs a{};
  a.f32 = q.scalar_type() == at::kFloat;
  a.cache = kind;
  a.qkv = q.data_ptr();
  a.k_cache = cache.data_ptr();
  a.v_cache = cache.data_ptr();
  a.rows = int(q.size(0));
  a.n_q = int(heads);
  a.n_kv = 1;
  a.dim = a.vdim = int(cache.size(3));
  a.stride = int(q.size(1));
  a.block_size = int(cache.size(2));
  a.block_tables = i32(block_tables, "block_tables");
  a.max_blocks = int(block_tables.size(1));
  a.window = 1 << 30;
  a.scale = float(scale);
  a.out = out.data_ptr();
  if (tiles) {
    a.tiles = i32(*tiles, "tiles");
    a.n_tiles = int(tiles->size(1));
    a.tile_rows = 32;
  } else {
    a.positions = i32(*positions, "positions");
  }
  rlli::launch_latent_rows(a, !tiles.has_value(), stream_of(q));
}

Tensor latent_attn(const Tensor& q, const Tensor& cache,
                   const Tensor& block_tables, double scale, int64_t heads,
                   const OptTensor& positions, const OptTensor& tiles,
                   const OptTensor& pos0) {
  const bool f32 = act_f32(q, "q");
  const int kind = cache_kind(cache, f32);
  const int64_t R = cache.size(3), rows = q.size(0);
  TORCH_CHECK(q.dim() == 2 && q.size(1) == heads * R,
              "queries must be [rows, heads * rank]");
  TORCH_CHECK(R <= 1024, "kv rank out of range");
  TORCH_CHECK(block_tables.dim() == 2);
  if (tiles) {
    TORCH_CHECK(tiles->dim() == 2 && tiles->size(0) == 4 && pos0.has_value());
  } else {
    TORCH_CHECK(positions.has_value() && positions->numel() == rows &&
                block_tables.size(0) == rows,
                "one position and block table per row");
  }
  Tensor out = at::empty_like(q);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  if (!latent_fast(cache, f32)) {
    latent_plain(q, cache, kind, block_tables, scale, heads, positions,
                 tiles, out);
    check_launch("latent_attn");
    return out;
  }
  rlli::LatentAttnArgs a{};
  a.q = q.data_ptr();
  a.cache = cache.data_ptr();
  a.cache_kind = kind;
  a.block_tables = i32(block_tables, "block_tables");
  a.rows = int(rows);
  a.heads = int(heads);
  a.rank = int(R);
  const int64_t block = cache.size(2);
  while ((int64_t(1) << a.block_shift) < block) ++a.block_shift;
  a.max_blocks = int(block_tables.size(1));
  a.scale = float(scale);
  a.out = out.data_ptr();
  int64_t wgs;
  if (tiles) {
    a.tiles = i32(*tiles, "tiles");
    a.pos0 = i32(*pos0, "pos0");
    a.n_tiles = int(tiles->size(1));
    wgs = a.n_tiles;
  } else {
    a.positions = i32(*positions, "positions");
    const int t = rlli::latent_tile(a.heads, true);
    wgs = rows * ((heads + t - 1) / t);
  }
  // enough workgroups for the chip, at least 128 keys each
  const int64_t most = int64_t(a.max_blocks) * block / 128;
  a.n_split = int(std::max<int64_t>(
      1, std::min<int64_t>({32, most, (512 + wgs - 1) /
                                          std::max<int64_t>(wgs, 1)})));
  Tensor pa, pm;
  if (a.n_split > 1) {
    auto fo = q.options().dtype(at::kFloat);
    pa = at::empty({rows * heads, a.n_split, R}, fo);
    pm = at::empty({rows * heads, a.n_split, 2}, fo);
    a.part_acc = pa.data_ptr<float>();
    a.part_ml = pm.data_ptr<float>();
  }
  rlli::launch_latent_attn(a, stream_of(q));
  check_launch("latent_attn");
  return out;
}

Tensor latent_gather(const Tensor& cache, const Tensor& block_tables,
                     const Tensor& blocks, int64_t tokens) {
  rlli::GatherArgs a{};
  a.cache_kind = cache_kind(cache, false);
  a.rank = int(cache.size(3));
  TORCH_CHECK(a.rank % 8 == 0, "kv rank must be a multiple of 8 here");
  TORCH_CHECK(block_tables.dim() == 2 && blocks.dim() == 2 &&
              blocks.size(0) == 4 &&
              tokens == blocks.size(1) * rlli::kGatherRows);
  a.cache = cache.data_ptr();
  a.block_tables = i32(block_tables, "block_tables");
  a.blocks = i32(blocks, "blocks");
  a.n = int(blocks.size(1));
  a.block_size = int(cache.size(2));
  a.max_blocks = int(block_tables.size(1));
  Tensor out = at::empty({tokens, a.rank},
                         cache.options().dtype(at::kBFloat16));
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(cache.device());
  rlli::launch_latent_gather(a, stream_of(cache));
  check_launch("latent_gather");
  return out;
}

bool expanded_ok(int64_t dim, int64_t vdim) {
  return rlli::expanded_ok(int(dim), int(vdim));
}

void expanded_attn(const Tensor& q, const Tensor& k, const Tensor& vt,
                   const OptTensor& gate, const Tensor& tiles,
                   const Tensor& kv_off, int64_t heads, double scale,
                   Tensor out) {
  rlli::ExpandedAttnArgs a{};
  TORCH_CHECK(!act_f32(q, "q"), "the expanded form is bf16");
  same_act(k, q, "k");
  same_act(vt, q, "vt");
  const int64_t rows = q.size(0);
  TORCH_CHECK(q.dim() == 2 && k.dim() == 2 && vt.dim() == 2 &&
              q.size(1) == k.size(1) && q.size(1) % heads == 0 &&
              vt.size(0) % heads == 0 && vt.size(1) == k.size(0) &&
              k.size(0) % 64 == 0, "q/k/v mismatch");
  a.heads = int(heads);
  a.dim = int(q.size(1) / heads);
  a.vdim = int(vt.size(0) / heads);
  a.tokens = int(k.size(0));
  TORCH_CHECK(rlli::expanded_ok(a.dim, a.vdim), "head sizes out of range");
  a.out_stride = row_stride(out, q, rows, heads * a.vdim, "out");
  TORCH_CHECK(a.out_stride % 4 == 0 &&
              reinterpret_cast<uintptr_t>(out.data_ptr()) % 8 == 0,
              "out rows must be 8-byte aligned");
  if (gate) {
    a.gate_stride = row_stride(*gate, q, rows, heads * a.vdim, "gate");
    TORCH_CHECK(a.gate_stride % 4 == 0 &&
                reinterpret_cast<uintptr_t>(gate->data_ptr()) % 8 == 0,
                "gate rows must be 8-byte aligned");
    a.gate = gate->data_ptr();
  }
  a.q = q.data_ptr();
  a.k = k.data_ptr();
  a.vt = vt.data_ptr();
  a.out = out.data_ptr();
  a.tiles = i32(tiles, "tiles");
  a.kv_off = i32(kv_off, "kv_off");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4);
  a.n_tiles = int(tiles.size(1));
  a.scale = float(scale);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  rlli::launch_expanded_attn(a, stream_of(q));
  check_launch("expanded_attn");
}

}  // namespace

TORCH_LIBRARY(rlli_lat, m) {
  m.def("block_embed(Tensor ids, Tensor table, Tensor? pos_table, "
        "Tensor positions, Tensor(a!) x, Tensor gain, int groups, float eps, "
        "Tensor? taps, Tensor(b!)? tail, Tensor? slots, int n_decode) "
        "-> (Tensor, Tensor)");
  m.def("block_step(Tensor(a!) x, Tensor y, Tensor gain, int groups, "
        "float eps, Tensor positions, Tensor? taps, Tensor(b!)? tail, "
        "Tensor? slots, int n_decode, Tensor? rows, bool keep) "
        "-> (Tensor, Tensor)");
  m.def("conv_prompt(Tensor h, Tensor taps, Tensor(a!)? tail, Tensor spans, "
        "Tensor portions, Tensor(b!) out) -> ()");
  m.def("gate_act(Tensor gate_up, Tensor(a!) out, str act) -> ()");
  m.def("latent_prep(Tensor proj, Tensor q_norm, Tensor kv_norm, float eps, "
        "Tensor(a!) cache, Tensor slots) -> Tensor");
  m.def("head_linear(Tensor x, Tensor w, Tensor? gate, Tensor(a!) out) "
        "-> ()");
  m.def("latent_fast(Tensor cache, bool f32) -> bool");
  m.def("latent_attn(Tensor q, Tensor cache, Tensor block_tables, "
        "float scale, int heads, Tensor? positions, Tensor? tiles, "
        "Tensor? pos0) -> Tensor");
  m.def("latent_gather(Tensor cache, Tensor block_tables, Tensor blocks, "
        "int tokens) -> Tensor");
  m.def("expanded_ok(int dim, int vdim) -> bool", &expanded_ok);
  m.def("expanded_attn(Tensor q, Tensor k, Tensor vt, Tensor? gate, "
        "Tensor tiles, Tensor kv_off, int heads, float scale, "
        "Tensor(a!) out) -> ()");
}

TORCH_LIBRARY_IMPL(rlli_lat, CUDA, m) {
  m.impl("block_embed", &block_embed);
  m.impl("block_step", &block_step);
  m.impl("conv_prompt", &conv_prompt);
  m.impl("gate_act", &gate_act);
  m.impl("latent_prep", &latent_prep);
  m.impl("head_linear", &head_linear);
  m.impl("latent_fast", &latent_fast);
  m.impl("latent_attn", &latent_attn);
  m.impl("latent_gather", &latent_gather);
  m.impl("expanded_attn", &expanded_attn);
}
