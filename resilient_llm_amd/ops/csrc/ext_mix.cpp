// Torch bindings (torch.ops.rlli_mix.*) of the mixed-layer model kernels.
// Every shape, dtype and index-table assumption of a kernel is checked
// here before it is launched.

#include "ext_common.h"
#include "mix.h"

namespace {

using namespace rlli_ext;

// ---------------------------------------------------------------- hyper
void check_streams(const Tensor& x) {
  TORCH_CHECK(x.dim() == 3 && x.is_cuda() && x.is_contiguous() &&
              x.scalar_type() == at::kFloat, "streams must be f32 [T,S,W]");
  TORCH_CHECK(x.size(1) >= 1 && x.size(1) <= 8, "1..8 residual streams");
  TORCH_CHECK(x.size(2) % 8 == 0 && x.size(2) <= 8192,
              "width must be a multiple of 8, at most 8192");
}

Tensor hyper_embed(const Tensor& ids, const Tensor& table,
                   const Tensor& w_embed, Tensor x, const Tensor& in_w,
                   const Tensor& gain, double eps) {
  rlli::HyperArgs a{};
  check_streams(x);
  a.f32 = act_f32(table, "table");
  a.n = int(x.size(0));
  a.streams = int(x.size(1));
  a.width = int(x.size(2));
  TORCH_CHECK(table.dim() == 2 && table.size(1) == a.width);
  a.table = table.data_ptr();
  a.ids = i32(ids, "ids");
  TORCH_CHECK(ids.numel() == a.n, "ids/streams mismatch");
  a.w_embed = f32_vec(w_embed, a.width, "w_embed");
  a.x = x.data_ptr<float>();
  a.in_w = f32_vec(in_w, a.streams, "in_w");
  a.gain = f32_vec(gain, a.width, "gain");
  a.eps = float(eps);
  a.parts = 1;
  Tensor h = at::empty({a.n, a.width}, table.options());
  a.h = h.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  rlli::launch_hyper_embed(a, stream_of(x));
  check_launch("hyper_embed");
  return h;
}

// in_w absent: the plain sum of the streams; rows: final subset, streams
// are then left as they are
Tensor hyper_step(Tensor x, const Tensor& y, const Tensor& mix,
                  const Tensor& out_w, const OptTensor& in_w,
                  const Tensor& gain, double eps, const OptTensor& rows,
                  bool keep) {
  rlli::HyperArgs a{};
  check_streams(x);
  a.f32 = act_f32(y, "y");
  a.streams = int(x.size(1));
  a.width = int(x.size(2));
  const int64_t T = x.size(0);
  TORCH_CHECK(y.numel() % (T * a.width ? T * a.width : 1) == 0 &&
              y.size(0) == T && y.size(-1) == a.width, "y/streams mismatch");
  a.parts = T ? int(y.numel() / (T * a.width)) : 1;
  a.x = x.data_ptr<float>();
  a.y = y.data_ptr();
  a.mix = f32_vec(mix, int64_t(a.streams) * a.streams, "mix");
  a.out_w = f32_vec(out_w, a.streams, "out_w");
  a.in_w = in_w ? f32_vec(*in_w, a.streams, "in_w") : nullptr;
  a.gain = f32_vec(gain, a.width, "gain");
  a.eps = float(eps);
  a.n = int(T);
  a.keep = keep;
  if (rows) {
    TORCH_CHECK(rows->is_cuda() && rows->is_contiguous() &&
                rows->scalar_type() == at::kLong && !keep);
    a.rows = rows->data_ptr<int64_t>();
    a.n = int(rows->numel());
  }
  Tensor h = at::empty({a.n, a.width}, y.options());
  a.h = h.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  rlli::launch_hyper_step(a, stream_of(x));
  check_launch("hyper_step");
  return h;
}

Tensor relu2(const Tensor& x) {
  const bool f32 = act_f32(x, "x");
  Tensor out = at::empty_like(x);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(x.device());
  rlli::launch_relu2(x.data_ptr(), out.data_ptr(), x.numel(), f32,
                     stream_of(x));
  check_launch("relu2");
  return out;
}

// --------------------------------------------------------- window attention
rlli::WindowAttnArgs window_args(const Tensor& qkv, const Tensor& k_cache,
                                 const Tensor& v_cache,
                                 const Tensor& positions,
                                 const Tensor& cos_sin, const Tensor& slots,
                                 const Tensor& block_tables,
                                 const OptTensor& sink, double scale,
                                 int64_t n_q, int64_t window,
                                 int64_t keep_first, bool has_kv) {
  rlli::WindowAttnArgs a{};
  a.f32 = act_f32(qkv, "qkv");
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 4 &&
              k_cache.is_cuda() && k_cache.is_contiguous() &&
              v_cache.is_cuda() && v_cache.is_contiguous() &&
              k_cache.scalar_type() == v_cache.scalar_type() &&
              k_cache.size(0) == v_cache.size(0) &&
              k_cache.size(1) == v_cache.size(1) &&
              k_cache.size(2) == v_cache.size(2), "k/v cache mismatch");
  if (k_cache.scalar_type() == at::kFloat8_e4m3fn) {
    TORCH_CHECK(!a.f32, "fp8 cache needs bf16 activations");
    a.cache = rlli::kCacheFP8;
  } else {
    TORCH_CHECK(k_cache.scalar_type() == qkv.scalar_type(),
                "cache dtype must match the activations (or be fp8)");
    a.cache = a.f32 ? rlli::kCacheF32 : rlli::kCacheBF16;
  }
  a.n_q = int(n_q);
  a.n_kv = int(k_cache.size(1));
  a.block_size = int(k_cache.size(2));
  a.dim = int(k_cache.size(3));
  a.vdim = int(v_cache.size(3));
  a.rows = int(qkv.size(0));
  a.stride = int(qkv.size(1));
  a.has_kv = has_kv;
  TORCH_CHECK(a.n_q % a.n_kv == 0, "heads must be a multiple of kv heads");
  TORCH_CHECK(a.vdim <= 512 && a.dim <= 4096, "head sizes out of range");
  TORCH_CHECK(a.stride == a.n_q * a.dim +
              (has_kv ? a.n_kv * (a.dim + a.vdim) : 0), "qkv width mismatch");
  TORCH_CHECK(window >= 1 && keep_first >= 0);
  a.window = int(std::min<int64_t>(window, 1 << 30));
  a.keep_first = int(std::min<int64_t>(keep_first, 1 << 30));
  a.scale = float(scale);
  a.qkv = qkv.data_ptr();
  a.qkv_rw = qkv.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  a.positions = i32(positions, "positions");
  a.slots = i32(slots, "slots");
  TORCH_CHECK(positions.numel() == a.rows && slots.numel() == a.rows,
              "one position and slot per row");
  TORCH_CHECK(cos_sin.is_cuda() && cos_sin.is_contiguous() &&
              cos_sin.scalar_type() == at::kFloat && cos_sin.dim() == 2 &&
              cos_sin.size(1) % 2 == 0 && cos_sin.size(1) <= a.dim);
  a.cos_sin = cos_sin.data_ptr<float>();
  a.rot = int(cos_sin.size(1));
  a.block_tables = i32(block_tables, "block_tables");
  TORCH_CHECK(block_tables.dim() == 2);
  a.max_blocks = int(block_tables.size(1));
  a.sink = sink ? f32_vec(*sink, a.n_q, "sink") : nullptr;
  return a;
}

// prompt rows: rotate + cache, then attend tile by tile; qkv is rotated
// in place
Tensor window_prefill(const Tensor& qkv, const Tensor& k_cache,
                      const Tensor& v_cache, const Tensor& positions,
                      const Tensor& cos_sin, const Tensor& slots,
                      const Tensor& block_tables, const Tensor& tiles,
                      int64_t tile_rows, const OptTensor& sink, double scale,
                      int64_t n_q, int64_t window, int64_t keep_first,
                      bool has_kv) {
  auto a = window_args(qkv, k_cache, v_cache, positions, cos_sin, slots,
                       block_tables, sink, scale, n_q, window, keep_first,
                       has_kv);
  a.tiles = i32(tiles, "tiles");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4);
  a.n_tiles = int(tiles.size(1));
  a.tile_rows = int(tile_rows);
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  auto st = stream_of(qkv);
  rlli::launch_window_rope_append(a, st);
  if (rlli::window_fast_ok(a)) {
    TORCH_CHECK(tile_rows ==
                32 * rlli::window_prefill_sub_tiles(a.n_q / a.n_kv),
                "tile height does not fit the head grouping");
    rlli::launch_window_prefill(a, st);
  } else {
    rlli::launch_window_rows(a, false, st);
  }
  check_launch("window_prefill");
  return out;
}

int64_t window_tile_rows(int64_t group) {
  return 32 * rlli::window_prefill_sub_tiles(int(group));
}

Tensor window_decode(const Tensor& qkv, const Tensor& k_cache,
                     const Tensor& v_cache, const Tensor& positions,
                     const Tensor& cos_sin, const Tensor& slots,
                     const Tensor& block_tables, const OptTensor& sink,
                     double scale, int64_t n_q, int64_t window,
                     int64_t keep_first, bool has_kv) {
  auto a = window_args(qkv, k_cache, v_cache, positions, cos_sin, slots,
                       block_tables, sink, scale, n_q, window, keep_first,
                       has_kv);
  TORCH_CHECK(block_tables.size(0) == a.rows, "one block table per row");
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  auto st = stream_of(qkv);
  if (!rlli::window_fast_ok(a)) {
    rlli::launch_window_rope_append(a, st);
    rlli::launch_window_rows(a, true, st);
    check_launch("window_decode");
    return out;
  }
  const int group = a.n_q / a.n_kv;
  const int hb = rlli::window_decode_heads_per_wg(group);
  const int64_t wgs = int64_t(std::max(a.rows, 1)) * a.n_kv *
                      ((group + hb - 1) / hb);
  // at most one split per 4 visible 16-token steps (one per wave)
  const int64_t reach = std::min<int64_t>(
      int64_t(a.max_blocks) * a.block_size,
      int64_t(a.window) + a.keep_first + 32);
  const int64_t useful = std::max<int64_t>(1, reach / 64);
  a.n_split = int(std::min<int64_t>(
      {16, useful, std::max<int64_t>(1, (512 + wgs - 1) / wgs)}));
  Tensor pa, pm;
  if (a.n_split > 1) {
    auto fo = qkv.options().dtype(at::kFloat);
    pa = at::empty({a.rows, n_q, a.n_split, a.vdim}, fo);
    pm = at::empty({a.rows, n_q, a.n_split, 2}, fo);
    a.part_acc = pa.data_ptr<float>();
    a.part_ml = pm.data_ptr<float>();
  }
  rlli::launch_window_decode(a, st);
  check_launch("window_decode");
  return out;
}

// ------------------------------------------------------------------ moe
void moe_sizes(rlli::MoeArgs& a, const Tensor& h, const Tensor& router,
               int64_t top) {
  a.f32 = act_f32(h, "h");
  same_act(router, h, "router");
  TORCH_CHECK(h.dim() == 2 && router.dim() == 2 &&
              router.size(1) == h.size(1));
  a.rows = int(h.size(0));
  a.width = int(h.size(1));
  a.experts = int(router.size(0));
  a.top = int(top);
  TORCH_CHECK(a.width % 8 == 0, "width must be a multiple of 8");
  TORCH_CHECK(a.experts >= 1 && a.experts <= 256 && a.top >= 1 &&
              a.top <= a.experts, "1 <= top <= experts <= 256");
  a.h = h.data_ptr();
  a.router = router.data_ptr();
}

std::tuple<Tensor, Tensor> moe_route(const Tensor& h, const Tensor& router,
                                     int64_t top) {
  rlli::MoeArgs a{};
  moe_sizes(a, h, router, top);
  Tensor ids = at::empty({a.rows, top}, h.options().dtype(at::kInt));
  Tensor w = at::empty({a.rows, top}, h.options().dtype(at::kFloat));
  a.ids = ids.data_ptr<int32_t>();
  a.weights = w.data_ptr<float>();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(h.device());
  rlli::launch_moe_route(a, stream_of(h));
  check_launch("moe_route");
  return {ids, w};
}

// [rows, top, width]: one output row per (token, choice)
Tensor moe_experts(const Tensor& h, const Tensor& router, const Tensor& w_up,
                   const Tensor& w_down, int64_t top, double limit) {
  rlli::MoeArgs a{};
  moe_sizes(a, h, router, top);
  same_act(w_up, h, "w_up");
  same_act(w_down, h, "w_down");
  TORCH_CHECK(w_up.dim() == 5 && w_up.size(0) == a.experts &&
              w_up.size(2) == 2 && w_up.size(3) == 16 &&
              w_up.size(4) == a.width, "w_up layout");
  a.ffp = int(w_up.size(1)) * 16;
  TORCH_CHECK(a.ffp % 64 == 0 && w_down.dim() == 3 &&
              w_down.size(0) == a.experts && w_down.size(1) == a.width &&
              w_down.size(2) == a.ffp, "w_down layout");
  a.limit = float(limit);
  a.w_up = w_up.data_ptr();
  a.w_down = w_down.data_ptr();
  const int64_t P = int64_t(a.rows) * top;
  // the tiled GEMMs index rows and one expert's weights with 32 bits
  const int64_t wide = std::max<int64_t>(a.width, a.ffp);
  TORCH_CHECK(P * wide < (int64_t(1) << 31) &&
              2 * int64_t(a.ffp) * a.width < (int64_t(1) << 31),
              "too many rows or too wide an expert for one call");
  // tall tiles once experts have enough rows each to fill them
  a.tile_m = (a.f32 || a.width % 64 != 0 || P < int64_t(48) * a.experts)
                 ? 16
                 : P < int64_t(384) * a.experts ? 128 : 256;
  a.max_tiles = int(P / a.tile_m + std::min<int64_t>(a.experts, P));
  auto io = h.options().dtype(at::kInt);
  Tensor ids = at::empty({a.rows, top}, io);
  Tensor w = at::empty({a.rows, top}, h.options().dtype(at::kFloat));
  Tensor plan = at::empty({P + 3 * int64_t(a.max_tiles) + 2 * a.experts}, io);
  Tensor act = at::empty({P, a.ffp}, h.options());
  Tensor y = at::empty({a.rows, top, a.width}, h.options());
  a.ids = ids.data_ptr<int32_t>();
  a.weights = w.data_ptr<float>();
  a.perm = plan.data_ptr<int32_t>();
  a.tile_expert = a.perm + P;
  a.tile_row0 = a.tile_expert + a.max_tiles;
  a.tile_rows = a.tile_row0 + a.max_tiles;
  a.counters = a.tile_rows + a.max_tiles;
  a.act = act.data_ptr();
  a.y = y.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(h.device());
  auto st = stream_of(h);
  rlli::launch_moe_route(a, st);
  rlli::launch_moe_plan(a, st);
  rlli::launch_moe_experts(a, st);
  check_launch("moe_experts");
  return y;
}

}  // namespace

TORCH_LIBRARY(rlli_mix, m) {
  m.def("hyper_embed(Tensor ids, Tensor table, Tensor w_embed, "
        "Tensor(a!) x, Tensor in_w, Tensor gain, float eps) -> Tensor");
  m.def("hyper_step(Tensor(a!) x, Tensor y, Tensor mix, Tensor out_w, "
        "Tensor? in_w, Tensor gain, float eps, Tensor? rows, bool keep) "
        "-> Tensor");
  m.def("relu2(Tensor x) -> Tensor");
  m.def("window_tile_rows(int group) -> int", &window_tile_rows);
  m.def("window_prefill(Tensor(a!) qkv, Tensor(b!) k_cache, "
        "Tensor(c!) v_cache, Tensor positions, Tensor cos_sin, Tensor slots, "
        "Tensor block_tables, Tensor tiles, int tile_rows, Tensor? sink, "
        "float scale, int n_q, int window, int keep_first, bool has_kv) "
        "-> Tensor");
  m.def("window_decode(Tensor(a!) qkv, Tensor(b!) k_cache, "
        "Tensor(c!) v_cache, Tensor positions, Tensor cos_sin, Tensor slots, "
        "Tensor block_tables, Tensor? sink, float scale, int n_q, "
        "int window, int keep_first, bool has_kv) -> Tensor");
  m.def("moe_route(Tensor h, Tensor router, int top) -> (Tensor, Tensor)");
  m.def("moe_experts(Tensor h, Tensor router, Tensor w_up, Tensor w_down, "
        "int top, float limit) -> Tensor");
}

TORCH_LIBRARY_IMPL(rlli_mix, CUDA, m) {
  m.impl("hyper_embed", &hyper_embed);
  m.impl("hyper_step", &hyper_step);
  m.impl("relu2", &relu2);
  m.impl("window_prefill", &window_prefill);
  m.impl("window_decode", &window_decode);
  m.impl("moe_route", &moe_route);
  m.impl("moe_experts", &moe_experts);
}
