// Torch bindings (torch.ops.rlli_mix.*) of the mixed-layer model kernels.
// Every shape, dtype and index-table assumption of a kernel is checked
// here before it is launched.

#include "ext_window.h"
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
// tiled prompt rows, rotated and cached before
Tensor window_tiled(const Tensor& qkv, const Tensor& k_cache,
                    const Tensor& v_cache, const Tensor& block_tables,
                    const Tensor& tiles, int64_t tile_rows,
                    const OptTensor& sink, double scale, int64_t n_q,
                    int64_t window, int64_t keep_first, bool has_kv) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, has_kv, scale, window,
                       keep_first, sink);
  window_tables(a, block_tables);
  window_tiles(a, tiles, tile_rows);
  TORCH_CHECK(!a.f32 && a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 256 &&
              a.vdim <= 256, "head sizes out of range");
  TORCH_CHECK(tile_rows ==
              32 * rlli::window_prefill_sub_tiles(a.n_q / a.n_kv),
              "tile height does not fit the head grouping");
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  rlli::launch_window_prefill(a, stream_of(qkv));
  check_launch("window_tiled");
  return out;
}

int64_t window_tile_rows(int64_t group) {
  return 32 * rlli::window_prefill_sub_tiles(int(group));
}

// ------------------------------------------------------------------ moe
void moe_sizes(rlli::MoeArgs& a, const Tensor& h, const Tensor& router,
               int64_t top, int64_t experts) {
  a.f32 = act_f32(h, "h");
  same_act(router, h, "router");
  TORCH_CHECK(h.dim() == 2 && router.dim() == 2 &&
              router.size(1) == h.size(1));
  a.rows = int(h.size(0));
  a.width = int(h.size(1));
  a.routes = int(router.size(0));
  a.experts = int(experts);
  a.top = int(top);
  a.groups = a.keep = 1;
  TORCH_CHECK(a.width % 8 == 0, "width must be a multiple of 8");
  TORCH_CHECK(a.experts >= 1 && a.experts <= a.routes && a.routes <= 256 &&
              a.top >= 1 && a.top <= a.routes,
              "1 <= top <= experts <= 256");
  a.h = h.data_ptr();
  a.router = router.data_ptr();
}

// softmax scores, a correction of the choice, groups
void moe_choice(rlli::MoeArgs& a, const OptTensor& correction,
                int64_t groups, int64_t keep) {
  a.softmax = true;
  a.correction = correction ? f32_vec(*correction, a.routes, "correction")
                            : nullptr;
  a.groups = int(groups);
  a.keep = int(keep);
  TORCH_CHECK(groups >= 1 && a.routes % groups == 0 && keep >= 1 &&
              keep <= groups && keep * (a.routes / groups) >= a.top,
              "groups must divide the routes, those kept hold the choice");
}

// the two GEMMs over [rows, top] choices: y [rows, top, width]
Tensor moe_run(rlli::MoeArgs& a, const Tensor& h, Tensor& ids, Tensor& w) {
  const int64_t P = int64_t(a.rows) * a.top;
  // the tiled GEMMs index rows and one expert's weights with 32 bits
  const int64_t wide = std::max<int64_t>(a.width, a.ffp);
  TORCH_CHECK(P * wide < (int64_t(1) << 31) &&
              (a.gated ? 2 : 1) * int64_t(a.ffp) * a.width <
                  (int64_t(1) << 31),
              "too many rows or too wide an expert for one call");
  // tall tiles once experts have enough rows each to fill them
  const int64_t each = P / a.routes;
  a.tile_m = (a.f32 || a.width % 64 != 0 || each < 48) ? 16
             : each < 384                              ? 128
                                                       : 256;
  a.max_tiles = int(P / a.tile_m + std::min<int64_t>(a.experts, P));
  auto io = h.options().dtype(at::kInt);
  ids = at::empty({a.rows, a.top}, io);
  w = at::empty({a.rows, a.top}, h.options().dtype(at::kFloat));
  Tensor plan = at::empty({P + 3 * int64_t(a.max_tiles) + 2 * a.experts}, io);
  Tensor act = at::empty({P, a.ffp}, h.options());
  Tensor y = at::empty({a.rows, a.top, a.width}, h.options());
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

// the router alone
std::tuple<Tensor, Tensor> moe_pick(rlli::MoeArgs& a, const Tensor& h) {
  Tensor ids = at::empty({a.rows, a.top}, h.options().dtype(at::kInt));
  Tensor w = at::empty({a.rows, a.top}, h.options().dtype(at::kFloat));
  a.ids = ids.data_ptr<int32_t>();
  a.weights = w.data_ptr<float>();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(h.device());
  rlli::launch_moe_route(a, stream_of(h));
  check_launch("moe_route");
  return {ids, w};
}

std::tuple<Tensor, Tensor> moe_route(const Tensor& h, const Tensor& router,
                                     int64_t top) {
  rlli::MoeArgs a{};
  moe_sizes(a, h, router, top, router.size(0));
  return moe_pick(a, h);
}

std::tuple<Tensor, Tensor> moe_route_softmax(const Tensor& h,
                                             const Tensor& router,
                                             const OptTensor& correction,
                                             int64_t top, int64_t groups,
                                             int64_t keep) {
  rlli::MoeArgs a{};
  moe_sizes(a, h, router, top, router.size(0));
  moe_choice(a, correction, groups, keep);
  return moe_pick(a, h);
}

void down_sizes(rlli::MoeArgs& a, const Tensor& h, const Tensor& w_down) {
  same_act(w_down, h, "w_down");
  TORCH_CHECK(a.ffp % 64 == 0 && w_down.dim() == 3 &&
              w_down.size(0) == a.experts && w_down.size(1) == a.width &&
              w_down.size(2) == a.ffp, "w_down layout");
  a.w_down = w_down.data_ptr();
}

// [rows, top, width]: one output row per (token, choice)
Tensor moe_experts(const Tensor& h, const Tensor& router, const Tensor& w_up,
                   const Tensor& w_down, int64_t top, double limit) {
  rlli::MoeArgs a{};
  moe_sizes(a, h, router, top, router.size(0));
  same_act(w_up, h, "w_up");
  TORCH_CHECK(w_up.dim() == 5 && w_up.size(0) == a.experts &&
              w_up.size(2) == 2 && w_up.size(3) == 16 &&
              w_up.size(4) == a.width, "w_up layout");
  a.ffp = int(w_up.size(1)) * 16;
  a.w_up = w_up.data_ptr();
  down_sizes(a, h, w_down);
  a.gated = true;
  a.limit = float(limit);
  Tensor ids, w;
  return moe_run(a, h, ids, w);
}

// the same for squared-relu experts, with the choice: a consumer that sums
// a token's rows skips identity experts' rows (never written) and adds their
// weight of h
std::tuple<Tensor, Tensor, Tensor> moe_relu2(
    const Tensor& h, const Tensor& router, const OptTensor& correction,
    const Tensor& w_up, const Tensor& w_down, int64_t top, int64_t groups,
    int64_t keep) {
  rlli::MoeArgs a{};
  moe_sizes(a, h, router, top, w_up.size(0));
  moe_choice(a, correction, groups, keep);
  same_act(w_up, h, "w_up");
  TORCH_CHECK(w_up.dim() == 3 && w_up.size(2) == a.width, "w_up layout");
  a.ffp = int(w_up.size(1));
  a.w_up = w_up.data_ptr();
  down_sizes(a, h, w_down);
  Tensor ids, w;
  Tensor y = moe_run(a, h, ids, w);
  return {y, ids, w};
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
  m.def("window_tiled(Tensor qkv, Tensor k_cache, Tensor v_cache, "
        "Tensor block_tables, Tensor tiles, int tile_rows, Tensor? sink, "
        "float scale, int n_q, int window, int keep_first, bool has_kv) "
        "-> Tensor");
  m.def("moe_route(Tensor h, Tensor router, int top) -> (Tensor, Tensor)");
  m.def("moe_experts(Tensor h, Tensor router, Tensor w_up, Tensor w_down, "
        "int top, float limit) -> Tensor");
  m.def("moe_route_softmax(Tensor h, Tensor router, Tensor? correction, "
        "int top, int groups, int keep) -> (Tensor, Tensor)");
  m.def("moe_relu2(Tensor h, Tensor router, Tensor? correction, "
        "Tensor w_up, Tensor w_down, int top, int groups, int keep) "
        "-> (Tensor, Tensor, Tensor)");
}

TORCH_LIBRARY_IMPL(rlli_mix, CUDA, m) {
  m.impl("hyper_embed", &hyper_embed);
  m.impl("hyper_step", &hyper_step);
  m.impl("relu2", &relu2);
  m.impl("window_tiled", &window_tiled);
  m.impl("moe_route", &moe_route);
  m.impl("moe_experts", &moe_experts);
  m.impl("moe_route_softmax", &moe_route_softmax);
  m.impl("moe_relu2", &moe_relu2);
}
