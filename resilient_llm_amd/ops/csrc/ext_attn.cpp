// Torch bindings (torch.ops.rlli_attn.*) of paged softmax attention.  Every
// shape, dtype and index-table assumption of a kernel is checked here before
// it is launched.

#include "ext_window.h"

namespace {

using namespace rlli_ext;

// positions, cache slots and rotation of every row, for writing the cache
void append_args(rlli::WindowAttnArgs& a, const Tensor& positions,
                 const OptTensor& cos_sin, const Tensor& slots,
                 const std::optional<double>& v_eps) {
  a.positions = i32(positions, "positions");
  a.slots = i32(slots, "slots");
  TORCH_CHECK(positions.numel() == a.rows && slots.numel() == a.rows,
              "one position and slot per row");
  if (cos_sin) {
    TORCH_CHECK(cos_sin->is_cuda() && cos_sin->is_contiguous() &&
                cos_sin->scalar_type() == at::kFloat && cos_sin->dim() == 2 &&
                cos_sin->size(1) % 2 == 0 && cos_sin->size(1) <= a.dim);
    a.cos_sin = cos_sin->data_ptr<float>();
    a.rot = int(cos_sin->size(1));
  }
  a.v_norm = v_eps.has_value();
  a.v_eps = v_eps ? float(*v_eps) : 0.f;
}

template <typename Args>
void score_args(Args& a, int64_t heads, const OptTensor& r1,
                const OptTensor& r2, double temp_coef, int64_t temp_every) {
  TORCH_CHECK(r1.has_value() == r2.has_value(), "r1 and r2 go together");
  if (r1) {
    a.r1 = f32_vec(*r1, heads, "r1");
    a.r2 = f32_vec(*r2, heads, "r2");
  }
  TORCH_CHECK(temp_every >= 0 && temp_every < (int64_t(1) << 31));
  a.temp_coef = float(temp_coef);
  a.temp_every = int(temp_every);
}

void window_append(const Tensor& qkv, const Tensor& k_cache,
                   const Tensor& v_cache, const Tensor& positions,
                   const OptTensor& cos_sin, const Tensor& slots, int64_t n_q,
                   bool has_kv, std::optional<double> v_eps) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, has_kv);
  append_args(a, positions, cos_sin, slots, v_eps);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  rlli::launch_window_rope_append(a, stream_of(qkv));
  check_launch("window_append");
}

// splits of a decode step that fill the chip, and room for their results;
// ``visible``: the most tokens that a query sees
// ``head_blocks``: workgroups per sequence, kv head and split
void decode_splits(rlli::WindowAttnArgs& a, const Tensor& qkv,
                   int head_blocks, int64_t visible, Tensor& pa, Tensor& pm) {
  const int64_t wgs =
      int64_t(std::max(a.rows, 1)) * a.n_kv * head_blocks;
  // at most one split per 4 visible 16-token steps (one per wave)
  const int64_t reach = std::min<int64_t>(
      int64_t(a.max_blocks) * a.block_size, visible);
  const int64_t useful = std::max<int64_t>(1, reach / 64);
  a.n_split = int(std::min<int64_t>(
      {16, useful, std::max<int64_t>(1, (512 + wgs - 1) / wgs)}));
  if (a.n_split == 1) return;
  auto fo = qkv.options().dtype(at::kFloat);
  pa = at::empty({a.rows, a.n_q, a.maps, a.n_split, a.vdim}, fo);
  pm = at::empty({a.rows, a.n_q, a.maps, a.n_split, 2}, fo);
  a.part_acc = pa.data_ptr<float>();
  a.part_ml = pm.data_ptr<float>();
}

// prompt rows, one wave each, at any sizes
Tensor window_rows(const Tensor& qkv, const Tensor& k_cache,
                   const Tensor& v_cache, const Tensor& block_tables,
                   const Tensor& tiles, int64_t tile_rows,
                   const OptTensor& sink, double scale, int64_t n_q,
                   int64_t window, int64_t keep_first, bool has_kv,
                   const OptTensor& r1, const OptTensor& r2, double temp_coef,
                   int64_t temp_every) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, has_kv, scale, window,
                       keep_first, sink);
  score_args(a, n_q, r1, r2, temp_coef, temp_every);
  window_tables(a, block_tables);
  window_tiles(a, tiles, tile_rows);
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  rlli::launch_window_rows(a, false, stream_of(qkv));
  check_launch("window_rows");
  return out;
}

bool window_fast(const Tensor& k_cache, const Tensor& v_cache, bool f32) {
  rlli::WindowAttnArgs a{};
  a.f32 = f32;
  a.dim = int(k_cache.size(3));
  a.vdim = int(v_cache.size(3));
  a.block_size = int(k_cache.size(2));
  return rlli::window_fast_ok(a);
}

Tensor window_decode(const Tensor& qkv, const Tensor& k_cache,
                     const Tensor& v_cache, const Tensor& positions,
                     const OptTensor& cos_sin, const Tensor& slots,
                     const Tensor& block_tables, const OptTensor& sink,
                     double scale, int64_t n_q, int64_t window,
                     int64_t keep_first, bool has_kv, const OptTensor& r1,
                     const OptTensor& r2, double temp_coef,
                     int64_t temp_every, std::optional<double> v_eps) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, has_kv, scale, window,
                       keep_first, sink);
  append_args(a, positions, cos_sin, slots, v_eps);
  score_args(a, n_q, r1, r2, temp_coef, temp_every);
  window_tables(a, block_tables);
  TORCH_CHECK(block_tables.size(0) == a.rows, "one block table per row");
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  auto st = stream_of(qkv);
  if (!rlli::window_fast_ok(a) || a.stride % 8) {
    rlli::launch_window_rope_append(a, st);
    rlli::launch_window_rows(a, true, st);
    check_launch("window_decode");
    return out;
  }
  const int group = a.n_q / a.n_kv;
  const int hb = rlli::window_decode_heads_per_wg(group);
  Tensor pa, pm;
  decode_splits(a, qkv, (group + hb - 1) / hb,
                int64_t(a.window) + a.keep_first + 32, pa, pm);
  rlli::launch_window_decode(a, st);
  check_launch("window_decode");
  return out;
}

// ------------------------------------------------ differential attention
// chunk, cap, difference, output norm and gate of either kernel's arguments
template <typename Args>
void diff_score(Args& a, int64_t chunk, double cap, double lambda,
                double out_scale, double eps) {
  TORCH_CHECK(chunk >= 1 && chunk <= (int64_t(1) << 30) && cap >= 0.0);
  a.chunk = int(chunk);
  a.cap = float(cap);
  a.lambda = float(lambda);
  a.out_scale = float(out_scale);
  a.eps = float(eps);
}

void diff_append_args(rlli::WindowAttnArgs& a, const Tensor& positions,
                      const OptTensor& cos_sin, const Tensor& slots,
                      const OptTensor& bias, const Tensor& q_norm, const Tensor& k_norm, double eps) {
  append_args(a, positions, cos_sin, slots, std::nullopt);
  if (bias)
    a.bias = f32_vec(*bias, int64_t(a.n_q + a.n_kv) * 2 * a.dim +
                                int64_t(a.n_kv) * a.vdim, "bias");
  a.q_norm = f32_vec(q_norm, a.dim, "q_norm");
  a.k_norm = f32_vec(k_norm, a.dim, "k_norm");
  a.eps = float(eps);
}

void diff_gate(rlli::WindowAttnArgs& a, const Tensor& qkv,
               const OptTensor& gate) {
  if (!gate) return;
  a.gate_stride = row_stride(*gate, qkv, a.rows, a.n_q, "gate");
  a.gate = gate->data_ptr();
}

void diff_append(const Tensor& qkv, const Tensor& k_cache,
                 const Tensor& v_cache, const Tensor& positions,
                 const OptTensor& cos_sin, const Tensor& slots, int64_t n_q,
                 const OptTensor& bias, const Tensor& q_norm,
                 const Tensor& k_norm, double eps) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, true, 1.0, 1, 0, {}, 2);
  diff_append_args(a, positions, cos_sin, slots, bias, q_norm, k_norm, eps);
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  rlli::launch_diff_append(a, stream_of(qkv));
  check_launch("diff_append");
}

// prompt rows, one wave each, at any sizes
Tensor diff_rows(const Tensor& qkv, const Tensor& k_cache,
                 const Tensor& v_cache, const Tensor& block_tables,
                 const Tensor& tiles, int64_t tile_rows,
                 const OptTensor& gate, double scale, int64_t n_q,
                 int64_t chunk, double cap, double lambda, double out_scale,
                 double eps) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, true, scale, 1, 0, {}, 2);
  diff_score(a, chunk, cap, lambda, out_scale, eps);
  diff_gate(a, qkv, gate);
  window_tables(a, block_tables);
  window_tiles(a, tiles, tile_rows);
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  rlli::launch_diff_rows(a, false, stream_of(qkv));
  check_launch("diff_rows");
  return out;
}

Tensor diff_decode(const Tensor& qkv, const Tensor& k_cache,
                   const Tensor& v_cache, const Tensor& positions,
                   const OptTensor& cos_sin, const Tensor& slots,
                   const Tensor& block_tables, const OptTensor& gate,
                   double scale, int64_t n_q, const OptTensor& bias,
                   const Tensor& q_norm, const Tensor& k_norm, int64_t chunk, double cap,
                   double lambda, double out_scale, double eps) {
  auto a = window_args(qkv, k_cache, v_cache, n_q, true, scale, 1, 0, {}, 2);
  diff_append_args(a, positions, cos_sin, slots, bias, q_norm, k_norm, eps);
  diff_score(a, chunk, cap, lambda, out_scale, eps);
  diff_gate(a, qkv, gate);
  window_tables(a, block_tables);
  TORCH_CHECK(block_tables.size(0) == a.rows, "one block table per row");
  Tensor out = at::empty({a.rows, n_q * a.vdim}, qkv.options());
  a.out = out.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(qkv.device());
  auto st = stream_of(qkv);
  if (!rlli::diff_fast_ok(a)) {
    rlli::launch_diff_append(a, st);
    rlli::launch_diff_rows(a, true, st);
    check_launch("diff_decode");
    return out;
  }
  Tensor pa, pm;
  decode_splits(a, qkv, rlli::diff_head_blocks(a.n_q / a.n_kv), chunk, pa,
                pm);
  rlli::launch_diff_decode(a, st);
  check_launch("diff_decode");
  return out;
}

// a sequence's keys [tokens, kv heads * dim] and values, transposed
std::tuple<Tensor, Tensor> kv_gather(const Tensor& k_cache,
                                     const Tensor& v_cache,
                                     const Tensor& block_tables,
                                     const Tensor& blocks, int64_t tokens) {
  TORCH_CHECK(k_cache.dim() == 4 && v_cache.dim() == 4 &&
              k_cache.is_cuda() && k_cache.is_contiguous() &&
              v_cache.is_cuda() && v_cache.is_contiguous() &&
              k_cache.scalar_type() == v_cache.scalar_type() &&
              k_cache.size(0) == v_cache.size(0) &&
              k_cache.size(1) == v_cache.size(1) &&
              k_cache.size(2) == v_cache.size(2), "k/v cache mismatch");
  rlli::KvGatherArgs a{};
  const bool fp8 = k_cache.scalar_type() == at::kFloat8_e4m3fn;
  TORCH_CHECK(fp8 || k_cache.scalar_type() == at::kBFloat16,
              "16-bit or fp8 caches only");
  a.cache_kind = fp8 ? rlli::kCacheFP8 : rlli::kCacheBF16;
  a.n_kv = int(k_cache.size(1));
  a.block_size = int(k_cache.size(2));
  a.dim = int(k_cache.size(3));
  a.vdim = int(v_cache.size(3));
  TORCH_CHECK(rlli::expanded_ok(a.dim, a.vdim), "head sizes out of range");
  TORCH_CHECK(block_tables.dim() == 2 && blocks.dim() == 2 &&
              blocks.size(0) == 4 &&
              tokens == blocks.size(1) * rlli::kKvGatherRows);
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  a.block_tables = i32(block_tables, "block_tables");
  a.max_blocks = int(block_tables.size(1));
  a.blocks = i32(blocks, "blocks");
  a.n = int(blocks.size(1));
  a.tokens = int(tokens);
  auto o = k_cache.options().dtype(at::kBFloat16);
  Tensor k = at::empty({tokens, int64_t(a.n_kv) * a.dim}, o);
  Tensor vt = at::empty({int64_t(a.n_kv) * a.vdim, tokens}, o);
  a.k = k.data_ptr();
  a.vt = vt.data_ptr();
  c10::hip::HIPGuardMasqueradingAsCUDA guard(k_cache.device());
  rlli::launch_kv_gather(a, stream_of(k_cache));
  check_launch("kv_gather");
  return {k, vt};
}

bool expanded_ok(int64_t dim, int64_t vdim, int64_t maps) {
  return rlli::expanded_ok(int(dim), int(vdim), int(maps));
}

rlli::ExpandedAttnArgs expanded_args(const Tensor& q, const Tensor& k,
                                     const Tensor& vt, const Tensor& tiles,
                                     const Tensor& kv_off, int64_t heads,
                                     int64_t kv_heads, int64_t maps,
                                     double scale, Tensor& out) {
  rlli::ExpandedAttnArgs a{};
  TORCH_CHECK(q.scalar_type() == at::kBFloat16, "the tiled form is bf16");
  same_act(k, q, "k");
  same_act(vt, q, "vt");
  const int64_t rows = q.size(0);
  TORCH_CHECK(q.dim() == 2 && k.dim() == 2 && vt.dim() == 2 &&
              kv_heads >= 1 && heads % kv_heads == 0 &&
              k.size(1) % (kv_heads * maps) == 0 &&
              vt.size(0) % kv_heads == 0 &&
              vt.size(1) == k.size(0) && k.size(0) % 64 == 0,
              "q/k/v mismatch");
  a.heads = int(heads);
  a.n_kv = int(kv_heads);
  a.maps = int(maps);
  a.dim = int(k.size(1) / (kv_heads * maps));
  a.vdim = int(vt.size(0) / kv_heads);
  a.tokens = int(k.size(0));
  TORCH_CHECK(rlli::expanded_ok(a.dim, a.vdim, a.maps),
              "head sizes out of range");
  a.q_stride = row_stride(q, k, rows, heads * maps * a.dim, "q");
  TORCH_CHECK(a.q_stride % 8 == 0 &&
              reinterpret_cast<uintptr_t>(q.data_ptr()) % 16 == 0,
              "query rows must be 16-byte aligned");
  a.out_stride = row_stride(out, q, rows, heads * a.vdim, "out");
  TORCH_CHECK(a.out_stride % 4 == 0 &&
              reinterpret_cast<uintptr_t>(out.data_ptr()) % 8 == 0,
              "out rows must be 8-byte aligned");
  a.q = q.data_ptr();
  a.k = k.data_ptr();
  a.vt = vt.data_ptr();
  a.out = out.data_ptr();
  a.tiles = i32(tiles, "tiles");
  a.kv_off = i32(kv_off, "kv_off");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4);
  a.n_tiles = int(tiles.size(1));
  a.scale = float(scale);
  return a;
}

void expanded_attn(const Tensor& q, const Tensor& k, const Tensor& vt,
                   const OptTensor& gate, const Tensor& tiles,
                   const Tensor& kv_off, int64_t heads, int64_t kv_heads,
                   double scale, Tensor out, const OptTensor& r1,
                   const OptTensor& r2, double temp_coef,
                   int64_t temp_every) {
  auto a = expanded_args(q, k, vt, tiles, kv_off, heads, kv_heads, 1, scale,
                         out);
  score_args(a, heads, r1, r2, temp_coef, temp_every);
  if (gate) {
    a.gate_stride = row_stride(*gate, q, q.size(0), heads * a.vdim, "gate");
    TORCH_CHECK(a.gate_stride % 4 == 0 &&
                reinterpret_cast<uintptr_t>(gate->data_ptr()) % 8 == 0,
                "gate rows must be 8-byte aligned");
    a.gate = gate->data_ptr();
  }
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  rlli::launch_expanded_attn(a, stream_of(q));
  check_launch("expanded_attn");
}

// gate: [rows, heads]
void diff_expanded(const Tensor& q, const Tensor& k, const Tensor& vt,
                   const OptTensor& gate, const Tensor& tiles,
                   const Tensor& kv_off, int64_t heads, int64_t kv_heads,
                   double scale, Tensor out, int64_t chunk, double cap,
                   double lambda, double out_scale, double eps) {
  auto a = expanded_args(q, k, vt, tiles, kv_off, heads, kv_heads, 2, scale,
                         out);
  diff_score(a, chunk, cap, lambda, out_scale, eps);
  if (gate) {
    a.gate_stride = row_stride(*gate, q, q.size(0), heads, "gate");
    a.gate = gate->data_ptr();
  }
  c10::hip::HIPGuardMasqueradingAsCUDA guard(q.device());
  rlli::launch_expanded_attn(a, stream_of(q));
  check_launch("diff_expanded");
}

}  // namespace

TORCH_LIBRARY(rlli_attn, m) {
  m.def("window_append(Tensor(a!) qkv, Tensor(b!) k_cache, "
        "Tensor(c!) v_cache, Tensor positions, Tensor? cos_sin, "
        "Tensor slots, int n_q, bool has_kv, float? v_eps) -> ()");
  m.def("window_rows(Tensor qkv, Tensor k_cache, Tensor v_cache, "
        "Tensor block_tables, Tensor tiles, int tile_rows, Tensor? sink, "
        "float scale, int n_q, int window, int keep_first, bool has_kv, "
        "Tensor? r1, Tensor? r2, float temp_coef, int temp_every) -> Tensor");
  m.def("window_fast(Tensor k_cache, Tensor v_cache, bool f32) -> bool");
  m.def("window_decode(Tensor(a!) qkv, Tensor(b!) k_cache, "
        "Tensor(c!) v_cache, Tensor positions, Tensor? cos_sin, "
        "Tensor slots, Tensor block_tables, Tensor? sink, float scale, "
        "int n_q, int window, int keep_first, bool has_kv, Tensor? r1, "
        "Tensor? r2, float temp_coef, int temp_every, float? v_eps) "
        "-> Tensor");
  m.def("kv_gather(Tensor k_cache, Tensor v_cache, Tensor block_tables, "
        "Tensor blocks, int tokens) -> (Tensor, Tensor)");
  m.def("expanded_ok(int dim, int vdim, int maps=1) -> bool", &expanded_ok);
  m.def("diff_append(Tensor(a!) qkv, Tensor(b!) k_cache, "
        "Tensor(c!) v_cache, Tensor positions, Tensor? cos_sin, "
        "Tensor slots, int n_q, Tensor? bias, Tensor q_norm, "
        "Tensor k_norm, float eps) "
        "-> ()");
  m.def("diff_rows(Tensor qkv, Tensor k_cache, Tensor v_cache, "
        "Tensor block_tables, Tensor tiles, int tile_rows, Tensor? gate, "
        "float scale, int n_q, int chunk, float cap, float lam, "
        "float out_scale, float eps) -> Tensor");
  m.def("diff_decode(Tensor(a!) qkv, Tensor(b!) k_cache, Tensor(c!) v_cache, "
        "Tensor positions, Tensor? cos_sin, Tensor slots, "
        "Tensor block_tables, Tensor? gate, float scale, int n_q, "
        "Tensor? bias, Tensor q_norm, Tensor k_norm, int chunk, float cap, float lam, "
        "float out_scale, float eps) -> Tensor");
  m.def("diff_expanded(Tensor q, Tensor k, Tensor vt, Tensor? gate, "
        "Tensor tiles, Tensor kv_off, int heads, int kv_heads, float scale, "
        "Tensor(a!) out, int chunk, float cap, float lam, float out_scale, "
        "float eps) -> ()");
  m.def("expanded_attn(Tensor q, Tensor k, Tensor vt, Tensor? gate, "
        "Tensor tiles, Tensor kv_off, int heads, int kv_heads, float scale, "
        "Tensor(a!) out, Tensor? r1, Tensor? r2, float temp_coef, "
        "int temp_every) -> ()");
}

TORCH_LIBRARY_IMPL(rlli_attn, CUDA, m) {
  m.impl("window_append", &window_append);
  m.impl("window_rows", &window_rows);
  m.impl("window_fast", &window_fast);
  m.impl("window_decode", &window_decode);
  m.impl("kv_gather", &kv_gather);
  m.impl("expanded_attn", &expanded_attn);
  m.impl("diff_append", &diff_append);
  m.impl("diff_rows", &diff_rows);
  m.impl("diff_decode", &diff_decode);
  m.impl("diff_expanded", &diff_expanded);
}
