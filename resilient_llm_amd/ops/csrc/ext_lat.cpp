// Torch bindings (torch.ops.rlli_lat.*) of the latent attention kernels.

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

}  // namespace

TORCH_LIBRARY(rlli_lat, m) {
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
}

TORCH_LIBRARY_IMPL(rlli_lat, CUDA, m) {
  m.impl("latent_prep", &latent_prep);
  m.impl("head_linear", &head_linear);
  m.impl("latent_fast", &latent_fast);
  m.impl("latent_attn", &latent_attn);
  m.impl("latent_gather", &latent_gather);
}
