// Checks shared by the bindings of windowed attention (ext_attn.cpp,
// ext_mix.cpp).
#pragma once

#include "attn.h"
#include "ext_common.h"

namespace rlli_ext {

// cache and head sizes, mask and scale; the caller adds rows and tables
inline rlli::WindowAttnArgs window_args(
    const Tensor& qkv, const Tensor& k_cache, const Tensor& v_cache,
    int64_t n_q, bool has_kv, double scale = 1.0, int64_t window = 1,
    int64_t keep_first = 0, const OptTensor& sink = {}, int maps = 1) {
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
  a.maps = maps;
  TORCH_CHECK(k_cache.size(3) % maps == 0, "a key per map");
  a.dim = int(k_cache.size(3)) / maps;
  a.vdim = int(v_cache.size(3));
  TORCH_CHECK(qkv.dim() == 2);
  a.rows = int(qkv.size(0));
  a.stride = int(qkv.size(1));
  a.has_kv = has_kv;
  TORCH_CHECK(a.n_q % a.n_kv == 0, "heads must be a multiple of kv heads");
  TORCH_CHECK(a.vdim <= 512 && a.dim <= 4096, "head sizes out of range");
  const int need = a.n_q * maps * a.dim +
                   (has_kv ? a.n_kv * (maps * a.dim + a.vdim) : 0);
  // with two maps further columns (a gate) may follow
  TORCH_CHECK(maps == 1 ? a.stride == need : a.stride >= need,
              "qkv width mismatch");
  TORCH_CHECK(window >= 1 && keep_first >= 0);
  a.window = int(std::min<int64_t>(window, 1 << 30));
  a.keep_first = int(std::min<int64_t>(keep_first, 1 << 30));
  a.scale = float(scale);
  a.qkv = qkv.data_ptr();
  a.qkv_rw = qkv.data_ptr();
  a.k_cache = k_cache.data_ptr();
  a.v_cache = v_cache.data_ptr();
  a.sink = sink ? f32_vec(*sink, a.n_q, "sink") : nullptr;
  return a;
}

inline void window_tables(rlli::WindowAttnArgs& a,
                          const Tensor& block_tables) {
  a.block_tables = i32(block_tables, "block_tables");
  TORCH_CHECK(block_tables.dim() == 2);
  a.max_blocks = int(block_tables.size(1));
}

inline void window_tiles(rlli::WindowAttnArgs& a, const Tensor& tiles,
                         int64_t tile_rows) {
  a.tiles = i32(tiles, "tiles");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(0) == 4);
  a.n_tiles = int(tiles.size(1));
  a.tile_rows = int(tile_rows);
}

}  // namespace rlli_ext
