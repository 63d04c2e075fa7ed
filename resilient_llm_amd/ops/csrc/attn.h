// Launch declarations of paged softmax attention (window_attn.hip,
// window_prefill.hip, expanded_attn.hip).
#pragma once

#include "act.h"

namespace rlli {

// ---- window_attn.hip / window_prefill.hip ----------------------------
// what a query at position p is multiplied by
DEV_INLINE float query_temp(int p, float coef, int every) {
  return every > 0 ? 1.f + coef * logf(float((p + 1) / every + 1)) : 1.f;
}

struct WindowAttnArgs {
  const void* qkv;         // [rows, stride]: q heads | k heads | v heads
  void* qkv_rw;            // the same, writable (rotation in place)
  void* k_cache;           // [blocks, n_kv, block, dim]
  void* v_cache;           // [blocks, n_kv, block, vdim]
  const int32_t* positions;
  const float* cos_sin;    // [max_pos, rot] = cos(rot/2) | sin(rot/2)
  const int32_t* slots;
  const int32_t* block_tables;
  const int32_t* tiles;    // [4, n_tiles]: row0, pos0, rows, seq
  const float* sink;       // [n_q] or null
  void* out;               // [rows, n_q * vdim]
  float* part_acc;         // split scratch (decode)
  float* part_ml;
  int rows, n_tiles, tile_rows, n_q, n_kv, dim, vdim, rot, stride;
  int block_size, max_blocks, window, keep_first, n_split;
  float scale;
  const float* r1;         // [n_q] a score loses r1 ln(1 + r2 distance), or
  const float* r2;         // null
  float temp_coef;         // query temperature by position, see query_temp
  int temp_every;          // (0: none)
  float v_eps;
  bool v_norm;             // values are cached over their root mean square
  bool has_kv;             // this layer projects and appends k/v
  bool f32;
  int cache;               // CacheKind
};
void launch_window_rope_append(const WindowAttnArgs& a, hipStream_t stream);
void launch_window_decode(const WindowAttnArgs& a, hipStream_t stream);
void launch_window_rows(const WindowAttnArgs& a, bool decode,
                        hipStream_t stream);
void launch_window_prefill(const WindowAttnArgs& a, hipStream_t stream);
bool window_fast_ok(const WindowAttnArgs& a);
int window_decode_heads_per_wg(int group);
int window_prefill_sub_tiles(int group);

// ---- expanded_attn.hip -------------------------------------------------
struct ExpandedAttnArgs {
  const void* q;           // [rows, heads * dim], rows q_stride apart
  const void* k;           // [tokens, n_kv * dim]
  const void* vt;          // [n_kv * vdim, tokens]
  const void* gate;        // [rows, heads * vdim] or null
  void* out;               // [rows, heads * vdim], rows out_stride apart
  const int32_t* tiles;    // [4, n_tiles]: row, position, rows, sequence
  const int32_t* kv_off;   // [sequences] first token in k / vt, mult. of 64
  int64_t q_stride, gate_stride, out_stride;
  int n_tiles, heads, n_kv, dim, vdim, tokens;
  float scale;
  const float* r1;         // distance bias and query temperature as above
  const float* r2;
  float temp_coef;
  int temp_every;
};
constexpr int kExpandedRows = 128;
bool expanded_ok(int dim, int vdim);
void launch_expanded_attn(const ExpandedAttnArgs& a, hipStream_t stream);

// sequences' keys and values out of their pages, values transposed
struct KvGatherArgs {
  const void* k_cache;     // [blocks, n_kv, block, dim]
  const void* v_cache;     // [blocks, n_kv, block, vdim]
  void* k;                 // [tokens, n_kv * dim]
  void* vt;                // [n_kv * vdim, tokens]
  const int32_t* block_tables;
  const int32_t* blocks;   // [4, n]: sequence, token, tokens, output row
  int n, n_kv, dim, vdim, block_size, max_blocks, tokens;
  int cache_kind;
};
constexpr int kKvGatherRows = 64;
void launch_kv_gather(const KvGatherArgs& a, hipStream_t stream);

}  // namespace rlli
