// Launch declarations of paged softmax attention (window_attn.hip,
// window_prefill.hip, diff_attn.hip, expanded_attn.hip).
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
  void* k_cache;           // [blocks, n_kv, block, maps * dim]
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
  int chunk;               // > 0: a query sees its chunk of this many
                           // positions instead of a window
  float cap;               // > 0: a score becomes cap tanh(score / cap)
  // Differential attention: a head has two maps, queries and keys of their
  // own (side by side, dim each) over the same values; its output is
  // map 1 - lambda map 2, over its root mean square, times out_scale and
  // the sigmoid of the head's gate.
  int maps;                // 1 or 2
  const float* bias;       // [q | k | v] added to them, or null (maps = 2)
  const float* q_norm;     // [dim] norms of queries and keys per head and
  const float* k_norm;     // map, ahead of the rotation (maps = 2)
  float eps;               // of those norms and the output's
  float lambda, out_scale;
  const void* gate;        // [rows, n_q], rows gate_stride apart, or null
  int64_t gate_stride;
};
// first position that a query at ``pos`` may see (kept tokens aside)
DEV_INLINE int first_seen(const WindowAttnArgs& a, int pos) {
  return a.chunk > 0 ? pos / a.chunk * a.chunk : max(0, pos - a.window + 1);
}
constexpr float kTwoLog2e = 2.8853900817779268f;
void launch_diff_append(const WindowAttnArgs& a, hipStream_t stream);
void launch_diff_decode(const WindowAttnArgs& a, hipStream_t stream);
void launch_diff_rows(const WindowAttnArgs& a, bool decode,
                      hipStream_t stream);
bool diff_fast_ok(const WindowAttnArgs& a);
int diff_head_blocks(int group);     // workgroups per kv head, sequence, split
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
  const void* q;           // [rows, heads * maps * dim], q_stride apart
  const void* k;           // [tokens, n_kv * maps * dim]
  const void* vt;          // [n_kv * vdim, tokens]
  const void* gate;        // [rows, heads * vdim] ([rows, heads] with two
                           // maps) or null
  void* out;               // [rows, heads * vdim], rows out_stride apart
  const int32_t* tiles;    // [4, n_tiles]: row, position, rows, sequence
  const int32_t* kv_off;   // [sequences] where position 0 is (or would be) in
                           // k / vt, mult. of 64
  int64_t q_stride, gate_stride, out_stride;
  int n_tiles, heads, n_kv, dim, vdim, tokens;
  float scale;
  const float* r1;         // distance bias and query temperature as above
  const float* r2;
  float temp_coef;
  int temp_every;
  int maps;                // 2: differential attention as above
  int chunk;
  float cap, eps, lambda, out_scale;
};
constexpr int kExpandedRows = 128;
bool expanded_ok(int dim, int vdim, int maps = 1);
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
