// Launch declarations of the parallel-block kernels (block.hip) and of
// latent attention (latent.hip, latent_prefill.hip), bound by ext_lat.cpp.
#pragma once

#include "mix.h"

namespace rlli {

// ---- block.hip ---------------------------------------------------------
struct BlockArgs {
  const void* table;       // embedding table (embed launch) or null
  const int32_t* ids;      // token ids (embed launch)
  const void* pos_table;   // learned positions (embed launch) or null
  const int32_t* positions;     // [rows]
  float* x;                // [rows, width] residual
  const void* y;           // [rows, width] what the last block adds
  const float* gain;       // [width] gain of the next norm
  const int64_t* rows;     // row subset (final norm) or null
  void* h;                 // [n, width] normed
  void* hc;                // [n, width] normed + convolved, or null
  const float* taps;       // [n_taps, width], the last meets the own row
  void* tail;              // [slots, n_taps - 1, width] earlier inputs
  const int32_t* slots;    // [n_decode]
  int n, width, groups, n_taps, n_decode;
  int n_positions;         // rows of pos_table
  float eps;
  bool keep;               // write the residual back
  bool f32;
};
// rows [0, n_decode) also get their convolution, from the tail
void launch_block_step(const BlockArgs& a, hipStream_t stream);

struct ConvArgs {
  const void* h;           // [rows, width]
  void* out;               // [rows, width]: h + conv(h)
  const float* taps;       // [n_taps, width]
  void* tail;              // [slots, n_taps - 1, width]
  const int32_t* spans;    // [5, n_spans]: row, position, rows, offset in
                           // its portion, slot
  const int32_t* portions; // [5, n_portions], the same for whole portions
  int n_spans, n_portions, width, n_taps;
  bool f32;
};
void launch_conv_prompt(const ConvArgs& a, hipStream_t stream);

enum ActKind { kActRelu = 0, kActSilu = 1 };
void launch_gate_act(const void* gate_up, void* out, int rows, int ff,
                     int64_t out_stride, int act, bool f32,
                     hipStream_t stream);

// ---- latent.hip --------------------------------------------------------
struct LatentPrepArgs {
  const void* proj;        // [rows, stride]: query latent | kv latent | ...
  const float* q_norm;     // [q_rank]
  const float* kv_norm;    // [kv_rank]
  void* cq;                // [rows, q_rank]
  void* cache;             // [blocks, 1, block, kv_rank]
  const int32_t* slots;    // [rows]
  int rows, stride, q_rank, kv_rank;
  float eps;
  bool f32;
  int cache_kind;
};
void launch_latent_prep(const LatentPrepArgs& a, hipStream_t stream);

// y[t, h, :] = w[h] x[t, h, :], optionally times sigmoid(gate)
struct HeadLinearArgs {
  const void* x;           // [rows, heads * k], rows x_stride apart
  const void* w;           // [heads, n, k]
  const void* gate;        // [rows, heads * n], rows gate_stride apart
  void* y;                 // [rows, heads * n], rows y_stride apart
  int64_t x_stride, gate_stride, y_stride;
  int rows, heads, n, k;
  bool f32;
};
void launch_head_linear(const HeadLinearArgs& a, hipStream_t stream);

// attention of absorbed queries over the cached latents
struct LatentAttnArgs {
  const void* q;           // [rows * heads, rank]
  const void* cache;       // [blocks, 1, block, rank]
  const int32_t* block_tables;
  const int32_t* positions;     // [rows] (decode: one row per sequence)
  const int32_t* tiles;    // [4, n_tiles] (prompt): first query vector,
                           // offset in its portion, vectors, sequence
  const int32_t* pos0;     // [sequences] first position of the portion
  void* out;               // [rows * heads, rank]
  float* part_acc;         // [rows * heads, n_split, rank]
  float* part_ml;          // [rows * heads, n_split, 2]
  int rows, n_tiles, heads, rank, max_blocks, n_split;
  int block_shift;         // log2 of the page size
  float scale;
  int cache_kind;
};
bool latent_fast_ok(int rank, int block_size, bool f32);
// query vectors of one workgroup; a prompt's tile has kLatentVectors
constexpr int kLatentVectors = 32;
int latent_tile(int heads, bool decode);
void launch_latent_attn(const LatentAttnArgs& a, hipStream_t stream);
void launch_latent_rows(const WindowAttnArgs& a, bool decode,
                        hipStream_t stream);

// ---- latent_prefill.hip ------------------------------------------------
struct ExpandedAttnArgs {
  const void* q;           // [rows, heads * dim]
  const void* k;           // [tokens, heads * dim]
  const void* vt;          // [heads * vdim, tokens]
  const void* gate;        // [rows, heads * vdim] or null
  void* out;               // [rows, heads * vdim], rows out_stride apart
  const int32_t* tiles;    // [4, n_tiles]: row, position, rows, sequence
  const int32_t* kv_off;   // [sequences] first token in k / vt, mult. of 64
  int64_t gate_stride, out_stride;
  int n_tiles, heads, dim, vdim, tokens;
  float scale;
};
constexpr int kExpandedRows = 128;
bool expanded_ok(int dim, int vdim);
void launch_expanded_attn(const ExpandedAttnArgs& a, hipStream_t stream);

struct GatherArgs {
  const void* cache;       // [blocks, 1, block, rank]
  void* out;               // [tokens, rank]
  const int32_t* block_tables;
  const int32_t* blocks;   // [4, n]: sequence, token, tokens, output row
  int n, rank, block_size, max_blocks;
  int cache_kind;
};
constexpr int kGatherRows = 64;
void launch_latent_gather(const GatherArgs& a, hipStream_t stream);

}  // namespace rlli
