// Launch declarations of latent attention (latent.hip), bound by
// ext_lat.cpp.
#pragma once

#include "act.h"
#include "attn.h"

namespace rlli {

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
