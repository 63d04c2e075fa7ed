// Launch declarations of the residual-block kernels (block.hip), bound by
// ext_blk.cpp.
#pragma once

#include "act.h"

namespace rlli {

// ---- block.hip ---------------------------------------------------------
struct BlockArgs {
  const void* table;       // embedding table (embed launch) or null
  const int32_t* ids;      // token ids (embed launch)
  const void* pos_table;   // learned positions (embed launch) or null
  const int32_t* positions;     // [rows]
  float* x;                // [rows, width] residual
  const void* y;           // [rows, width] what the last block adds, or
                           // with part_ids [rows, parts, width]: their sum
  const int32_t* part_ids; // [rows, parts] or null; from part_limit on, a
                           // part is part_w part_h instead
  const float* part_w;     // [rows, parts]
  const void* part_h;      // [rows, width]
  int parts, part_limit;
  const float* y_bias;     // [width] added to y, or null
  const void* y2;          // its second half (merge), or null
  const float* gain1;      // [width] gains of y's and y2's own norms (merge)
  const float* gain2;
  const float* gain;       // [width] gain of the next norm
  const int64_t* rows;     // row subset (final norm) or null
  void* h;                 // [n, width] normed
  void* hc;                // [branches, n, width] normed + convolved, or null
  const float* taps;       // [branches, n_taps, width], the last meets the
                           // own row
  void* tail;              // [slots, ring, width] earlier inputs
  const int32_t* slots;    // [n_decode]
  int n, width, groups, n_taps, ring, branches, n_decode;
  int n_positions;         // rows of pos_table
  float embed_scale;
  float eps;
  bool keep;               // write the residual back
  bool f32;
};
// rows [0, n_decode) also get their convolution, from the tail
void launch_block_step(const BlockArgs& a, hipStream_t stream);

struct ConvArgs {
  const void* h;           // [rows, width], rows h_stride apart
  void* out;               // [branches, rows, width]: h + conv(h), or
                           // silu(conv(h))
  const float* taps;       // [branches, n_taps, width]
  void* tail;              // [slots, ring, width]
  const int32_t* spans;    // [5, n_spans]: row, position, rows, offset in
                           // its portion, slot
  const int32_t* portions; // [5, n_portions], the same for whole portions
  int64_t h_stride, out_stride, branch_stride;
  int n_spans, n_portions, width, n_taps, ring, branches;
  bool silu;
  bool f32;
};
void launch_conv_prompt(const ConvArgs& a, hipStream_t stream);

// out = act(gate) * up; kActClampGlu: g sigmoid(1.702 g) (u + 1) with
// g <= limit, |u| <= limit
enum ActKind { kActRelu = 0, kActSilu = 1, kActClampGlu = 2 };
void launch_gate_act(const void* gate_up, void* out, int rows, int ff,
                     int64_t out_stride, int act, float limit, bool f32,
                     hipStream_t stream);

// out = cap * tanh(x / cap), 32-bit
void launch_soft_cap(const void* x, float* out, int64_t n, float cap,
                     bool f32, hipStream_t stream);

}  // namespace rlli
