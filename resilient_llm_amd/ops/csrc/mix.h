// Launch declarations of the residual-stream, windowed prompt attention and
// expert kernels, bound by ext_mix.cpp.
#pragma once

#include "act.h"
#include "attn.h"

namespace rlli {

// ---- hyper.hip -------------------------------------------------------
struct HyperArgs {
  const void* table;       // embedding table (embed launch) or null
  const int32_t* ids;      // token ids (embed launch)
  const float* w_embed;    // embedding norm gain (embed launch)
  float* x;                // [rows, streams, width] residual streams
  const void* y;           // [rows, parts, width] sublayer output
  const float* mix;        // [streams, streams] (from, to)
  const float* out_w;      // [streams]
  const float* in_w;       // [streams] of the next sublayer
  const float* gain;       // [width] gain of the next norm
  const int64_t* rows;     // row subset (final norm) or null
  void* h;                 // [n, width] normed input of the next sublayer
  int n, streams, width, parts;
  float eps;
  bool keep;               // write the streams back
  bool f32;
};
void launch_hyper_embed(const HyperArgs& a, hipStream_t stream);
void launch_hyper_step(const HyperArgs& a, hipStream_t stream);
void launch_relu2(const void* x, void* out, int64_t n, bool f32,
                  hipStream_t stream);

// ---- moe.hip -----------------------------------------------------------
struct MoeArgs {
  const void* h;           // [rows, width]
  const void* router;      // [routes, width]
  const float* correction; // [routes] added for the choice only, or null
  const void* w_up;        // [experts, ffp/16, 2, 16, width] gate | up, or
                           // [experts, ffp, width] without a gate
  const void* w_down;      // [experts, width, ffp]
  int32_t* ids;            // [rows, top]; from ``experts`` on: identity
  float* weights;          // [rows, top]
  int32_t* perm;           // [rows * top] experts' pairs in expert order
  int32_t* tile_expert;    // [max_tiles]
  int32_t* tile_row0;      // [max_tiles]
  int32_t* tile_rows;      // [max_tiles]
  int32_t* counters;       // [2 * experts + 1]
  void* act;               // [rows * top, ffp]
  void* y;                 // [rows, top, width]
  int rows, width, experts, top, ffp, tile_m, max_tiles;
  int routes;              // experts and identity experts
  int groups, keep;        // only the best ``keep`` groups of neighbouring
                           // routes can be chosen
  bool softmax;            // scores: softmax, chosen ones scaled to sum 1
                           // (else sigmoid as they are)
  bool gated;              // gated experts, weight on the input; else relu
                           // squared, weight on the output
  float limit;
  bool f32;
};
void launch_moe_route(const MoeArgs& a, hipStream_t stream);
void launch_moe_plan(const MoeArgs& a, hipStream_t stream);
void launch_moe_experts(const MoeArgs& a, hipStream_t stream);

}  // namespace rlli
