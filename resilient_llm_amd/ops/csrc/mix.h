// Shared pieces of the mixed-layer model kernels (hyper-connections,
// windowed attention, gated linear attention, mixture of experts) and
// the launch declarations that ext_mix.cpp binds.
//
// Every kernel takes its activation type as a template parameter:
// uint16_t (bf16 bits, the serving precision) or float (true 32-bit).
#pragma once

#include "common.h"

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef short s16x8_t __attribute__((ext_vector_type(8)));

DEV_INLINE float act_load(const uint16_t* p) { return bf16_to_f32(*p); }
DEV_INLINE float act_load(const float* p) { return *p; }
DEV_INLINE void act_store(uint16_t* p, float v) { *p = f32_to_bf16(v); }
DEV_INLINE void act_store(float* p, float v) { *p = v; }

// four neighbours at once; the caller guarantees 4-element alignment
DEV_INLINE f32x4_t act_load4(const uint16_t* p) {
  const uint2 r = *reinterpret_cast<const uint2*>(p);
  return f32x4_t{__uint_as_float(r.x << 16),
                 __uint_as_float(r.x & 0xffff0000u),
                 __uint_as_float(r.y << 16),
                 __uint_as_float(r.y & 0xffff0000u)};
}
DEV_INLINE f32x4_t act_load4(const float* p) {
  return *reinterpret_cast<const f32x4_t*>(p);
}
DEV_INLINE void act_store4(uint16_t* p, f32x4_t v) {
  uint2 r;
  r.x = uint32_t(f32_to_bf16(v[0])) | (uint32_t(f32_to_bf16(v[1])) << 16);
  r.y = uint32_t(f32_to_bf16(v[2])) | (uint32_t(f32_to_bf16(v[3])) << 16);
  *reinterpret_cast<uint2*>(p) = r;
}
DEV_INLINE void act_store4(float* p, f32x4_t v) {
  *reinterpret_cast<f32x4_t*>(p) = v;
}

// Cache codec of the 32-bit mode, same interface as CacheBF16/CacheFP8.
struct CacheF32 {
  using elem = float;
  struct vec8 { float f[8]; };
  static DEV_INLINE void to_f32(const vec8& raw, float* out8) {
#pragma unroll
    for (int i = 0; i < 8; ++i) out8[i] = raw.f[i];
  }
};

DEV_INLINE float cache_load(const uint16_t* p) { return bf16_to_f32(*p); }
DEV_INLINE float cache_load(const float* p) { return *p; }
DEV_INLINE float cache_load(const uint8_t* p) {
  return __builtin_amdgcn_cvt_f32_fp8(int(*p), 0);
}
DEV_INLINE void cache_store(uint16_t* p, float v) { *p = f32_to_bf16(v); }
DEV_INLINE void cache_store(float* p, float v) { *p = v; }
DEV_INLINE void cache_store(uint8_t* p, float v) {
  *p = uint8_t(__builtin_amdgcn_cvt_pk_fp8_f32(v, v, 0, false) & 0xff);
}

// Eight consecutive k-values of one matrix row per lane, and the MFMA
// that contracts them: lane l holds row l & 15 and k = (l >> 4) * 8 + j.
// The 32-bit form walks the same eight values with eight 16x16x4 steps,
// pairing slot l >> 4 of step j with k = (l >> 4) * 8 + j on both sides.
template <typename T> struct Frag8;
template <> struct Frag8<uint16_t> {
  s16x8_t v;
  DEV_INLINE void zero() { v = s16x8_t{0, 0, 0, 0, 0, 0, 0, 0}; }
  DEV_INLINE void load(const uint16_t* p) {
    v = *reinterpret_cast<const s16x8_t*>(p);
  }
  static DEV_INLINE f32x4_t mma(const Frag8& a, const Frag8& b, f32x4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
  }
};
template <> struct Frag8<float> {
  f32x4_t lo, hi;
  DEV_INLINE void zero() {
    lo = f32x4_t{0.f, 0.f, 0.f, 0.f};
    hi = lo;
  }
  DEV_INLINE void load(const float* p) {
    lo = *reinterpret_cast<const f32x4_t*>(p);
    hi = *reinterpret_cast<const f32x4_t*>(p + 4);
  }
  static DEV_INLINE f32x4_t mma(const Frag8& a, const Frag8& b, f32x4_t c) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.lo[j], b.lo[j], c, 0, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.hi[j], b.hi[j], c, 0, 0, 0);
    return c;
  }
};

namespace rlli {

// element type of a paged cache
enum CacheKind { kCacheBF16 = 0, kCacheFP8 = 1, kCacheF32 = 2 };

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

// ---- window_attn.hip / window_prefill.hip ----------------------------
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

// ---- gla.hip -----------------------------------------------------------
struct GlaArgs {
  const void* proj;        // [rows, stride]: q | k | v | gate | low-rank
                           // (HGRN2: q | forget logit | v)
  const void* a2;          // [heads * dim, rank]
  const float* a2_bias;    // [heads * dim]
  const float* lower;      // [heads * dim] (HGRN2)
  const float* norm;       // [vdim]
  float* state;            // [slots, heads, dim, vpad]
  const int32_t* slots;    // [sequences]
  const int32_t* positions;     // [rows] (decode)
  const int32_t* tiles;    // [4, n_tiles] chunks of kGlaChunk rows
  const int32_t* seqs;     // [4, n_seqs]: first tile, tiles, pos0, slot
  float* qd;               // [n_tiles, heads, 64, dpad] scratch
  float* kd;               // [n_tiles, heads, dpad, 64]
  float* sc;               // [n_tiles, heads, 64, 64]
  float* dec;              // [n_tiles, heads, dpad]
  float* o;                // [rows, heads * vdim]
  void* out;               // [rows, heads * vdim], rows out_stride apart
  int rows, n_tiles, n_seqs, heads, dim, vdim, vpad, dpad, rank, stride;
  int off_k, off_v, off_g, off_a;   // columns of proj
  int out_stride, n_slots;
  float tau, eps;
  bool forget;             // HGRN2 instead of GLA
  bool f32;
};
constexpr int kGlaChunk = 64;
void launch_gla_decode(const GlaArgs& a, hipStream_t stream);
void launch_gla_prefill(const GlaArgs& a, hipStream_t stream);

// ---- moe.hip -----------------------------------------------------------
struct MoeArgs {
  const void* h;           // [rows, width]
  const void* router;      // [experts, width]
  const void* w_up;        // [experts, ffp/16, 2, 16, width] gate | up
  const void* w_down;      // [experts, width, ffp]
  int32_t* ids;            // [rows, top]
  float* weights;          // [rows, top]
  int32_t* perm;           // [rows * top] pairs in expert order
  int32_t* tile_expert;    // [max_tiles]
  int32_t* tile_row0;      // [max_tiles]
  int32_t* tile_rows;      // [max_tiles]
  int32_t* counters;       // [2 * experts + 1]
  void* act;               // [rows * top, ffp]
  void* y;                 // [rows, top, width]
  int rows, width, experts, top, ffp, tile_m, max_tiles;
  float limit;
  bool f32;
};
void launch_moe_route(const MoeArgs& a, hipStream_t stream);
void launch_moe_plan(const MoeArgs& a, hipStream_t stream);
void launch_moe_experts(const MoeArgs& a, hipStream_t stream);

}  // namespace rlli
