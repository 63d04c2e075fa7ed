// Launch declarations of the linear recurrences (gla.hip, delta.hip,
// mlstm.hip, rec_scan.hip), bound by ext_rec.cpp.
//
// All of them carry a [dim, vdim] f32 matrix per head.  Decode is one kernel
// per layer.  Prompts run in chunks of kRecChunk rows: a kernel per (chunk,
// head) prepares the chunk's operands, the scan of rec_scan.hip walks the
// chunks of a sequence, and a last one norms and gates.
#pragma once

#include "act.h"

namespace rlli {

constexpr int kRecChunk = 64;

// ---- rec_scan.hip ------------------------------------------------------
//   kScanPlain  O = Qd S + A V,  S = diag(dec) S + Kd^T V
//               decay per key channel, already in Qd, Kd and A
//   kScanMax    one decay per head and everything relative to a running
//               maximum m; a column of ones behind the values carries the
//               normalizer
//   kScanDelta  one decay per head, V replaced by U = Ub - W S
// The last two read queries and keys as they are; row factors carry norms
// and decays.
enum ScanMode { kScanPlain = 0, kScanMax = 1, kScanDelta = 2 };
struct ScanArgs {
  const void* v;           // value rows (plain, max), head h at h * vdim
  const void* q;           // query rows (max, delta), head h / group
  const float* qd;         // [n_tiles, heads, 64, dpad] (plain)
  const void* kt;          // [n_tiles, heads / group, dpad, 64] keys down
                           // the columns: f32 decayed (plain), or as they are
  const float* sc;         // [n_tiles, heads, 64, 64] A
  const float* dec;        // [n_tiles, heads, dpad] (plain), [n_tiles, heads]
  const float* rows;       // [n_tiles, heads, 3, 64]: running log-decay F,
                           // a = i - F, running maximum of a (max); query
                           // factor, key factor, unused (delta)
  const float* w;          // [n_tiles, heads, 64, dpad] (delta)
  const float* ub;         // [n_tiles, heads, 64, ubp] (delta)
  float* state;            // [slots, heads, dim, vpad]
  const float* m;          // [slots, heads] (max)
  float* m_new;            // [n_seqs, heads] (max)
  float* o;                // [rows + 64, heads, opad], spare rows behind
  float* mrow;             // [rows + 64, heads] (max)
  const int32_t* tiles;    // [4, n_tiles] chunks of kRecChunk rows
  const int32_t* seqs;     // [4, n_seqs]: first tile, tiles, pos0, slot
  int64_t v_stride, q_stride;
  int n_rows, n_tiles, n_seqs, heads, group, dim, dpad, vdim, vpad, opad, ubp;
  int cols;                // value columns of state and o
  float qscale;            // (max)
  int mode;
  bool f32;
};
void launch_rec_scan(const ScanArgs& a, hipStream_t stream);

// o over its root mean square, times norm and gate
enum GateKind { kGateNone = 0, kGateSilu = 1, kGateSigmoid = 2 };
struct RecGateArgs {
  const float* o;          // [rows, heads, opad]
  const float* mrow;       // [rows, heads]: o is first divided by
                           // max(|o[vdim]|, e^-mrow) + 1e-6, or null
  const void* gate;        // gate rows, head h at h * vdim
  const float* norm;       // [vdim] or, norm_stride = vdim, [heads, vdim]
  void* out;               // [rows, heads * vdim], rows out_stride apart
  const float* m_new;      // running maxima that return to their slots
  float* m;
  const int32_t* seqs;
  int64_t gate_stride, out_stride;
  int rows, heads, vdim, opad, norm_stride, n_seqs;
  int kind;
  float eps;
  bool f32;
};
void launch_rec_gate(const RecGateArgs& a, hipStream_t stream);

// ---- gla.hip -----------------------------------------------------------
enum GlaKind { kGla = 0, kHgrn2 = 1, kRwkv = 2 };
struct GlaArgs {
  const void* proj;        // query rows, stride apart; keys (HGRN2: forget
                           // logits), values and gates at their offsets
  const void* a1;          // low-rank half of the decay, a1_stride apart
  const void* a2;          // [heads * dim, rank]
  const float* a2_bias;    // [heads * dim]
  const float* lower;      // [heads * dim] (HGRN2)
  const float* bonus;      // [heads * dim] (RWKV)
  const float* norm;       // [vdim] or, norm_stride = vdim, [heads, vdim]
  float* state;            // [slots, heads, dim, vpad]
  const int32_t* slots;    // [sequences]
  const int32_t* positions;     // [rows] (decode)
  const int32_t* tiles;    // [4, n_tiles] chunks of kRecChunk rows
  const int32_t* seqs;     // [4, n_seqs]: first tile, tiles, pos0, slot
  float* qd;               // [n_tiles, heads, 64, dpad] scratch
  float* kd;               // [n_tiles, heads, dpad, 64]
  float* sc;               // [n_tiles, heads, 64, 64]
  float* dec;              // [n_tiles, heads, dpad]
  float* o;                // [rows + 64, heads * vdim]
  void* out;               // [rows, heads * vdim], rows out_stride apart
  int64_t off_k, off_v, off_g;  // from proj
  int64_t stride, a1_stride;
  int rows, n_tiles, n_seqs, heads, dim, vdim, vpad, dpad, rank;
  int out_stride, n_slots, norm_stride;
  float tau, eps;
  int kind;                // GlaKind
  bool f32;
};
void launch_gla_decode(const GlaArgs& a, hipStream_t stream);
void launch_gla_prefill(const GlaArgs& a, hipStream_t stream);

// ---- delta.hip ---------------------------------------------------------
struct DeltaArgs {
  const void* proj;        // [rows, stride]: q | k | v | gate | beta | decay
  const void* x;           // [rows, channels] convolved q | k | v (prompt)
  const float* taps;       // [n_taps, channels] (decode)
  void* tail;              // [slots, ring, channels] (decode)
  const float* a_rate;     // [heads] exp(A_log)
  const float* dt_bias;    // [heads]
  const float* norm;       // [vdim]
  float* state;            // [slots, heads, dim, vpad]
  const int32_t* slots;
  const int32_t* positions;
  const int32_t* tiles;
  const int32_t* seqs;
  void* kt;                // scratch, see ScanArgs
  float* sc;
  float* dec;
  float* row_f;
  float* w;
  float* ub;
  float* o;
  void* out;               // [rows, heads * vdim], rows out_stride apart
  int64_t stride, x_stride, out_stride;
  int off_g, off_b, off_a, channels, n_taps, ring;
  int rows, n_tiles, n_seqs, heads, kv_heads, dim, vdim, vpad, dpad, ubp;
  float eps;
  bool f32;
};
void launch_delta_decode(const DeltaArgs& a, hipStream_t stream);
void launch_delta_prefill(const DeltaArgs& a, hipStream_t stream);

// ---- mlstm.hip ---------------------------------------------------------
struct MlstmArgs {
  const void* proj;        // [rows, stride]: q | k | v | gate | i | f
  const float* i_bias;     // [heads]
  const float* f_bias;     // [heads]
  const float* norm;       // [heads * vdim]
  float* state;            // [slots, heads, dim, vpad], vdim + 1 columns
  float* m;                // [slots, heads] running maximum
  const int32_t* slots;
  const int32_t* positions;
  const int32_t* tiles;
  const int32_t* seqs;
  void* kt;                // scratch, see ScanArgs
  float* sc;
  float* row_f;
  float* o;                // [rows + 64, heads, opad]
  float* mrow;
  float* m_new;
  void* out;               // [rows, heads * vdim], rows out_stride apart
  int64_t stride, out_stride;
  int off_k, off_v, off_g, off_i, off_f;
  int rows, n_tiles, n_seqs, heads, dim, vdim, vpad, dpad, opad;
  float cap, eps;
  bool f32;
};
void launch_mlstm_decode(const MlstmArgs& a, hipStream_t stream);
void launch_mlstm_prefill(const MlstmArgs& a, hipStream_t stream);

}  // namespace rlli
