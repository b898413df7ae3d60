// Host-visible launch interface of the kernels over bfloat16 weights: linears with the epilogues a
// layered decoder needs, attention over chunks or a sliding window, the Mamba-2 recurrence, the gated
// delta rule, and routed experts.  Plain structs and device pointers; launchers are asynchronous on the stream and assume
// validated sizes.  `f32` selects float activations (else bfloat16); weights are bfloat16 in both.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace llmopt {

// The step words in device memory every stateful kernel reads: the position of the first token of the
// step in its sequence, and the sequence's state slot.
constexpr uint32_t kStatePosition = 0, kStateSlot = 1, kStateWords = 2;

enum class DenseEpilogue : uint32_t {
  kStore = 0,     // out[r, c] (activation type)
  kStoreF32 = 1,  // out_f32[r, c]
  kAdd = 2,       // stream[r, c] += result * (row_gate ? sigmoid(row_gate[r * row_gate_stride]) : 1)
  kGated = 3,     // out[r, c] = act(gate) * up
  kQkv = 4,       // kStore, with the value columns mixed with another layer's values
  kSplit = 5,     // columns below `split` to out, the rest to out_f32 as float32
};

// Values of a layer, mixed per token with those of the first mixing layer.
// mode 0: as they are; 1: this is the first such layer, its values are kept in v_first;
// 2: (1 - lambda) v + lambda v_first.
struct ValueMix {
  uint32_t mode;
  float lambda;
  float *v_first;  // f32 [m, n_v]
};

struct DenseLinearArgs {
  bool f32;
  const void *x;         // activations [m, k], row stride ldx
  const uint16_t *w;     // bf16 [n, k]
  const uint16_t *w_up;  // kGated: the second matrix
  uint32_t m, n, k, ldx;
  DenseEpilogue epilogue;
  uint32_t activation;
  float limit;           // kGated, clamped activation
  void *out;
  float *out_f32;        // kStoreF32, kSplit, and the stream of kAdd
  uint32_t ld_out, ld_f32;
  const float *row_gate;
  uint32_t row_gate_stride;
  uint32_t split;        // kSplit; kQkv: first value column
  ValueMix mix;
  // routed rows (null: the plain product): see RoutePlan
  const uint32_t *tile_expert, *tile_first, *tile_rows, *row_source;
  uint32_t tiles, tile;  // most tiles the plan can fill, rows of a tile
};
hipError_t launch_dense_gemm(const DenseLinearArgs &args, hipStream_t stream);

// out[r, :] = x[row, :] / rms * weight with row = rows ? rows[r] : r; `groups` equal parts normalised each
// by its own root mean square.  gate != null: the input is x * silu(gate) (x, gate in the activation type).
struct DenseNormArgs {
  bool f32;
  const float *x;        // f32 [*, width], when x_act is null
  const void *x_act;     // activation type [rows, width]
  const void *gate;      // activation type, row stride ld_gate
  uint32_t ld_gate;
  const uint16_t *weight;  // bf16 [width]
  void *out;             // activation type [rows, width]
  const uint32_t *rows_index;
  uint32_t rows, width, groups;
  float epsilon;
};
hipError_t launch_dense_norm(const DenseNormArgs &args, hipStream_t stream);

// A sublayer's output joins the stream behind its norm:
//   stream_out[r, :] = x[row, :] + scale y[row, :] / rms(y[row, :]) * (offset + add_weight)
// with row = rows_index ? rows_index[r] : r; y == null: stream_out = x.  operand (activation type) is the new
// stream, or with norm_weight its norm, / rms * (offset + norm_weight).
struct NormAddArgs {
  bool f32;
  const float *x, *y;          // f32 [*, width]
  const uint16_t *add_weight;  // bf16 [width]
  const uint16_t *norm_weight; // may be null
  float *stream_out;           // f32 [rows, width], may be null
  void *operand;               // may be null
  const uint32_t *rows_index;
  uint32_t rows, width;
  float epsilon, offset, scale;
};
hipError_t launch_norm_add(const NormAddArgs &args, hipStream_t stream);

// values <- cap tanh(values / cap), in place.  (In the products' epilogue it would cost every large tile registers.)
hipError_t launch_soft_cap(float *values, uint64_t count, float cap, hipStream_t stream);

struct DenseEmbeddingArgs {
  const int64_t *tokens;
  const uint16_t *embed;  // bf16 [vocabulary, width]
  float *stream;          // f32 [m, width]
  uint32_t m, vocabulary, width;
  float scale;
};
hipError_t launch_dense_embedding(const DenseEmbeddingArgs &args, hipStream_t stream);

// ---- one token: matrix-vector products ----------------------------------------------------------

enum class GemvEpilogue : uint32_t {
  kStore = 0, kStoreF32 = 1, kAdd = 2, kGated = 3,
  kQkv = 4,    // q to out; mixed k, v straight to their cache rows
  kSsmIn = 5,  // z as it is, x | B | C through the convolution and silu, dt through softplus: all to out_f32
  kConvIn = 6,  // columns inner .. inner + channels through the convolution and silu, the others as they are
};

struct ChunkCache {
  void *keys, *values;  // [slot][kv_heads][capacity][dim] / [...][vdim], activation type
  uint32_t capacity;    // rows per head; position p lives in row p % capacity
  uint32_t span;        // positions of one chunk or window (capacity >= span); 0: all positions
  bool sliding;         // span: the position itself and the span - 1 before it, else chunks of span
};

struct DenseGemvArgs {
  bool f32;
  // input: norm_weight == null: activation-type row, or f32 (x_is_f32); else the f32 row normalised on the way in
  const void *x;
  bool x_is_f32;
  const uint16_t *norm_weight;
  uint32_t norm_groups;
  float epsilon;
  // a pending sublayer output joins the f32 row first (see NormAddArgs); the new row goes to stream_out
  const float *pending;
  const uint16_t *pending_weight;
  float *stream_out;
  float pending_scale, norm_offset;
  const uint16_t *w, *w_up;
  uint32_t n, k;
  GemvEpilogue epilogue;
  uint32_t activation;
  float limit;
  float softcap;  // kStoreF32: softcap tanh(result / softcap); 0: none
  void *out;
  float *out_f32;
  // kQkv
  const uint32_t *state;
  uint32_t n_q, n_k, dim, vdim, kv_heads;
  ChunkCache cache;
  ValueMix mix;
  // kSsmIn, kConvIn
  const uint16_t *conv, *conv_bias, *dt_bias;
  float *conv_state;  // f32 [slot][taps][channels], position p in row p % taps
  uint32_t inner, channels, taps;
};
bool dense_gemv_ok(const DenseGemvArgs &args);
hipError_t launch_dense_gemv(const DenseGemvArgs &args, hipStream_t stream);

// ---- attention ---------------------------------------------------------------------------------------

// Norm per head (weights over dim, shared by the heads) and rotation of queries and keys, in this order:
// component i < dims / 2 turns with component i + dims / 2 by position * frequencies[i].
struct HeadRotation {
  const uint16_t *q_norm, *k_norm;  // bf16 [dim]
  const double *frequencies;        // [dims / 2]
  uint32_t dims;                    // 0: no rotation
  float epsilon;
};

// q | k | v rows of m new tokens at positions state[0] .. + m - 1; earlier keys that the first token sees
// come from the cache.  score = cap tanh(scale q k / cap); the sink joins the denominator only.
struct ChunkAttentionArgs {
  bool f32;
  const void *qkv;  // [m, ld]: heads * dim, kv_heads * dim, kv_heads * vdim; one token: only q is read
  uint32_t ld, ld_out;
  float out_scale;
  // one token with row: the raw float32 q | k | v; its norm, rotation and cache rows are part of the launch,
  // and the output is float32 in out_row
  const float *row;
  HeadRotation rotation;
  float *out_row;
  ChunkCache cache;
  const uint16_t *sink;  // bf16 [heads], may be null
  const uint32_t *state;
  void *out;  // [m, heads * vdim]
  uint32_t m, heads, kv_heads, dim, vdim;
  float scale, softcap;  // softcap 0: none
  void *workspace;
  size_t workspace_bytes;
};
size_t chunk_attention_workspace_bytes(const ChunkAttentionArgs &args);
bool chunk_attention_ok(const ChunkAttentionArgs &args);
hipError_t launch_chunk_attention(const ChunkAttentionArgs &args, hipStream_t stream);
// k, v of the step's tokens into their cache rows (those that the ring still holds afterwards).
hipError_t launch_chunk_cache_write(const ChunkAttentionArgs &args, hipStream_t stream);
// Norm and rotation of the q and k columns, in place.
hipError_t launch_rotate_heads(const ChunkAttentionArgs &args, hipStream_t stream);

// ---- Mamba-2 ------------------------------------------------------------------------------------------

struct SsmArgs {
  bool f32;
  uint32_t m, heads, vdim, groups, state_size, taps;
  const uint32_t *step;  // state words
  const void *projected;  // [m, inner + channels] z | x B C, activation type
  const float *dt;        // f32 [m, heads], before softplus
  const uint16_t *conv, *conv_bias, *dt_bias, *a_log, *d_skip;
  float *conv_state;      // [slot][taps][channels]
  float *ssm_state;       // [slot][heads][vdim][state_size]
  void *y;                // m > 1: activation type [m, inner], without the gate
  // one token: the row kSsmIn left, and y * silu(z) as f32 [inner]
  const float *row;
  float *gated;
  void *workspace;
  size_t workspace_bytes;
};
constexpr uint32_t kSsmChunk = 64;
size_t ssm_workspace_bytes(const SsmArgs &args);
hipError_t launch_ssm_step(const SsmArgs &args, hipStream_t stream);
hipError_t launch_ssm_prefill(const SsmArgs &args, hipStream_t stream);

// ---- gated delta rule --------------------------------------------------------------------------------------

// Per head, with unit keys and queries (queries also / sqrt(dim)), decay per key channel, state S [dim][vdim]:
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//   out = o / rms(o) * norm * sigmoid(gate) * out_scale
// g = exp(-exp(a_log) softplus(decay + dt_bias)).  q, k (kv_heads) and v pass a convolution and silu first.
struct DeltaArgs {
  bool f32;
  uint32_t m, heads, kv_heads, dim, vdim, taps;
  const uint32_t *step;  // state words
  float epsilon, out_scale;
  const uint16_t *conv, *dt_bias, *a_log, *norm;  // conv [q | k | v channels][taps]
  float *conv_state;     // [slot][taps][channels]
  float *state;          // [slot][heads][dim][vdim]
  // more than one token
  const void *projected;  // activation type, row stride ld: q | k | v before the convolution
  uint32_t ld;
  const float *beta;      // f32 [m, heads], before the sigmoid
  const float *decay;     // f32 [m, heads * dim]
  const void *gate;       // activation type [m, heads * vdim], before the sigmoid
  void *out;              // activation type, row stride ld_out
  uint32_t ld_out;
  void *workspace;
  size_t workspace_bytes;
  // one token: float32 rows; decay = w_decay decay_in, gate = w_gate gate_in inside the launch
  const float *row, *row_beta, *decay_in, *gate_in;  // row: q | k | v behind the convolution and silu
  const uint16_t *w_decay, *w_gate;                  // [heads * dim][decay_rank], [heads * vdim][gate_rank]
  uint32_t decay_rank, gate_rank;
  float *out_row;
};
constexpr uint32_t kDeltaChunk = 64, kDeltaMaxWidth = 256, kDeltaMaxRank = 4096;
size_t delta_workspace_bytes(const DeltaArgs &args);
hipError_t launch_delta_step(const DeltaArgs &args, hipStream_t stream);
hipError_t launch_delta_prefill(const DeltaArgs &args, hipStream_t stream);

// ---- routed experts -------------------------------------------------------------------------------------

struct RoutePlan {
  uint32_t m, experts, top;
  const float *logits;  // f32 [m, ld_logits]
  uint32_t ld_logits;
  uint32_t *expert;     // [m, top]
  float *weight;        // [m, top]
  uint32_t *position;   // [m, top]: row of the sorted order
  uint32_t *row_token;  // [m * top]
  uint32_t *tile_expert, *tile_first, *tile_rows;  // [max_tiles]
  uint32_t max_tiles, tile;  // tile: rows of a product tile, 64 or 128
};
uint32_t route_tile_rows(uint32_t m, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff, bool f32);
uint32_t route_max_tiles(uint32_t m, uint32_t experts, uint32_t top, uint32_t tile);
// The `top` largest logits of every token (ties to the lower index), the softmax over them, the
// (token, choice) pairs sorted by expert and cut into product tiles of one expert.
hipError_t launch_route(const RoutePlan &plan, hipStream_t stream);
// stream[t, :] += sum_s weight[t, s] rows[position[t, s], :]
struct RouteCombineArgs {
  bool f32;
  const RoutePlan *plan;
  const void *rows;  // activation type [m * top, width]
  float *stream;
  uint32_t width;
};
hipError_t launch_route_combine(const RouteCombineArgs &args, hipStream_t stream);

// One token: every workgroup selects the experts from the logits itself.
struct MoeGemvArgs {
  bool f32;
  const float *logits;  // f32 [experts (+ 1: the shared expert's gate)]
  uint32_t experts, top, width, ff, shared_ff;
  const float *x;                 // f32 [width]
  const uint16_t *norm_weight;
  float epsilon;
  const uint16_t *gate, *up;      // bf16 [experts][ff, width]
  const uint16_t *down;           // bf16 [experts][width, ff]
  const uint16_t *shared_gate, *shared_up, *shared_down;
  float *hidden;                  // f32 [top][ff] then [shared_ff]
  float *stream;                  // f32 [width]
  uint32_t activation;
};
hipError_t launch_moe_gemv_up(const MoeGemvArgs &args, hipStream_t stream);
hipError_t launch_moe_gemv_down(const MoeGemvArgs &args, hipStream_t stream);

}  // namespace llmopt
