// Entry points of layered decoders whose norms sit on the sublayers' outputs and whose mixers run side by
// side on one input: a pending output that joins the stream at the next reader, the joint projection of
// several mixers, attention with normalised and rotated heads, the gated delta rule.  The conventions are
// those of ops_dense.cpp: names end in the activation type, any number of tokens m >= 1, step words.
//
// Pending outputs: a sublayer leaves its raw output y (float32); who reads the stream next adds
// scale y / rms(y) (offset + weight) to it and leaves the new stream in another buffer (one token: inside the
// launch of its product, where every workgroup needs the old row).  pending == 0: y, its weight and the new
// stream's buffer are not touched.
#include "ops_dense.h"

namespace llmopt {
namespace {

struct Pending {
  const float *x, *y;
  const uint16_t *weight;
  float *stream_out;
  float epsilon, offset, scale;
};

// Operands first .. first + 3: stream f32 [m, width], y f32 [m, width], its norm weight, new stream f32;
// parameters at `at`: u32 pending, f32 epsilon, offset, scale.
int read_pending(const DispatchRecord &record, int first, size_t at, uint64_t m, uint64_t width, bool stored, Pending *p) {
  const uint32_t pending = param_u32(record, at);
  p->epsilon = param_f32(record, at + 4);
  p->offset = param_f32(record, at + 8);
  p->scale = param_f32(record, at + 12);
  if (pending > 1 || !valid_epsilon(p->epsilon) || !std::isfinite(p->offset) || !std::isfinite(p->scale))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", record.name.c_str());
  const uint64_t rows = m * width * 4;
  if (int status = require_sizes(record, {{first, rows},
                                          {first + 1, pending ? rows : 0},
                                          {first + 2, pending ? width * 2 : 0},
                                          {first + 3, pending && stored ? rows : 0}}))
    return status;
  p->x = as_f32(record.buffers[first]);
  p->y = pending ? as_f32(record.buffers[first + 1]) : nullptr;
  p->weight = as_bf16(record.buffers[first + 2]);
  p->stream_out = pending && stored ? as_f32(record.buffers[first + 3]) : nullptr;
  if (p->stream_out == p->x)
    return fail(LLMOPT_ERR_INVALID, "%s cannot leave the new stream in place of the old one", record.name.c_str());
  return LLMOPT_OK;
}

NormAddArgs norm_add_args(bool f32, const Pending &p, uint32_t rows, uint32_t width) {
  NormAddArgs a = {};
  a.f32 = f32;
  a.x = p.x;
  a.y = p.y;
  a.add_weight = p.weight;
  a.stream_out = p.stream_out;
  a.rows = rows;
  a.width = width;
  a.epsilon = p.epsilon;
  a.offset = p.offset;
  a.scale = p.scale;
  return a;
}

// The product of one float32 row, a pending output included.
DenseGemvArgs row_product(bool f32, const Pending &p, const uint16_t *w, uint32_t n, uint32_t k) {
  DenseGemvArgs a = {};
  a.f32 = f32;
  a.x = p.x;
  a.x_is_f32 = true;
  a.norm_groups = 1;
  a.epsilon = p.epsilon;
  a.pending = p.y;
  a.pending_weight = p.weight;
  a.stream_out = p.stream_out;
  a.pending_scale = p.scale;
  a.norm_offset = p.offset;
  a.w = w;
  a.n = n;
  a.k = k;
  return a;
}

int too_long(const char *name) { return fail(LLMOPT_ERR_INVALID, "%s takes rows of at most 36864 values", name); }

// The stream of m > 1 tokens as a product's operand: a pending output joins it, bf16 rows go to `operand`.
template <bool F32>
int operand_rows(llmopt_hip_context *context, const char *name, const Pending &p, uint32_t m, uint32_t width, void *operand,
                 const void **x) {
  *x = F32 ? static_cast<const void *>(p.y ? p.stream_out : p.x) : operand;
  if (F32 && !p.y) return LLMOPT_OK;
  NormAddArgs a = norm_add_args(F32, p, m, width);
  a.operand = F32 ? nullptr : operand;
  return launched(launch_norm_add(a, context->stream), name);
}

// {u32 m, width, pending; f32 epsilon, offset, scale}; stream, y, its norm weight, new stream.
int norm_add(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 4)) return status;
  if (int status = require_parameter_bytes(record, 24)) return status;
  const uint32_t m = param_u32(record, 0), width = param_u32(record, 4);
  if (int status = require_positive(record, {m, width})) return status;
  Pending p;
  if (int status = read_pending(record, 0, 8, m, width, true, &p)) return status;
  if (!p.y) return fail(LLMOPT_ERR_INVALID, "%s takes a pending output", record.name.c_str());
  return launched(launch_norm_add(norm_add_args(true, p, m, width), context->stream), record.name.c_str());
}

// {u32 rows, width, vocabulary, m, pending; f32 epsilon, offset, scale, softcap}; stream, y, its norm weight, (unused),
// row indices u32 [rows] (each below m; one row of one: not read), final norm weight, head, logits f32
// [rows, vocabulary].
template <bool F32>
int pending_logits(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 8)) return status;
  if (int status = require_parameter_bytes(record, 36)) return status;
  const char *name = record.name.c_str();
  const uint32_t rows = param_u32(record, 0), width = param_u32(record, 4), vocabulary = param_u32(record, 8),
                 m = param_u32(record, 12);
  const float softcap = param_f32(record, 32);
  if (int status = require_positive(record, {rows, width, vocabulary, m})) return status;
  if (!(softcap >= 0.0f)) return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  Pending p;
  if (int status = read_pending(record, 0, 16, m, width, false, &p)) return status;
  if (int status = require_sizes(record, {{4, (uint64_t)rows * 4},
                                          {5, (uint64_t)width * 2},
                                          {6, (uint64_t)vocabulary * width * 2},
                                          {7, (uint64_t)rows * vocabulary * 4}}))
    return status;
  const bool single = m == 1 && rows == 1;
  const uint16_t *head = as_bf16(record.buffers[6]);
  if (single) {
    DenseGemvArgs a = row_product(F32, p, head, vocabulary, width);
    a.norm_weight = as_bf16(record.buffers[5]);
    a.epilogue = GemvEpilogue::kStoreF32;
    a.softcap = softcap;
    a.out_f32 = as_f32(record.buffers[7]);
    if (dense_gemv_ok(a)) return launched(launch_dense_gemv(a, context->stream), name);
  }
  Scratch scratch;
  const size_t normed = scratch.want((size_t)rows * width * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  NormAddArgs norm = norm_add_args(F32, p, rows, width);
  norm.norm_weight = as_bf16(record.buffers[5]);
  norm.operand = scratch.at<void>(normed);
  norm.rows_index = single ? nullptr : as_u32(record.buffers[4]);
  if (int status = launched(launch_norm_add(norm, context->stream), name)) return status;
  DenseLinearArgs a = linear(F32, scratch.at<void>(normed), head, rows, vocabulary, width);
  a.epilogue = DenseEpilogue::kStoreF32;
  a.out_f32 = as_f32(record.buffers[7]);
  a.ld_f32 = vocabulary;
  if (int status = launched(launch_dense_gemm(a, context->stream), name)) return status;
  if (softcap == 0.0f) return LLMOPT_OK;
  return launched(launch_soft_cap(a.out_f32, (uint64_t)rows * vocabulary, softcap, context->stream), name);
}

// {u32 m, width, n, split, conv_first, conv_channels, taps, slots, pending; f32 epsilon, offset, scale}; stream, y, its
// norm weight, new stream, weights [n, width], step words, convolution weights [conv_channels, taps], its ring f32
// [slots][taps][conv_channels], projected, extra.
// More than one token: projected [m, split] activation type, extra f32 [m, n - split] the columns behind.  One token:
// projected f32 [n], the convolution, its silu and the ring row done for its columns (conv_channels may be 0).
template <bool F32>
int joint_input(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 10)) return status;
  if (int status = require_parameter_bytes(record, 48)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), width = param_u32(record, 4), n = param_u32(record, 8),
                 split = param_u32(record, 12), first = param_u32(record, 16), channels = param_u32(record, 20),
                 taps = param_u32(record, 24), slots = param_u32(record, 28);
  if (int status = require_positive(record, {m, width, n, split, taps, slots})) return status;
  if (split > n || (uint64_t)first + channels > split)
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  Pending p;
  if (int status = read_pending(record, 0, 32, m, width, true, &p)) return status;
  if (int status = require_sizes(record, {{4, (uint64_t)n * width * 2},
                                          {5, kStateWords * 4},
                                          {6, (uint64_t)channels * taps * 2},
                                          {7, (uint64_t)slots * taps * channels * 4},
                                          {8, m == 1 ? (uint64_t)n * 4 : (uint64_t)m * split * kElement<F32>},
                                          {9, m == 1 ? 0 : (uint64_t)m * (n - split) * 4}}))
    return status;
  if (m == 1) {
    DenseGemvArgs a = row_product(F32, p, as_bf16(record.buffers[4]), n, width);
    a.epilogue = GemvEpilogue::kConvIn;
    a.out_f32 = as_f32(record.buffers[8]);
    a.state = as_u32(record.buffers[5]);
    a.conv = as_bf16(record.buffers[6]);
    a.conv_state = as_f32(record.buffers[7]);
    a.inner = first;
    a.channels = channels;
    a.taps = taps;
    if (!dense_gemv_ok(a)) return too_long(name);
    return launched(launch_dense_gemv(a, context->stream), name);
  }
  Scratch scratch;
  const size_t operand = scratch.want(F32 ? 0 : (size_t)m * width * 2);
  if (!F32 && !scratch.get(context)) return LLMOPT_ERR_FAILURE;
  const void *x;
  if (int status = operand_rows<F32>(context, name, p, m, width, F32 ? nullptr : scratch.at<void>(operand), &x)) return status;
  DenseLinearArgs a = linear(F32, x, as_bf16(record.buffers[4]), m, n, width);
  a.epilogue = DenseEpilogue::kSplit;
  a.split = split;
  a.out = record.buffers[8].device;
  a.ld_out = split;
  a.out_f32 = as_f32(record.buffers[9]);
  a.ld_f32 = n - split;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// {u32 m, heads, kv_heads, dim, vdim, ld, ld_out, capacity, span, sliding, slots, rotated; f32 scale, softcap, epsilon,
// out_scale}; projected rows (q | k | v from column 0 on, stride ld; q and k are normalised and rotated in place), q norm,
// k norm bf16 [dim], frequencies f64 [rotated / 2], step words, key ring, value ring, out (from column 0 on, stride
// ld_out).  One token: projected and out are float32 rows, q and k stay as they are.
template <bool F32>
int rotary_attention(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 8)) return status;
  if (int status = require_parameter_bytes(record, 64)) return status;
  const char *name = record.name.c_str();
  ChunkAttentionArgs a = {};
  a.f32 = F32;
  a.m = param_u32(record, 0);
  a.heads = param_u32(record, 4);
  a.kv_heads = param_u32(record, 8);
  a.dim = param_u32(record, 12);
  a.vdim = param_u32(record, 16);
  a.ld = param_u32(record, 20);
  a.ld_out = param_u32(record, 24);
  a.cache = {record.buffers[5].device, record.buffers[6].device, param_u32(record, 28), param_u32(record, 32),
             param_u32(record, 36) != 0};
  const uint32_t slots = param_u32(record, 40);
  a.rotation = {as_bf16(record.buffers[1]), as_bf16(record.buffers[2]),
                reinterpret_cast<const double *>(record.buffers[3].device), param_u32(record, 44), param_f32(record, 56)};
  a.scale = param_f32(record, 48);
  a.softcap = param_f32(record, 52);
  a.out_scale = param_f32(record, 60);
  if (int status = require_positive(record, {a.m, a.heads, a.kv_heads, a.dim, a.vdim, a.cache.capacity, slots})) return status;
  const uint64_t n = (uint64_t)a.heads * a.dim + (uint64_t)a.kv_heads * (a.dim + a.vdim), n_out = (uint64_t)a.heads * a.vdim;
  if (a.cache.span > a.cache.capacity || a.heads % a.kv_heads != 0 || !std::isfinite(a.scale) || !(a.softcap >= 0.0f) ||
      !std::isfinite(a.out_scale) || !valid_epsilon(a.rotation.epsilon) || a.rotation.dims > a.dim ||
      a.rotation.dims % 2 != 0 || a.ld < n || a.ld_out < n_out)
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  if (!chunk_attention_ok(a)) return fail(LLMOPT_ERR_INVALID, "%s takes heads of at most 256 values", name);
  const uint64_t rows = (uint64_t)slots * a.kv_heads * a.cache.capacity * kElement<F32>;
  const uint64_t element = a.m == 1 ? 4 : kElement<F32>;
  if (int status = require_sizes(record, {{0, ((uint64_t)(a.m - 1) * a.ld + n) * element},
                                          {1, (uint64_t)a.dim * 2},
                                          {2, (uint64_t)a.dim * 2},
                                          {3, (uint64_t)a.rotation.dims / 2 * 8},
                                          {4, kStateWords * 4},
                                          {5, rows * a.dim},
                                          {6, rows * a.vdim},
                                          {7, ((uint64_t)(a.m - 1) * a.ld_out + n_out) * element}}))
    return status;
  a.state = as_u32(record.buffers[4]);
  if (a.m == 1) {
    a.row = as_f32(record.buffers[0]);
    a.out_row = as_f32(record.buffers[7]);
    a.workspace_bytes = chunk_attention_workspace_bytes(a);
    if (a.workspace_bytes) {
      a.workspace = context_workspace(context, a.workspace_bytes);
      if (a.workspace == nullptr) return LLMOPT_ERR_FAILURE;
    }
    return launched(launch_chunk_attention(a, context->stream), name);
  }
  a.qkv = record.buffers[0].device;
  a.out = record.buffers[7].device;
  if (int status = launched(launch_rotate_heads(a, context->stream), name)) return status;
  if (int status = launched(launch_chunk_attention(a, context->stream), name)) return status;
  return launched(launch_chunk_cache_write(a, context->stream), name);
}

// {u32 m, heads, kv_heads, dim, vdim, taps, slots, ld, first, decay_first, gate_first, beta_first, decay_rank, gate_rank,
// ld_out, out_first; f32 epsilon, out_scale}; projected rows and extra as joint_input left them (columns: `first` q | k | v,
// the inputs of the low-rank products for decay and gate; extra, from column beta_first on: the write strengths f32
// [m, heads]), decay weights [heads * dim, decay_rank], dt bias [heads * dim], log decay rate [heads], gate weights
// [heads * vdim, gate_rank], norm weight [vdim], convolution weights, its ring, state f32 [slots][heads][dim][vdim], step
// words, out (columns out_first .. of rows of ld_out).  One token: projected and out are float32 rows.
template <bool F32>
int gated_delta(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 12)) return status;
  if (int status = require_parameter_bytes(record, 72)) return status;
  const char *name = record.name.c_str();
  DeltaArgs a = {};
  a.f32 = F32;
  a.m = param_u32(record, 0);
  a.heads = param_u32(record, 4);
  a.kv_heads = param_u32(record, 8);
  a.dim = param_u32(record, 12);
  a.vdim = param_u32(record, 16);
  a.taps = param_u32(record, 20);
  const uint32_t slots = param_u32(record, 24), first = param_u32(record, 32), decay_first = param_u32(record, 36),
                 gate_first = param_u32(record, 40), beta_first = param_u32(record, 44), out_first = param_u32(record, 60);
  a.ld = param_u32(record, 28);
  a.decay_rank = param_u32(record, 48);
  a.gate_rank = param_u32(record, 52);
  a.ld_out = param_u32(record, 56);
  a.epsilon = param_f32(record, 64);
  a.out_scale = param_f32(record, 68);
  if (int status = require_positive(record, {a.m, a.heads, a.kv_heads, a.dim, a.vdim, a.taps, slots, a.decay_rank, a.gate_rank}))
    return status;
  const uint64_t n_decay = (uint64_t)a.heads * a.dim, n_out = (uint64_t)a.heads * a.vdim;
  const uint64_t channels = 2 * (uint64_t)a.kv_heads * a.dim + n_out;
  if (a.heads % a.kv_heads != 0 || !valid_epsilon(a.epsilon) || !std::isfinite(a.out_scale) || first + channels > a.ld ||
      (uint64_t)decay_first + a.decay_rank > a.ld || (uint64_t)gate_first + a.gate_rank > a.ld || beta_first < a.ld ||
      out_first + n_out > a.ld_out)
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  if (a.dim > kDeltaMaxWidth || a.vdim > kDeltaMaxWidth || a.decay_rank > kDeltaMaxRank || a.gate_rank > kDeltaMaxRank)
    return fail(LLMOPT_ERR_INVALID, "%s takes heads of at most 256 values and ranks of at most 4096", name);
  const uint64_t element = a.m == 1 ? 4 : kElement<F32>;
  if (int status = require_sizes(
          record, {{0, a.m == 1 ? ((uint64_t)beta_first + a.heads) * 4 : (uint64_t)a.m * a.ld * element},
                   {1, a.m == 1 ? 0 : (uint64_t)a.m * a.heads * 4},
                   {2, n_decay * a.decay_rank * 2},
                   {3, n_decay * 2},
                   {4, (uint64_t)a.heads * 2},
                   {5, n_out * a.gate_rank * 2},
                   {6, (uint64_t)a.vdim * 2},
                   {7, channels * a.taps * 2},
                   {8, (uint64_t)slots * a.taps * channels * 4},
                   {9, (uint64_t)slots * n_decay * a.vdim * 4},
                   {10, kStateWords * 4},
                   {11, ((uint64_t)(a.m - 1) * a.ld_out + out_first + n_out) * element}}))
    return status;
  a.w_decay = as_bf16(record.buffers[2]);
  a.dt_bias = as_bf16(record.buffers[3]);
  a.a_log = as_bf16(record.buffers[4]);
  a.w_gate = as_bf16(record.buffers[5]);
  a.norm = as_bf16(record.buffers[6]);
  a.conv = as_bf16(record.buffers[7]);
  a.conv_state = as_f32(record.buffers[8]);
  a.state = as_f32(record.buffers[9]);
  a.step = as_u32(record.buffers[10]);
  if (a.m == 1) {
    const float *row = as_f32(record.buffers[0]);
    a.row = row + first;
    a.row_beta = row + beta_first;
    a.decay_in = row + decay_first;
    a.gate_in = row + gate_first;
    a.out_row = as_f32(record.buffers[11]) + out_first;
    return launched(launch_delta_step(a, context->stream), name);
  }
  const uint8_t *projected = reinterpret_cast<const uint8_t *>(record.buffers[0].device);
  Scratch scratch;
  const size_t decay = scratch.want((size_t)a.m * n_decay * 4), gate = scratch.want((size_t)a.m * n_out * element);
  a.workspace_bytes = delta_workspace_bytes(a);
  const size_t workspace = scratch.want(a.workspace_bytes);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  DenseLinearArgs low = linear(F32, projected + decay_first * element, a.w_decay, a.m, (uint32_t)n_decay, a.decay_rank);
  low.ldx = a.ld;
  low.epilogue = DenseEpilogue::kStoreF32;
  low.out_f32 = scratch.at<float>(decay);
  low.ld_f32 = (uint32_t)n_decay;
  if (int status = launched(launch_dense_gemm(low, context->stream), name)) return status;
  low = linear(F32, projected + gate_first * element, a.w_gate, a.m, (uint32_t)n_out, a.gate_rank);
  low.ldx = a.ld;
  low.epilogue = DenseEpilogue::kStore;
  low.out = scratch.at<void>(gate);
  low.ld_out = (uint32_t)n_out;
  if (int status = launched(launch_dense_gemm(low, context->stream), name)) return status;
  a.projected = projected + first * element;
  a.beta = as_f32(record.buffers[1]);
  a.decay = scratch.at<float>(decay);
  a.gate = scratch.at<void>(gate);
  a.out = reinterpret_cast<uint8_t *>(record.buffers[11].device) + out_first * element;
  a.workspace = scratch.at<void>(workspace);
  return launched(launch_delta_prefill(a, context->stream), name);
}

// {u32 m, n, k}; x [m, k] (one token: f32), weight [n, k], out f32 [m, n] = x w^T.
template <bool F32>
int linear_store(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 3)) return status;
  if (int status = require_parameter_bytes(record, 12)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), n = param_u32(record, 4), k = param_u32(record, 8);
  if (int status = require_positive(record, {m, n, k})) return status;
  if (int status = require_sizes(record, {{0, (uint64_t)m * k * (m == 1 ? 4 : kElement<F32>)},
                                          {1, (uint64_t)n * k * 2},
                                          {2, (uint64_t)m * n * 4}}))
    return status;
  if (m == 1) {
    Pending p = {};
    p.x = as_f32(record.buffers[0]);
    DenseGemvArgs a = row_product(F32, p, as_bf16(record.buffers[1]), n, k);
    a.epilogue = GemvEpilogue::kStoreF32;
    a.out_f32 = as_f32(record.buffers[2]);
    if (!dense_gemv_ok(a)) return too_long(name);
    return launched(launch_dense_gemv(a, context->stream), name);
  }
  DenseLinearArgs a = linear(F32, record.buffers[0].device, as_bf16(record.buffers[1]), m, n, k);
  a.epilogue = DenseEpilogue::kStoreF32;
  a.out_f32 = as_f32(record.buffers[2]);
  a.ld_f32 = n;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// {u32 m, width, ff, activation; f32 limit; u32 pending; f32 epsilon, offset, scale}; stream, y, its norm weight, new
// stream, gate, up [ff, width], down [width, ff], out f32 [m, width] (may be y): down(gated(gate x, up x)) of the new
// stream x.  activation 0 silu, 1 gelu (tanh form), 2 clamped by limit.
template <bool F32>
int pending_gated_ffn(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 8)) return status;
  if (int status = require_parameter_bytes(record, 36)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), width = param_u32(record, 4), ff = param_u32(record, 8),
                 activation = param_u32(record, 12);
  const float limit = param_f32(record, 16);
  if (int status = require_positive(record, {m, width, ff})) return status;
  if (activation > 2 || !(limit >= 0.0f)) return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  Pending p;
  if (int status = read_pending(record, 0, 20, m, width, true, &p)) return status;
  const uint64_t matrix = (uint64_t)ff * width * 2;
  if (int status = require_sizes(record, {{4, matrix}, {5, matrix}, {6, matrix}, {7, (uint64_t)m * width * 4}})) return status;
  const uint16_t *gate = as_bf16(record.buffers[4]), *up = as_bf16(record.buffers[5]), *down = as_bf16(record.buffers[6]);
  Scratch scratch;
  if (m == 1) {
    const size_t hidden = scratch.want((size_t)ff * 4);
    if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
    DenseGemvArgs a = row_product(F32, p, gate, ff, width);
    a.w_up = up;
    a.epilogue = GemvEpilogue::kGated;
    a.activation = activation;
    a.limit = limit;
    a.out_f32 = scratch.at<float>(hidden);
    Pending row = {};
    row.x = scratch.at<float>(hidden);
    DenseGemvArgs b = row_product(F32, row, down, width, ff);
    b.epilogue = GemvEpilogue::kStoreF32;
    b.out_f32 = as_f32(record.buffers[7]);
    if (!dense_gemv_ok(a) || !dense_gemv_ok(b)) return too_long(name);
    if (int status = launched(launch_dense_gemv(a, context->stream), name)) return status;
    return launched(launch_dense_gemv(b, context->stream), name);
  }
  const size_t operand = scratch.want(F32 ? 0 : (size_t)m * width * 2);
  const size_t hidden = scratch.want((size_t)m * ff * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  const void *x;
  if (int status = operand_rows<F32>(context, name, p, m, width, scratch.at<void>(operand), &x)) return status;
  DenseLinearArgs a = linear(F32, x, gate, m, ff, width);
  a.w_up = up;
  a.epilogue = DenseEpilogue::kGated;
  a.activation = activation;
  a.limit = limit;
  a.out = scratch.at<void>(hidden);
  a.ld_out = ff;
  if (int status = launched(launch_dense_gemm(a, context->stream), name)) return status;
  DenseLinearArgs b = linear(F32, scratch.at<void>(hidden), down, m, width, ff);
  b.epilogue = DenseEpilogue::kStoreF32;
  b.out_f32 = as_f32(record.buffers[7]);
  b.ld_f32 = width;
  return launched(launch_dense_gemm(b, context->stream), name);
}

}  // namespace

void register_parallel_kernels(std::vector<KernelEntryPoint> &table) {
  table.push_back({"llmopt_norm_add_f32", "reduction", norm_add});
  table.push_back({"llmopt_pending_logits_bf16", "linear", pending_logits<false>});
  table.push_back({"llmopt_pending_logits_f32", "linear", pending_logits<true>});
  table.push_back({"llmopt_joint_input_bf16", "linear", joint_input<false>});
  table.push_back({"llmopt_joint_input_f32", "linear", joint_input<true>});
  table.push_back({"llmopt_rotary_attention_bf16", "attention", rotary_attention<false>});
  table.push_back({"llmopt_rotary_attention_f32", "attention", rotary_attention<true>});
  table.push_back({"llmopt_gated_delta_bf16", "triangular-recurrence", gated_delta<false>});
  table.push_back({"llmopt_gated_delta_f32", "triangular-recurrence", gated_delta<true>});
  table.push_back({"llmopt_linear_store_bf16", "linear", linear_store<false>});
  table.push_back({"llmopt_linear_store_f32", "linear", linear_store<true>});
  table.push_back({"llmopt_pending_gated_ffn_bf16", "gated-linear", pending_gated_ffn<false>});
  table.push_back({"llmopt_pending_gated_ffn_f32", "gated-linear", pending_gated_ffn<true>});
}

}  // namespace llmopt
