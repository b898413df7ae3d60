// Entry points over bfloat16 weights (no reference kernels): the building blocks of a layered decoder -
// linears with a float32 residual stream, chunked attention with a softmax sink, the Mamba-2 mixer,
// dense and routed gated feed-forwards.  Every name ends in the activation type, `_bf16` or `_f32`
// (weights are bfloat16 in both; `_f32` uses no reduced-precision product anywhere).
//
// All take any number of tokens m >= 1: one token runs the matrix-vector kernels with the norm, the
// convolution, the cache write or the expert choice inside the launch; more run the matrix-core kernels.
// What moves from step to step - the position of the step's first token and the sequence's state slot -
// is read from two device words (`step words`: u32 position, u32 slot), so that one captured list
// serves every step and every slot.
#include <cstring>

#include "kernels/kernels.h"
#include "ops_dense.h"

namespace llmopt {
namespace {

template <bool F32>
hipError_t norm_rows(const float *x, const uint16_t *weight, void *out, uint32_t rows, uint32_t width, float epsilon,
                     const uint32_t *rows_index, hipStream_t stream) {
  DenseNormArgs norm = {};
  norm.f32 = F32;
  norm.x = x;
  norm.weight = weight;
  norm.out = out;
  norm.rows_index = rows_index;
  norm.rows = rows;
  norm.width = width;
  norm.groups = 1;
  norm.epsilon = epsilon;
  return launch_dense_norm(norm, stream);
}

// A product of a normalised float32 row (one token).
DenseGemvArgs normed_gemv(bool f32, const float *x, const uint16_t *norm, float epsilon, const uint16_t *w, uint32_t n,
                          uint32_t k) {
  DenseGemvArgs a = {};
  a.f32 = f32;
  a.x = x;
  a.x_is_f32 = true;
  a.norm_weight = norm;
  a.norm_groups = 1;
  a.epsilon = epsilon;
  a.w = w;
  a.n = n;
  a.k = k;
  return a;
}

// ---- embedding, logits ---------------------------------------------------------------------------------

// {u32 m, vocabulary, width; f32 scale}; tokens i64, embedding, stream f32.
int embedding_scaled(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 3)) return status;
  if (int status = require_parameter_bytes(record, 16)) return status;
  DenseEmbeddingArgs a = {};
  a.m = param_u32(record, 0);
  a.vocabulary = param_u32(record, 4);
  a.width = param_u32(record, 8);
  a.scale = param_f32(record, 12);
  if (int status = require_positive(record, {a.m, a.vocabulary, a.width})) return status;
  if (int status = require_sizes(record, {{0, (uint64_t)a.m * 8},
                                          {1, (uint64_t)a.vocabulary * a.width * 2},
                                          {2, (uint64_t)a.m * a.width * 4}}))
    return status;
  a.tokens = reinterpret_cast<const int64_t *>(record.buffers[0].device);
  a.embed = as_bf16(record.buffers[1]);
  a.stream = as_f32(record.buffers[2]);
  return launched(launch_dense_embedding(a, context->stream), record.name.c_str());
}

// {u32 rows, width, vocabulary; f32 epsilon; u32 m}; stream f32 [m, width], row indices u32 [rows] (each
// below m), norm weight, head, logits f32 [rows, vocabulary].  One row of one: the indices are not read.
template <bool F32>
int rms_logits(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 5)) return status;
  if (int status = require_parameter_bytes(record, 20)) return status;
  const char *name = record.name.c_str();
  const uint32_t rows = param_u32(record, 0), width = param_u32(record, 4), vocabulary = param_u32(record, 8);
  const uint32_t m = param_u32(record, 16);
  const float epsilon = param_f32(record, 12);
  if (int status = require_positive(record, {rows, width, vocabulary, m})) return status;
  if (!valid_epsilon(epsilon)) return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  if (int status = require_sizes(record, {{0, (uint64_t)m * width * 4},
                                          {1, (uint64_t)rows * 4},
                                          {2, (uint64_t)width * 2},
                                          {3, (uint64_t)vocabulary * width * 2},
                                          {4, (uint64_t)rows * vocabulary * 4}}))
    return status;
  if (m == 1 && rows == 1) {
    DenseGemvArgs a = normed_gemv(F32, as_f32(record.buffers[0]), as_bf16(record.buffers[2]), epsilon,
                                  as_bf16(record.buffers[3]), vocabulary, width);
    a.epilogue = GemvEpilogue::kStoreF32;
    a.out_f32 = as_f32(record.buffers[4]);
    if (dense_gemv_ok(a)) return launched(launch_dense_gemv(a, context->stream), name);
  }
  Scratch scratch;
  const size_t normed = scratch.want((size_t)rows * width * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  if (int status = launched(norm_rows<F32>(as_f32(record.buffers[0]), as_bf16(record.buffers[2]),
                                           scratch.at<void>(normed), rows, width, epsilon,
                                           m == 1 && rows == 1 ? nullptr : as_u32(record.buffers[1]), context->stream),
                            name))
    return status;
  DenseLinearArgs a = linear(F32, scratch.at<void>(normed), as_bf16(record.buffers[3]), rows, vocabulary, width);
  a.epilogue = DenseEpilogue::kStoreF32;
  a.out_f32 = as_f32(record.buffers[4]);
  a.ld_f32 = vocabulary;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// {u32 rows, n}; logits f32 [rows, n], token ids u32 [rows]: ties to the lower index.
int argmax_f32(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 2)) return status;
  if (int status = require_parameter_bytes(record, 8)) return status;
  const uint32_t rows = param_u32(record, 0), n = param_u32(record, 4);
  if (int status = require_positive(record, {rows, n})) return status;
  if (int status = require_sizes(record, {{0, (uint64_t)rows * n * 4}, {1, (uint64_t)rows * 4}})) return status;
  Scratch scratch;
  const size_t candidates = scratch.want((size_t)rows * 256 * 8);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  if (int status = launched(launch_argmax_candidates(as_f32(record.buffers[0]), scratch.at<void>(candidates), rows, n,
                                                     false, nullptr, context->stream),
                            record.name.c_str()))
    return status;
  return launched(launch_argmax_reduce(scratch.at<void>(candidates),
                                       reinterpret_cast<uint32_t *>(record.buffers[1].device), rows, context->stream),
                  record.name.c_str());
}

// ---- attention mixer -------------------------------------------------------------------------------------

// {u32 m, width, heads, kv_heads, dim, vdim; f32 epsilon; u32 mix_mode; f32 lambda; u32 capacity, chunk,
// slots}; stream f32 [m, width], norm weight, q | k | v weights [n, width], step words, qkv out [m, n],
// first values f32 [m, kv_heads * vdim] (mix_mode 1: written, 2: read), key ring, value ring.
// One token: k and v go to their ring rows and only q is written to qkv; more: qkv only.
template <bool F32>
int rms_qkv(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 8)) return status;
  if (int status = require_parameter_bytes(record, 48)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), width = param_u32(record, 4), heads = param_u32(record, 8),
                 kv_heads = param_u32(record, 12), dim = param_u32(record, 16), vdim = param_u32(record, 20),
                 capacity = param_u32(record, 36), chunk = param_u32(record, 40), slots = param_u32(record, 44);
  const float epsilon = param_f32(record, 24);
  ValueMix mix = {};
  mix.mode = param_u32(record, 28);
  mix.lambda = param_f32(record, 32);
  mix.v_first = as_f32(record.buffers[5]);
  if (int status = require_positive(record, {m, width, heads, kv_heads, dim, vdim, capacity, slots})) return status;
  if (mix.mode > 2 || chunk > capacity || heads % kv_heads != 0 || !valid_epsilon(epsilon))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  const uint32_t n_q = heads * dim, n_k = kv_heads * dim, n_v = kv_heads * vdim, n = n_q + n_k + n_v;
  const uint64_t rows = (uint64_t)slots * kv_heads * capacity * kElement<F32>;
  if (int status = require_sizes(record, {{0, (uint64_t)m * width * 4},
                                          {1, (uint64_t)width * 2},
                                          {2, (uint64_t)n * width * 2},
                                          {3, kStateWords * 4},
                                          {4, (uint64_t)m * n * kElement<F32>},
                                          {5, mix.mode ? (uint64_t)m * n_v * 4 : 0},
                                          {6, rows * dim},
                                          {7, rows * vdim}}))
    return status;
  if (m == 1) {
    DenseGemvArgs a = normed_gemv(F32, as_f32(record.buffers[0]), as_bf16(record.buffers[1]), epsilon,
                                  as_bf16(record.buffers[2]), n, width);
    a.epilogue = GemvEpilogue::kQkv;
    a.out = record.buffers[4].device;
    a.state = as_u32(record.buffers[3]);
    a.n_q = n_q;
    a.n_k = n_k;
    a.dim = dim;
    a.vdim = vdim;
    a.kv_heads = kv_heads;
    a.cache = {record.buffers[6].device, record.buffers[7].device, capacity, chunk};
    a.mix = mix;
    if (!dense_gemv_ok(a)) return fail(LLMOPT_ERR_INVALID, "%s takes rows of at most 36864 values", name);
    return launched(launch_dense_gemv(a, context->stream), name);
  }
  Scratch scratch;
  const size_t normed = scratch.want((size_t)m * width * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  if (int status = launched(norm_rows<F32>(as_f32(record.buffers[0]), as_bf16(record.buffers[1]),
                                           scratch.at<void>(normed), m, width, epsilon, nullptr, context->stream),
                            name))
    return status;
  DenseLinearArgs a = linear(F32, scratch.at<void>(normed), as_bf16(record.buffers[2]), m, n, width);
  a.epilogue = DenseEpilogue::kQkv;
  a.out = record.buffers[4].device;
  a.ld_out = n;
  a.split = n_q + n_k;
  a.mix = mix;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// {u32 m, heads, kv_heads, dim, vdim, capacity, chunk, slots, has_sink; f32 scale, softcap}; qkv rows, sink
// bf16 [heads] (has_sink == 0: not read), step words, key ring, value ring, out [m, heads * vdim].
// Leaves the step's keys and values in the rings (one token: the projection already did).
template <bool F32>
int chunk_attention(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 6)) return status;
  if (int status = require_parameter_bytes(record, 44)) return status;
  const char *name = record.name.c_str();
  ChunkAttentionArgs a = {};
  a.f32 = F32;
  a.m = param_u32(record, 0);
  a.heads = param_u32(record, 4);
  a.kv_heads = param_u32(record, 8);
  a.dim = param_u32(record, 12);
  a.vdim = param_u32(record, 16);
  a.cache = {record.buffers[3].device, record.buffers[4].device, param_u32(record, 20), param_u32(record, 24)};
  const uint32_t slots = param_u32(record, 28), has_sink = param_u32(record, 32);
  a.scale = param_f32(record, 36);
  a.softcap = param_f32(record, 40);
  if (int status = require_positive(record, {a.m, a.heads, a.kv_heads, a.dim, a.vdim, a.cache.capacity, slots}))
    return status;
  if (a.cache.span > a.cache.capacity || a.heads % a.kv_heads != 0 || !std::isfinite(a.scale) || !(a.softcap >= 0.0f))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  if (!chunk_attention_ok(a))
    return fail(LLMOPT_ERR_INVALID, "%s takes heads of at most 256 values", name);
  const uint64_t rows = (uint64_t)slots * a.kv_heads * a.cache.capacity * kElement<F32>;
  const uint32_t n = a.heads * a.dim + a.kv_heads * (a.dim + a.vdim);
  if (int status = require_sizes(record, {{0, (uint64_t)a.m * n * kElement<F32>},
                                          {1, has_sink ? (uint64_t)a.heads * 2 : 0},
                                          {2, kStateWords * 4},
                                          {3, rows * a.dim},
                                          {4, rows * a.vdim},
                                          {5, (uint64_t)a.m * a.heads * a.vdim * kElement<F32>}}))
    return status;
  a.qkv = record.buffers[0].device;
  a.sink = has_sink ? as_bf16(record.buffers[1]) : nullptr;
  a.state = as_u32(record.buffers[2]);
  a.out = record.buffers[5].device;
  a.ld = n;
  a.ld_out = a.heads * a.vdim;
  a.out_scale = 1.0f;
  a.workspace_bytes = chunk_attention_workspace_bytes(a);
  if (a.workspace_bytes) {
    a.workspace = context_workspace(context, a.workspace_bytes);
    if (a.workspace == nullptr) return LLMOPT_ERR_FAILURE;
  }
  if (int status = launched(launch_chunk_attention(a, context->stream), name)) return status;
  return a.m == 1 ? LLMOPT_OK : launched(launch_chunk_cache_write(a, context->stream), name);
}

// {u32 m, n, k}; x [m, k], weight [n, k], stream f32 [m, n]: stream += x w^T.
template <bool F32>
int linear_add(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 3)) return status;
  if (int status = require_parameter_bytes(record, 12)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), n = param_u32(record, 4), k = param_u32(record, 8);
  if (int status = require_positive(record, {m, n, k})) return status;
  if (int status = require_sizes(record, {{0, (uint64_t)m * k * kElement<F32>},
                                          {1, (uint64_t)n * k * 2},
                                          {2, (uint64_t)m * n * 4}}))
    return status;
  if (m == 1) {
    DenseGemvArgs a = {};
    a.f32 = F32;
    a.x = record.buffers[0].device;
    a.w = as_bf16(record.buffers[1]);
    a.n = n;
    a.k = k;
    a.epilogue = GemvEpilogue::kAdd;
    a.out_f32 = as_f32(record.buffers[2]);
    if (dense_gemv_ok(a)) return launched(launch_dense_gemv(a, context->stream), name);
  }
  DenseLinearArgs a = linear(F32, record.buffers[0].device, as_bf16(record.buffers[1]), m, n, k);
  a.epilogue = DenseEpilogue::kAdd;
  a.out_f32 = as_f32(record.buffers[2]);
  a.ld_f32 = n;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// ---- Mamba-2 mixer ----------------------------------------------------------------------------------------

// {u32 m, width, heads, vdim, groups, state_size, taps, slots; f32 epsilon}; stream, norm weight, weights
// [2 * heads * vdim + 2 * groups * state_size + heads, width], step words, convolution weights [channels,
// taps], its bias, dt bias, convolution ring f32 [slots][taps][channels], projected, dt f32 [m, heads].
// More than one token: projected [m, z | x B C], dt before the softplus.  One token: projected is the f32
// row z | x B C | dt with the convolution, its silu and the softplus done and the ring row written.
struct SsmSizes {
  uint32_t m, width, heads, vdim, groups, state_size, taps, slots;
  uint32_t inner() const { return heads * vdim; }
  uint32_t channels() const { return inner() + 2 * groups * state_size; }
};

template <bool F32>
int rms_ssm_input(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 10)) return status;
  if (int status = require_parameter_bytes(record, 36)) return status;
  const char *name = record.name.c_str();
  const SsmSizes s = {param_u32(record, 0),  param_u32(record, 4),  param_u32(record, 8),  param_u32(record, 12),
                      param_u32(record, 16), param_u32(record, 20), param_u32(record, 24), param_u32(record, 28)};
  const float epsilon = param_f32(record, 32);
  if (int status = require_positive(record, {s.m, s.width, s.heads, s.vdim, s.groups, s.state_size, s.taps, s.slots}))
    return status;
  if (s.heads % s.groups != 0 || !valid_epsilon(epsilon))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  const uint32_t columns = s.inner() + s.channels(), n = columns + s.heads;
  if (int status = require_sizes(record, {{0, (uint64_t)s.m * s.width * 4},
                                          {1, (uint64_t)s.width * 2},
                                          {2, (uint64_t)n * s.width * 2},
                                          {3, kStateWords * 4},
                                          {4, (uint64_t)s.channels() * s.taps * 2},
                                          {5, (uint64_t)s.channels() * 2},
                                          {6, (uint64_t)s.heads * 2},
                                          {7, (uint64_t)s.slots * s.taps * s.channels() * 4},
                                          {8, s.m == 1 ? (uint64_t)n * 4 : (uint64_t)s.m * columns * kElement<F32>},
                                          {9, (uint64_t)s.m * s.heads * 4}}))
    return status;
  if (s.m == 1) {
    DenseGemvArgs a = normed_gemv(F32, as_f32(record.buffers[0]), as_bf16(record.buffers[1]), epsilon,
                                  as_bf16(record.buffers[2]), n, s.width);
    a.epilogue = GemvEpilogue::kSsmIn;
    a.out_f32 = as_f32(record.buffers[8]);
    a.state = as_u32(record.buffers[3]);
    a.conv = as_bf16(record.buffers[4]);
    a.conv_bias = as_bf16(record.buffers[5]);
    a.dt_bias = as_bf16(record.buffers[6]);
    a.conv_state = as_f32(record.buffers[7]);
    a.inner = s.inner();
    a.channels = s.channels();
    a.taps = s.taps;
    if (!dense_gemv_ok(a)) return fail(LLMOPT_ERR_INVALID, "%s takes rows of at most 36864 values", name);
    return launched(launch_dense_gemv(a, context->stream), name);
  }
  Scratch scratch;
  const size_t normed = scratch.want((size_t)s.m * s.width * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  if (int status = launched(norm_rows<F32>(as_f32(record.buffers[0]), as_bf16(record.buffers[1]),
                                           scratch.at<void>(normed), s.m, s.width, epsilon, nullptr, context->stream),
                            name))
    return status;
  DenseLinearArgs a = linear(F32, scratch.at<void>(normed), as_bf16(record.buffers[2]), s.m, n, s.width);
  a.epilogue = DenseEpilogue::kSplit;
  a.split = columns;
  a.out = record.buffers[8].device;
  a.ld_out = columns;
  a.out_f32 = as_f32(record.buffers[9]);
  a.ld_f32 = s.heads;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// {u32 m, heads, vdim, groups, state_size, taps, slots}; step words, projected and dt as above, convolution
// weights, its bias, dt bias, log decay rate, skip gain, convolution ring, recurrent state f32
// [slots][heads][vdim][state_size], y.  y: [m, inner] without the output gate; one token: f32 [inner],
// multiplied by silu(z).
template <bool F32>
int ssm_mix(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 11)) return status;
  if (int status = require_parameter_bytes(record, 28)) return status;
  const char *name = record.name.c_str();
  const SsmSizes s = {param_u32(record, 0),  0,                     param_u32(record, 4),  param_u32(record, 8),
                      param_u32(record, 12), param_u32(record, 16), param_u32(record, 20), param_u32(record, 24)};
  if (int status = require_positive(record, {s.m, s.heads, s.vdim, s.groups, s.state_size, s.taps, s.slots}))
    return status;
  if (s.heads % s.groups != 0) return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  if (s.state_size > 256) return fail(LLMOPT_ERR_INVALID, "%s takes states of at most 256 values", name);
  const uint32_t columns = s.inner() + s.channels();
  if (int status = require_sizes(
          record, {{0, kStateWords * 4},
                   {1, s.m == 1 ? (uint64_t)(columns + s.heads) * 4 : (uint64_t)s.m * columns * kElement<F32>},
                   {2, (uint64_t)s.m * s.heads * 4},
                   {3, (uint64_t)s.channels() * s.taps * 2},
                   {4, (uint64_t)s.channels() * 2},
                   {5, (uint64_t)s.heads * 2},
                   {6, (uint64_t)s.heads * 2},
                   {7, (uint64_t)s.heads * 2},
                   {8, (uint64_t)s.slots * s.taps * s.channels() * 4},
                   {9, (uint64_t)s.slots * s.inner() * s.state_size * 4},
                   {10, (uint64_t)s.m * s.inner() * (s.m == 1 ? 4 : kElement<F32>)}}))
    return status;
  SsmArgs a = {};
  a.f32 = F32;
  a.m = s.m;
  a.heads = s.heads;
  a.vdim = s.vdim;
  a.groups = s.groups;
  a.state_size = s.state_size;
  a.taps = s.taps;
  a.step = as_u32(record.buffers[0]);
  a.projected = record.buffers[1].device;
  a.dt = as_f32(record.buffers[2]);
  a.conv = as_bf16(record.buffers[3]);
  a.conv_bias = as_bf16(record.buffers[4]);
  a.dt_bias = as_bf16(record.buffers[5]);
  a.a_log = as_bf16(record.buffers[6]);
  a.d_skip = as_bf16(record.buffers[7]);
  a.conv_state = as_f32(record.buffers[8]);
  a.ssm_state = as_f32(record.buffers[9]);
  if (s.m == 1) {
    a.row = as_f32(record.buffers[1]);
    a.gated = as_f32(record.buffers[10]);
    return launched(launch_ssm_step(a, context->stream), name);
  }
  a.y = record.buffers[10].device;
  a.workspace_bytes = ssm_workspace_bytes(a);
  a.workspace = context_workspace(context, a.workspace_bytes);
  if (a.workspace == nullptr) return LLMOPT_ERR_FAILURE;
  return launched(launch_ssm_prefill(a, context->stream), name);
}

// {u32 m, inner, ld_gate, norm_groups, width; f32 epsilon}; y [m, inner], gate (columns 0 .. inner - 1 of rows
// of ld_gate), norm weight [inner], output weights [width, inner], stream.  stream += norm(y silu(gate)) w^T,
// every one of norm_groups parts by its own root mean square.  One token: y is f32 with the gate applied.
template <bool F32>
int gated_norm_linear_add(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 5)) return status;
  if (int status = require_parameter_bytes(record, 24)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), inner = param_u32(record, 4), ld_gate = param_u32(record, 8),
                 groups = param_u32(record, 12), width = param_u32(record, 16);
  const float epsilon = param_f32(record, 20);
  if (int status = require_positive(record, {m, inner, groups, width})) return status;
  if (inner % groups != 0 || ld_gate < inner || !valid_epsilon(epsilon))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  if (int status = require_sizes(
          record, {{0, (uint64_t)m * inner * (m == 1 ? 4 : kElement<F32>)},
                   {1, m == 1 ? 0 : ((uint64_t)(m - 1) * ld_gate + inner) * kElement<F32>},
                   {2, (uint64_t)inner * 2},
                   {3, (uint64_t)width * inner * 2},
                   {4, (uint64_t)m * width * 4}}))
    return status;
  if (m == 1) {
    DenseGemvArgs a = normed_gemv(F32, as_f32(record.buffers[0]), as_bf16(record.buffers[2]), epsilon,
                                  as_bf16(record.buffers[3]), width, inner);
    a.norm_groups = groups;
    a.epilogue = GemvEpilogue::kAdd;
    a.out_f32 = as_f32(record.buffers[4]);
    if (!dense_gemv_ok(a)) return fail(LLMOPT_ERR_INVALID, "%s takes rows of at most 36864 values", name);
    return launched(launch_dense_gemv(a, context->stream), name);
  }
  Scratch scratch;
  const size_t normed = scratch.want((size_t)m * inner * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  DenseNormArgs norm = {};
  norm.f32 = F32;
  norm.x_act = record.buffers[0].device;
  norm.gate = record.buffers[1].device;
  norm.ld_gate = ld_gate;
  norm.weight = as_bf16(record.buffers[2]);
  norm.out = scratch.at<void>(normed);
  norm.rows = m;
  norm.width = inner;
  norm.groups = groups;
  norm.epsilon = epsilon;
  if (int status = launched(launch_dense_norm(norm, context->stream), name)) return status;
  DenseLinearArgs a = linear(F32, scratch.at<void>(normed), as_bf16(record.buffers[3]), m, width, inner);
  a.epilogue = DenseEpilogue::kAdd;
  a.out_f32 = as_f32(record.buffers[4]);
  a.ld_f32 = width;
  return launched(launch_dense_gemm(a, context->stream), name);
}

// ---- feed-forwards ----------------------------------------------------------------------------------------

// {u32 m, width, ff; f32 epsilon; u32 activation}; stream, norm weight, gate, up [ff, width], down [width, ff].
// stream += down(act(gate h) * up h), h the normalised stream; activation 0 silu, 1 gelu (tanh form).
template <bool F32>
int rms_gated_ffn_add(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 5)) return status;
  if (int status = require_parameter_bytes(record, 20)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), width = param_u32(record, 4), ff = param_u32(record, 8),
                 activation = param_u32(record, 16);
  const float epsilon = param_f32(record, 12);
  if (int status = require_positive(record, {m, width, ff})) return status;
  if (activation > 1 || !valid_epsilon(epsilon))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  const uint64_t matrix = (uint64_t)ff * width * 2;
  if (int status = require_sizes(record, {{0, (uint64_t)m * width * 4}, {1, (uint64_t)width * 2}, {2, matrix},
                                          {3, matrix}, {4, matrix}}))
    return status;
  float *stream = as_f32(record.buffers[0]);
  Scratch scratch;
  if (m == 1) {
    const size_t hidden = scratch.want((size_t)ff * 4);
    if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
    DenseGemvArgs up = normed_gemv(F32, stream, as_bf16(record.buffers[1]), epsilon, as_bf16(record.buffers[2]), ff, width);
    up.w_up = as_bf16(record.buffers[3]);
    up.epilogue = GemvEpilogue::kGated;
    up.activation = activation;
    up.out_f32 = scratch.at<float>(hidden);
    DenseGemvArgs down = {};
    down.f32 = F32;
    down.x = scratch.at<float>(hidden);
    down.x_is_f32 = true;
    down.w = as_bf16(record.buffers[4]);
    down.n = width;
    down.k = ff;
    down.epilogue = GemvEpilogue::kAdd;
    down.out_f32 = stream;
    if (!dense_gemv_ok(up) || !dense_gemv_ok(down))
      return fail(LLMOPT_ERR_INVALID, "%s takes rows of at most 36864 values", name);
    if (int status = launched(launch_dense_gemv(up, context->stream), name)) return status;
    return launched(launch_dense_gemv(down, context->stream), name);
  }
  const size_t normed = scratch.want((size_t)m * width * kElement<F32>);
  const size_t hidden = scratch.want((size_t)m * ff * kElement<F32>);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  if (int status = launched(norm_rows<F32>(stream, as_bf16(record.buffers[1]), scratch.at<void>(normed), m, width,
                                           epsilon, nullptr, context->stream),
                            name))
    return status;
  DenseLinearArgs up = linear(F32, scratch.at<void>(normed), as_bf16(record.buffers[2]), m, ff, width);
  up.w_up = as_bf16(record.buffers[3]);
  up.epilogue = DenseEpilogue::kGated;
  up.activation = activation;
  up.out = scratch.at<void>(hidden);
  up.ld_out = ff;
  if (int status = launched(launch_dense_gemm(up, context->stream), name)) return status;
  DenseLinearArgs down = linear(F32, scratch.at<void>(hidden), as_bf16(record.buffers[4]), m, width, ff);
  down.epilogue = DenseEpilogue::kAdd;
  down.out_f32 = stream;
  down.ld_f32 = width;
  return launched(launch_dense_gemm(down, context->stream), name);
}

// {u32 m, width, experts, top, ff, shared_ff; f32 epsilon; u32 activation}; stream, norm weight, router
// [experts (+ 1), width] (the last row: the shared expert's gate), gate, up [experts][ff, width], down
// [experts][width, ff], the shared expert's gate, up, down (shared_ff == 0: not read).
// stream += sum over the `top` experts of softmax weight * expert(h) (+ sigmoid(gate) shared(h)).
template <bool F32>
int rms_routed_ffn_add(llmopt_hip_context *context, const DispatchRecord &record) {
  if (int status = require_buffer_count(record, 9)) return status;
  if (int status = require_parameter_bytes(record, 32)) return status;
  const char *name = record.name.c_str();
  const uint32_t m = param_u32(record, 0), width = param_u32(record, 4), experts = param_u32(record, 8),
                 top = param_u32(record, 12), ff = param_u32(record, 16), shared_ff = param_u32(record, 20),
                 activation = param_u32(record, 28);
  const float epsilon = param_f32(record, 24);
  if (int status = require_positive(record, {m, width, experts, top, ff})) return status;
  if (top > experts || experts > 2048 || activation > 1 || !valid_epsilon(epsilon))
    return fail(LLMOPT_ERR_INVALID, "%s input metadata is inconsistent", name);
  const uint32_t columns = experts + (shared_ff ? 1 : 0);
  const uint64_t matrices = (uint64_t)experts * ff * width * 2, shared = (uint64_t)shared_ff * width * 2;
  if (int status = require_sizes(record, {{0, (uint64_t)m * width * 4}, {1, (uint64_t)width * 2},
                                          {2, (uint64_t)columns * width * 2}, {3, matrices}, {4, matrices},
                                          {5, matrices}, {6, shared}, {7, shared}, {8, shared}}))
    return status;
  float *stream = as_f32(record.buffers[0]);
  const uint16_t *norm = as_bf16(record.buffers[1]), *router = as_bf16(record.buffers[2]);
  Scratch scratch;
  const size_t logits = scratch.want((size_t)m * columns * 4);
  if (m == 1) {
    const size_t hidden = scratch.want(((size_t)top * ff + shared_ff) * 4);
    if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
    DenseGemvArgs route = normed_gemv(F32, stream, norm, epsilon, router, columns, width);
    route.epilogue = GemvEpilogue::kStoreF32;
    route.out_f32 = scratch.at<float>(logits);
    if (!dense_gemv_ok(route)) return fail(LLMOPT_ERR_INVALID, "%s takes rows of at most 36864 values", name);
    if (int status = launched(launch_dense_gemv(route, context->stream), name)) return status;
    MoeGemvArgs a = {};
    a.f32 = F32;
    a.logits = scratch.at<float>(logits);
    a.experts = experts;
    a.top = top;
    a.width = width;
    a.ff = ff;
    a.shared_ff = shared_ff;
    a.x = stream;
    a.norm_weight = norm;
    a.epsilon = epsilon;
    a.gate = as_bf16(record.buffers[3]);
    a.up = as_bf16(record.buffers[4]);
    a.down = as_bf16(record.buffers[5]);
    a.shared_gate = as_bf16(record.buffers[6]);
    a.shared_up = as_bf16(record.buffers[7]);
    a.shared_down = as_bf16(record.buffers[8]);
    a.hidden = scratch.at<float>(hidden);
    a.stream = stream;
    a.activation = activation;
    if (int status = launched(launch_moe_gemv_up(a, context->stream), name)) return status;
    return launched(launch_moe_gemv_down(a, context->stream), name);
  }
  const size_t pairs = (size_t)m * top;
  RoutePlan plan = {};
  plan.m = m;
  plan.experts = experts;
  plan.top = top;
  plan.ld_logits = columns;
  plan.tile = route_tile_rows(m, experts, top, width, ff, F32);
  plan.max_tiles = route_max_tiles(m, experts, top, plan.tile);
  const size_t normed = scratch.want((size_t)m * width * kElement<F32>);
  const size_t hidden = scratch.want(std::max(pairs * ff, (size_t)m * shared_ff) * kElement<F32>);
  const size_t rows = scratch.want(pairs * width * kElement<F32>);
  const size_t expert = scratch.want(pairs * 4), weight = scratch.want(pairs * 4), position = scratch.want(pairs * 4),
               row_token = scratch.want(pairs * 4);
  const size_t tile_expert = scratch.want((size_t)plan.max_tiles * 4), tile_first = scratch.want((size_t)plan.max_tiles * 4),
               tile_rows = scratch.want((size_t)plan.max_tiles * 4);
  if (!scratch.get(context)) return LLMOPT_ERR_FAILURE;
  plan.logits = scratch.at<float>(logits);
  plan.expert = scratch.at<uint32_t>(expert);
  plan.weight = scratch.at<float>(weight);
  plan.position = scratch.at<uint32_t>(position);
  plan.row_token = scratch.at<uint32_t>(row_token);
  plan.tile_expert = scratch.at<uint32_t>(tile_expert);
  plan.tile_first = scratch.at<uint32_t>(tile_first);
  plan.tile_rows = scratch.at<uint32_t>(tile_rows);
  void *h = scratch.at<void>(normed);
  if (int status = launched(norm_rows<F32>(stream, norm, h, m, width, epsilon, nullptr, context->stream), name))
    return status;
  DenseLinearArgs route = linear(F32, h, router, m, columns, width);
  route.epilogue = DenseEpilogue::kStoreF32;
  route.out_f32 = scratch.at<float>(logits);
  route.ld_f32 = columns;
  if (int status = launched(launch_dense_gemm(route, context->stream), name)) return status;
  if (int status = launched(launch_route(plan, context->stream), name)) return status;
  // the chosen experts, rows sorted by expert
  DenseLinearArgs up = linear(F32, h, as_bf16(record.buffers[3]), (uint32_t)pairs, ff, width);
  up.w_up = as_bf16(record.buffers[4]);
  up.epilogue = DenseEpilogue::kGated;
  up.activation = activation;
  up.out = scratch.at<void>(hidden);
  up.ld_out = ff;
  up.tile_expert = plan.tile_expert;
  up.tile_first = plan.tile_first;
  up.tile_rows = plan.tile_rows;
  up.tiles = plan.max_tiles;
  up.tile = plan.tile;
  up.row_source = plan.row_token;
  if (int status = launched(launch_dense_gemm(up, context->stream), name)) return status;
  DenseLinearArgs down = linear(F32, scratch.at<void>(hidden), as_bf16(record.buffers[5]), (uint32_t)pairs, width, ff);
  down.epilogue = DenseEpilogue::kStore;
  down.out = scratch.at<void>(rows);
  down.ld_out = width;
  down.tile_expert = plan.tile_expert;
  down.tile_first = plan.tile_first;
  down.tile_rows = plan.tile_rows;
  down.tiles = plan.max_tiles;
  down.tile = plan.tile;
  if (int status = launched(launch_dense_gemm(down, context->stream), name)) return status;
  RouteCombineArgs combine = {F32, &plan, scratch.at<void>(rows), stream, width};
  if (int status = launched(launch_route_combine(combine, context->stream), name)) return status;
  if (shared_ff == 0) return LLMOPT_OK;
  // the expert every token runs
  DenseLinearArgs shared_up = linear(F32, h, as_bf16(record.buffers[6]), m, shared_ff, width);
  shared_up.w_up = as_bf16(record.buffers[7]);
  shared_up.epilogue = DenseEpilogue::kGated;
  shared_up.activation = activation;
  shared_up.out = scratch.at<void>(hidden);
  shared_up.ld_out = shared_ff;
  if (int status = launched(launch_dense_gemm(shared_up, context->stream), name)) return status;
  DenseLinearArgs shared_down = linear(F32, scratch.at<void>(hidden), as_bf16(record.buffers[8]), m, width, shared_ff);
  shared_down.epilogue = DenseEpilogue::kAdd;
  shared_down.out_f32 = stream;
  shared_down.ld_f32 = width;
  shared_down.row_gate = scratch.at<float>(logits) + experts;
  shared_down.row_gate_stride = columns;
  return launched(launch_dense_gemm(shared_down, context->stream), name);
}

}  // namespace

void register_dense_kernels(std::vector<KernelEntryPoint> &table) {
  table.push_back({"llmopt_embedding_scaled_bf16", "embedding", embedding_scaled});
  table.push_back({"llmopt_argmax_f32", "reduction", argmax_f32});
  table.push_back({"llmopt_rms_logits_bf16", "linear", rms_logits<false>});
  table.push_back({"llmopt_rms_logits_f32", "linear", rms_logits<true>});
  table.push_back({"llmopt_rms_qkv_chunk_bf16", "linear", rms_qkv<false>});
  table.push_back({"llmopt_rms_qkv_chunk_f32", "linear", rms_qkv<true>});
  table.push_back({"llmopt_chunk_attention_bf16", "attention", chunk_attention<false>});
  table.push_back({"llmopt_chunk_attention_f32", "attention", chunk_attention<true>});
  table.push_back({"llmopt_linear_add_bf16", "linear", linear_add<false>});
  table.push_back({"llmopt_linear_add_f32", "linear", linear_add<true>});
  table.push_back({"llmopt_rms_ssm_input_bf16", "short-conv", rms_ssm_input<false>});
  table.push_back({"llmopt_rms_ssm_input_f32", "short-conv", rms_ssm_input<true>});
  table.push_back({"llmopt_ssm_mix_bf16", "triangular-recurrence", ssm_mix<false>});
  table.push_back({"llmopt_ssm_mix_f32", "triangular-recurrence", ssm_mix<true>});
  table.push_back({"llmopt_gated_norm_linear_add_bf16", "gated-linear", gated_norm_linear_add<false>});
  table.push_back({"llmopt_gated_norm_linear_add_f32", "gated-linear", gated_norm_linear_add<true>});
  table.push_back({"llmopt_rms_gated_ffn_add_bf16", "gated-linear", rms_gated_ffn_add<false>});
  table.push_back({"llmopt_rms_gated_ffn_add_f32", "gated-linear", rms_gated_ffn_add<true>});
  table.push_back({"llmopt_rms_routed_ffn_add_bf16", "moe-swiglu-ffn", rms_routed_ffn_add<false>});
  table.push_back({"llmopt_rms_routed_ffn_add_f32", "moe-swiglu-ffn", rms_routed_ffn_add<true>});
}

}  // namespace llmopt
