// Matrix-vector products of one token with bfloat16 weights (decode), with the RMSNorm that feeds them
// and the epilogues that follow them in the same launch.
//
// A wave streams ROWS weight rows side by side: 64 lanes x 16 bytes of each row per step of 512 columns,
// four steps requested before the first is used.  The activation is staged once per workgroup in LDS as
// float32, normalised on the way in where the launch carries a norm weight (it is never rounded to the
// activation type), the first and the last four values of every piece of eight in two planes so that a
// wave's 16-byte reads are conflict-free.  Every row's sum meets in one wave reduction; lane r of the
// wave then runs the epilogue of row r.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr uint32_t kGemvMaxK = 36 * 1024;  // float32 activations in 144 KB of LDS
constexpr int kWaves = 4;

// x[k] of the staged activation lives at plane (k / 4) % 2, element 4 (k / 8) + k % 4.
__device__ __forceinline__ uint32_t staged_index(uint32_t k, uint32_t plane) {
  return ((k >> 2) & 1) * plane + ((k >> 3) << 2) + (k & 3);
}

// A row of at most PIECES * 1024 values through registers: one trip to memory.
template <int PIECES, typename Ahead>
__device__ __forceinline__ void stage_normed_row(const DenseGemvArgs &a, float *xs, uint32_t plane, float *scratch,
                                                 Ahead ahead) {
  const uint32_t k = a.k;
  const float *x = static_cast<const float *>(a.x);
  const __bf16 *weight = reinterpret_cast<const __bf16 *>(a.norm_weight);
  f32x4 v[PIECES];
  bf16x4 w[PIECES];
  float sum = 0.0f;
#pragma unroll
  for (int q = 0; q < PIECES; ++q) {
    const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 4;
    v[q] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    if (i < k) {
      v[q] = *reinterpret_cast<const f32x4 *>(x + i);
      w[q] = *reinterpret_cast<const bf16x4 *>(weight + i);
    }
  }
  ahead();
#pragma unroll
  for (int q = 0; q < PIECES; ++q)
    sum += v[q][0] * v[q][0] + v[q][1] * v[q][1] + v[q][2] * v[q][2] + v[q][3] * v[q][3];
  sum = block_sum<kWaves>(sum, scratch);
  const float inverse = 1.0f / sqrtf(sum / (float)k + a.epsilon);
#pragma unroll
  for (int q = 0; q < PIECES; ++q) {
    const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 4;
    if (i < k) {
      f32x4 out;
#pragma unroll
      for (int e = 0; e < 4; ++e) out[e] = v[q][e] * inverse * (a.norm_offset + (float)w[q][e]);
      *reinterpret_cast<f32x4 *>(xs + staged_index(i, plane)) = out;
    }
  }
  __syncthreads();
}

// The f32 row x with a pending sublayer output added behind its norm (the first workgroup stores the new row),
// normalised itself where the launch carries a norm weight.  A row of at most PIECES * 1024 values.
template <int PIECES, typename Ahead>
__device__ __forceinline__ void stage_pending_row(const DenseGemvArgs &a, float *xs, uint32_t plane, float *scratch,
                                                  Ahead ahead) {
  const uint32_t k = a.k;
  const float *x = static_cast<const float *>(a.x);
  const __bf16 *add = reinterpret_cast<const __bf16 *>(a.pending_weight);
  const __bf16 *weight = reinterpret_cast<const __bf16 *>(a.norm_weight);
  f32x4 v[PIECES], y[PIECES];
  bf16x4 w[PIECES];
  float sum = 0.0f;
#pragma unroll
  for (int q = 0; q < PIECES; ++q) {
    const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 4;
    v[q] = y[q] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    w[q] = bf16x4{0, 0, 0, 0};
    if (i < k) {
      v[q] = *reinterpret_cast<const f32x4 *>(x + i);
      y[q] = *reinterpret_cast<const f32x4 *>(a.pending + i);
      w[q] = *reinterpret_cast<const bf16x4 *>(add + i);
    }
  }
  ahead();
#pragma unroll
  for (int q = 0; q < PIECES; ++q)
    sum += y[q][0] * y[q][0] + y[q][1] * y[q][1] + y[q][2] * y[q][2] + y[q][3] * y[q][3];
  const float factor = a.pending_scale / sqrtf(block_sum<kWaves>(sum, scratch) / (float)k + a.epsilon);
  sum = 0.0f;
#pragma unroll
  for (int q = 0; q < PIECES; ++q)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      v[q][e] = fmaf(y[q][e] * factor, a.norm_offset + (float)w[q][e], v[q][e]);
      sum += v[q][e] * v[q][e];
    }
  if (blockIdx.x == 0 && a.stream_out) {
#pragma unroll
    for (int q = 0; q < PIECES; ++q) {
      const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 4;
      if (i < k) *reinterpret_cast<f32x4 *>(a.stream_out + i) = v[q];
    }
  }
  float inverse = 1.0f;
  if (weight) inverse = 1.0f / sqrtf(block_sum<kWaves>(sum, scratch) / (float)k + a.epsilon);
#pragma unroll
  for (int q = 0; q < PIECES; ++q) {
    const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 4;
    if (i < k) {
      if (weight) {
        const bf16x4 own = *reinterpret_cast<const bf16x4 *>(weight + i);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[q][e] *= inverse * (a.norm_offset + (float)own[e]);
      }
      *reinterpret_cast<f32x4 *>(xs + staged_index(i, plane)) = v[q];
    }
  }
  __syncthreads();
}

// The same for any length, through the staged row.
__device__ __forceinline__ void stage_pending_any(const DenseGemvArgs &a, float *xs, uint32_t plane, float *scratch) {
  const uint32_t k = a.k;
  const float *x = static_cast<const float *>(a.x);
  float sum = 0.0f;
  for (uint32_t i = threadIdx.x; i < k; i += kWaves * 64) sum += a.pending[i] * a.pending[i];
  const float factor = a.pending_scale / sqrtf(block_sum<kWaves>(sum, scratch) / (float)k + a.epsilon);
  sum = 0.0f;
  for (uint32_t i = threadIdx.x; i < k; i += kWaves * 64) {
    const float w = a.norm_offset + (float)reinterpret_cast<const __bf16 *>(a.pending_weight)[i];
    const float v = fmaf(a.pending[i] * factor, w, x[i]);
    if (blockIdx.x == 0 && a.stream_out) a.stream_out[i] = v;
    sum += v * v;
    xs[staged_index(i, plane)] = v;
  }
  if (a.norm_weight) {
    const float inverse = 1.0f / sqrtf(block_sum<kWaves>(sum, scratch) / (float)k + a.epsilon);
    for (uint32_t i = threadIdx.x; i < k; i += kWaves * 64)
      xs[staged_index(i, plane)] *= inverse * (a.norm_offset + (float)reinterpret_cast<const __bf16 *>(a.norm_weight)[i]);
  }
  __syncthreads();
}

// How a launch stages its row.  One kernel each: a kernel's registers are those of its largest branch, and they decide
// how many loads a CU keeps in flight.
enum class Staging {
  kPlainShort,    // rows of whole pieces of eight, at most 8192 values
  kPlain,
  kNormedShort,   // one norm over a row of whole pieces of four, at most 4096 values
  kNormed,
  kPendingShort,  // the same with a pending output
  kPending,
};

inline Staging staging_of(const DenseGemvArgs &a) {
  if (a.pending) return a.k % 4 == 0 && a.k <= 4096 ? Staging::kPendingShort : Staging::kPending;
  if (a.norm_weight) return a.k % 4 == 0 && a.k <= 4096 && a.norm_groups == 1 ? Staging::kNormedShort : Staging::kNormed;
  return a.k % 8 == 0 && a.k <= 8192 ? Staging::kPlainShort : Staging::kPlain;
}

template <typename T, int PIECES, typename Ahead>
__device__ __forceinline__ void stage_plain_row(const DenseGemvArgs &a, float *xs, uint32_t plane, Ahead ahead) {
  const uint32_t k = a.k;
  f32x8 v[PIECES];
#pragma unroll
  for (int q = 0; q < PIECES; ++q) {
    const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 8;
    if (i < k)
      v[q] = a.x_is_f32 ? *reinterpret_cast<const f32x8 *>(static_cast<const float *>(a.x) + i)
                        : convert_frag<float>(*reinterpret_cast<const Frag<T> *>(static_cast<const T *>(a.x) + i));
  }
  ahead();
#pragma unroll
  for (int q = 0; q < PIECES; ++q) {
    const uint32_t i = (q * kWaves * 64 + threadIdx.x) * 8;
    if (i < k) {
      *reinterpret_cast<f32x4 *>(xs + (i >> 1)) = f32x4{v[q][0], v[q][1], v[q][2], v[q][3]};
      *reinterpret_cast<f32x4 *>(xs + plane + (i >> 1)) = f32x4{v[q][4], v[q][5], v[q][6], v[q][7]};
    }
  }
  __syncthreads();
}

// Stages the row x (f32, or the activation type where it is plain), normalised in `groups` parts by norm_weight.  `ahead`
// is called once the row has been requested (loads return in order: what it requests does not delay the row).
template <typename T, Staging STAGING, typename Ahead>
__device__ __forceinline__ void stage_activation(const DenseGemvArgs &a, float *xs, uint32_t plane, float *scratch,
                                                 Ahead ahead) {
  const uint32_t k = a.k;
  // whole pieces behind the row's end read as zeros
  for (uint32_t i = k + threadIdx.x; i < ((k + 7) & ~7u); i += kWaves * 64) xs[staged_index(i, plane)] = 0.0f;
  if (STAGING == Staging::kPlainShort) return stage_plain_row<T, 4>(a, xs, plane, ahead);
  if (STAGING == Staging::kNormedShort) return stage_normed_row<4>(a, xs, plane, scratch, ahead);
  if (STAGING == Staging::kPendingShort) return stage_pending_row<4>(a, xs, plane, scratch, ahead);
  if (STAGING == Staging::kPending) {
    if ((k & 3) == 0 && k <= 8 * 4 * kWaves * 64) return stage_pending_row<8>(a, xs, plane, scratch, ahead);
    ahead();
    return stage_pending_any(a, xs, plane, scratch);
  }
  if (STAGING == Staging::kPlain) {
    if ((k & 7) == 0 && k <= 8 * 8 * kWaves * 64) return stage_plain_row<T, 8>(a, xs, plane, ahead);
    ahead();
    for (uint32_t i = threadIdx.x; i < k; i += kWaves * 64)
      xs[staged_index(i, plane)] =
          a.x_is_f32 ? static_cast<const float *>(a.x)[i] : to_f32(static_cast<const T *>(a.x)[i]);
    __syncthreads();
    return;
  }
  if (a.norm_groups == 1 && (k & 3) == 0 && k <= 8 * 4 * kWaves * 64)
    return stage_normed_row<8>(a, xs, plane, scratch, ahead);
  ahead();
  const float *x = static_cast<const float *>(a.x);
  const __bf16 *weight = reinterpret_cast<const __bf16 *>(a.norm_weight);
  const uint32_t part = k / a.norm_groups;
  for (uint32_t g = 0; g < a.norm_groups; ++g) {
    float sum = 0.0f;
    for (uint32_t i = g * part + threadIdx.x; i < (g + 1) * part; i += kWaves * 64) sum += x[i] * x[i];
    sum = block_sum<kWaves>(sum, scratch);
    const float inverse = 1.0f / sqrtf(sum / (float)part + a.epsilon);
    for (uint32_t i = g * part + threadIdx.x; i < (g + 1) * part; i += kWaves * 64)
      xs[staged_index(i, plane)] = x[i] * inverse * (a.norm_offset + (float)weight[i]);
  }
  __syncthreads();
}

// ROWS weight rows streamed against the staged activation in blocks of STEPS * 512 columns; the first block
// is requested by `request`, ahead of the staging where the rows are known by then.
template <int ROWS, bool VEC, int STEPS = 4>
struct RowStream {
  const __bf16 *rows[ROWS];
  bf16x8 w[STEPS][ROWS];
  float sums[ROWS];

  __device__ __forceinline__ void fetch(uint32_t k0, uint32_t k, int lane) {
#pragma unroll
    for (int s = 0; s < STEPS; ++s) {
      const uint32_t kk = k0 + s * 512 + lane * 8;
#pragma unroll
      for (int r = 0; r < ROWS; ++r) w[s][r] = load_piece(rows[r] + kk, (int)k - (int)kk, VEC);
    }
  }
  __device__ __forceinline__ void request(uint32_t k, int lane) { fetch(0, k, lane); }

  // every lane ends with every sum
  __device__ __forceinline__ void run(const float *xs, uint32_t plane, uint32_t k, int lane) {
#pragma unroll
    for (int r = 0; r < ROWS; ++r) sums[r] = 0.0f;
    for (uint32_t k0 = 0; k0 < k; k0 += 512 * STEPS) {
      if (k0 > 0) fetch(k0, k, lane);
#pragma unroll
      for (int s = 0; s < STEPS; ++s) {
        const uint32_t kk = k0 + s * 512 + lane * 8;
        if (kk >= k) continue;
        const f32x4 lo = *reinterpret_cast<const f32x4 *>(xs + (kk >> 1));
        const f32x4 hi = *reinterpret_cast<const f32x4 *>(xs + plane + (kk >> 1));
#pragma unroll
        for (int r = 0; r < ROWS; ++r) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            sums[r] = fmaf((float)w[s][r][e], lo[e], sums[r]);
            sums[r] = fmaf((float)w[s][r][4 + e], hi[e], sums[r]);
          }
        }
      }
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) sums[r] = wave_sum(sums[r]);
  }
};

template <typename T>
__device__ __forceinline__ void cache_store(const DenseGemvArgs &a, uint32_t n, float v) {
  const uint32_t position = a.state[kStatePosition], slot = a.state[kStateSlot];
  const uint32_t ring = position % a.cache.capacity;
  if (n < a.n_q + a.n_k) {
    const uint32_t c = n - a.n_q, head = c / a.dim;
    static_cast<T *>(a.cache.keys)[(((size_t)slot * a.kv_heads + head) * a.cache.capacity + ring) * a.dim + c % a.dim] = (T)v;
    return;
  }
  const uint32_t c = n - a.n_q - a.n_k, head = c / a.vdim;
  if (a.mix.mode == 1) a.mix.v_first[c] = v;
  if (a.mix.mode == 2) v = (1.0f - a.mix.lambda) * v + a.mix.lambda * a.mix.v_first[c];
  static_cast<T *>(a.cache.values)[(((size_t)slot * a.kv_heads + head) * a.cache.capacity + ring) * a.vdim + c % a.vdim] = (T)v;
}

__device__ __forceinline__ float bf16_at(const uint16_t *p, size_t i) {
  return (float)reinterpret_cast<const __bf16 *>(p)[i];
}

// Channel c's input v of the short convolution into its ring; the output behind silu.
__device__ __forceinline__ float conv_step(const DenseGemvArgs &a, uint32_t c, float v) {
  const uint32_t position = a.state[kStatePosition], slot = a.state[kStateSlot];
  float *ring = a.conv_state + (size_t)slot * a.taps * a.channels + c;
  float sum = (a.conv_bias ? bf16_at(a.conv_bias, c) : 0.0f) + bf16_at(a.conv, (size_t)c * a.taps + a.taps - 1) * v;
  for (uint32_t back = 1; back < a.taps; ++back)
    if (back <= position)
      sum = fmaf(bf16_at(a.conv, (size_t)c * a.taps + a.taps - 1 - back),
                 ring[(size_t)((position - back) % a.taps) * a.channels], sum);
  ring[(size_t)(position % a.taps) * a.channels] = v;
  return silu_f32(sum);
}

// Row n of the recurrent layer's input projection.
__device__ __forceinline__ void ssm_in_store(const DenseGemvArgs &a, uint32_t n, float v) {
  if (n >= a.inner && n < a.inner + a.channels) {
    v = conv_step(a, n - a.inner, v);
  } else if (n >= a.inner + a.channels) {
    v = softplus_f32(v + bf16_at(a.dt_bias, n - a.inner - a.channels));
  }
  a.out_f32[n] = v;
}

template <typename T>
__device__ __forceinline__ void gemv_epilogue(const DenseGemvArgs &a, uint32_t n, float v, float up) {
  switch (a.epilogue) {
    case GemvEpilogue::kStore: static_cast<T *>(a.out)[n] = (T)v; return;
    case GemvEpilogue::kStoreF32: a.out_f32[n] = soft_capped(v, a.softcap); return;
    case GemvEpilogue::kAdd: a.out_f32[n] += v; return;
    case GemvEpilogue::kGated: a.out_f32[n] = gated_value(v, up, a.activation, a.limit); return;
    case GemvEpilogue::kQkv:
      if (n < a.n_q) static_cast<T *>(a.out)[n] = (T)v;
      else cache_store<T>(a, n, v);
      return;
    case GemvEpilogue::kSsmIn: ssm_in_store(a, n, v); return;
    case GemvEpilogue::kConvIn:
      a.out_f32[n] = n >= a.inner && n < a.inner + a.channels ? conv_step(a, n - a.inner, v) : v;
      return;
  }
}

template <typename T, int ROWS, bool GATED, bool VEC, Staging STAGING>
__global__ __launch_bounds__(256) void dense_gemv_kernel(DenseGemvArgs a) {
  extern __shared__ __attribute__((aligned(16))) float xs[];
  __shared__ float scratch[kWaves];
  const uint32_t plane = ((a.k + 7) >> 3) << 2;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  constexpr int OUTPUTS = GATED ? ROWS / 2 : ROWS;
  const uint32_t first = (blockIdx.x * kWaves + wave) * OUTPUTS;
  RowStream<ROWS, VEC> stream;
#pragma unroll
  for (int r = 0; r < ROWS; ++r) {
    const uint16_t *matrix = GATED && (r & 1) ? a.w_up : a.w;
    const uint32_t n = min(first + (GATED ? r / 2 : r), a.n - 1);
    stream.rows[r] = reinterpret_cast<const __bf16 *>(matrix) + (size_t)n * a.k;
  }
  stage_activation<T, STAGING>(a, xs, plane, scratch, [&] { stream.request(a.k, lane); });
  if (first >= a.n) return;
  stream.run(xs, plane, a.k, lane);
  const float(&sums)[ROWS] = stream.sums;
  float mine = 0.0f, up = 0.0f;
#pragma unroll
  for (int o = 0; o < OUTPUTS; ++o)
    if (lane == o) {
      mine = sums[GATED ? 2 * o : o];
      if (GATED) up = sums[2 * o + 1];
    }
  if (lane < OUTPUTS && first + lane < a.n) gemv_epilogue<T>(a, first + lane, mine, up);
}

template <typename T, int ROWS, bool GATED, bool VEC, Staging STAGING>
hipError_t run_staged(const DenseGemvArgs &a, hipStream_t stream) {
  static bool allowed[kMaxDevices] = {};
  const auto kernel = dense_gemv_kernel<T, ROWS, GATED, VEC, STAGING>;
  const uint32_t bytes = ((a.k + 7) / 8) * 32;
  if (bytes > 48 * 1024)
    if (hipError_t status = allow_dynamic_lds(reinterpret_cast<const void *>(kernel), kGemvMaxK * 4, allowed)) return status;
  const uint32_t per = kWaves * (GATED ? ROWS / 2 : ROWS);
  kernel<<<(a.n + per - 1) / per, 256, bytes, stream>>>(a);
  return hipGetLastError();
}

template <typename T, int ROWS, bool GATED, bool VEC>
hipError_t run_gemv(const DenseGemvArgs &a, hipStream_t stream) {
  switch (staging_of(a)) {
    case Staging::kPlainShort: return run_staged<T, ROWS, GATED, VEC, Staging::kPlainShort>(a, stream);
    case Staging::kPlain: return run_staged<T, ROWS, GATED, VEC, Staging::kPlain>(a, stream);
    case Staging::kNormedShort: return run_staged<T, ROWS, GATED, VEC, Staging::kNormedShort>(a, stream);
    case Staging::kNormed: return run_staged<T, ROWS, GATED, VEC, Staging::kNormed>(a, stream);
    case Staging::kPendingShort: return run_staged<T, ROWS, GATED, VEC, Staging::kPendingShort>(a, stream);
    case Staging::kPending: return run_staged<T, ROWS, GATED, VEC, Staging::kPending>(a, stream);
  }
  return hipErrorInvalidValue;
}

template <typename T>
hipError_t pick_gemv(const DenseGemvArgs &a, hipStream_t stream) {
  const bool vec = a.k % 8 == 0, gated = a.epilogue == GemvEpilogue::kGated;
  if (gated) {
    if (!vec) return run_gemv<T, 2, true, false>(a, stream);
    if (a.n <= 2048) return run_gemv<T, 2, true, true>(a, stream);
    return run_gemv<T, 4, true, true>(a, stream);
  }
  if (!vec) return run_gemv<T, 1, false, false>(a, stream);
  if (a.n <= 2048) return run_gemv<T, 1, false, true>(a, stream);
  if (a.n <= 8192) return run_gemv<T, 2, false, true>(a, stream);
  return run_gemv<T, 4, false, true>(a, stream);
}

// ---- routed experts, one token ----------------------------------------------------------------------

// Rank of every expert among the logits (ties to the lower index): ids / weights of the `top` best.
// Called by a whole workgroup of THREADS threads; logits may be in global memory.
template <int THREADS>
__device__ __forceinline__ void select_experts(const float *logits, uint32_t experts, uint32_t top, float *z,
                                               uint32_t *ids, float *weights) {
  for (uint32_t e = threadIdx.x; e < experts; e += THREADS) z[e] = logits[e];
  __syncthreads();
  for (uint32_t e = threadIdx.x; e < experts; e += THREADS) {
    const float mine = z[e];
    uint32_t rank = 0;
    for (uint32_t other = 0; other < experts; ++other) rank += z[other] > mine || (z[other] == mine && other < e);
    if (rank < top) {
      ids[rank] = e;
      weights[rank] = mine;
    }
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    const float best = weights[0];
    float total = 0.0f;
    for (uint32_t s = 0; s < top; ++s) {
      weights[s] = __expf(weights[s] - best);
      total += weights[s];
    }
    for (uint32_t s = 0; s < top; ++s) weights[s] /= total;
  }
  __syncthreads();
}

// blockIdx.y: choice 0 .. top - 1, or `top`: the shared expert.  A wave owns kUpOutputs hidden values.
constexpr int kUpOutputs = 4, kUpSteps = 2;

template <bool VEC, Staging STAGING>
__global__ __launch_bounds__(256) void moe_gemv_up_kernel(MoeGemvArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float scratch[kWaves];
  const uint32_t plane = ((a.width + 7) >> 3) << 2;
  float *xs = lds, *z = lds + 2 * plane, *weights = z + a.experts;
  uint32_t *ids = reinterpret_cast<uint32_t *>(weights + a.top);
  const bool shared = blockIdx.y == a.top;
  const uint32_t n_total = shared ? a.shared_ff : a.ff;
  if (blockIdx.x * kWaves * kUpOutputs >= n_total) return;
  DenseGemvArgs in = {};
  in.x = a.x;
  in.norm_weight = a.norm_weight;
  in.norm_groups = 1;
  in.epsilon = a.epsilon;
  in.k = a.width;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const uint32_t first = (blockIdx.x * kWaves + wave) * kUpOutputs;
  RowStream<2 * kUpOutputs, VEC, kUpSteps> stream;
  // the choice is made, and its weights are requested, while the activation is on its way to LDS
  stage_activation<float, STAGING>(in, xs, plane, scratch, [&] {
    uint32_t expert = 0;
    if (!shared) {
      select_experts<256>(a.logits, a.experts, a.top, z, ids, weights);
      expert = ids[blockIdx.y];
    }
    const uint16_t *gate = shared ? a.shared_gate : a.gate + (size_t)expert * a.ff * a.width;
    const uint16_t *up = shared ? a.shared_up : a.up + (size_t)expert * a.ff * a.width;
#pragma unroll
    for (int r = 0; r < 2 * kUpOutputs; ++r)
      stream.rows[r] =
          reinterpret_cast<const __bf16 *>((r & 1) ? up : gate) + (size_t)min(first + r / 2, n_total - 1) * a.width;
    stream.request(a.width, lane);
  });
  if (first >= n_total) return;
  stream.run(xs, plane, a.width, lane);
  float g = 0.0f, u = 0.0f;
#pragma unroll
  for (int o = 0; o < kUpOutputs; ++o)
    if (lane == o) {
      g = stream.sums[2 * o];
      u = stream.sums[2 * o + 1];
    }
  if (lane < kUpOutputs && first + lane < n_total)
    a.hidden[(size_t)blockIdx.y * a.ff + first + lane] = gate_activation(g, a.activation) * u;
}

// stream[n] += sum_s weight_s down[expert_s][n] . hidden_s (+ sigmoid(gate) shared_down[n] . hidden_shared).
// A workgroup owns ROWS columns of the stream; its waves take the choices in pieces of 1024 in turn.
constexpr int kDownWaves = 8;

template <int ROWS, bool VEC>
__global__ __launch_bounds__(kDownWaves * 64) void moe_gemv_down_kernel(MoeGemvArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  __shared__ float partial[kDownWaves][ROWS];
  float *z = lds, *weights = z + a.experts;
  uint32_t *ids = reinterpret_cast<uint32_t *>(weights + a.top);
  select_experts<kDownWaves * 64>(a.logits, a.experts, a.top, z, ids, weights);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const uint32_t first = blockIdx.x * ROWS;
  float acc[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r) acc[r] = 0.0f;
  const uint32_t per = (a.ff + 1023) / 1024, units = a.top * per + (a.shared_ff + 1023) / 1024;
  for (uint32_t unit = wave; unit < units; unit += kDownWaves) {
    const uint32_t s = min(unit / per, a.top);
    const bool shared = s == a.top;
    const uint32_t k = shared ? a.shared_ff : a.ff, k0 = (unit - s * per) * 1024;
    const __bf16 *down = reinterpret_cast<const __bf16 *>(shared ? a.shared_down : a.down + (size_t)ids[s] * a.width * a.ff);
    const float weight = shared ? sigmoid_f32(a.logits[a.experts]) : weights[s];
    const float *hidden = a.hidden + (size_t)s * a.ff;
    f32x8 h[2];
    bf16x8 w[2][ROWS];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const uint32_t kk = k0 + i * 512 + lane * 8;
      const int count = (int)k - (int)kk;
      h[i] = load_piece(hidden + kk, count, VEC);
#pragma unroll
      for (int r = 0; r < ROWS; ++r)
        w[i][r] = load_piece(down + (size_t)min(first + r, a.width - 1) * k + kk, count, VEC);
    }
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      float sum = 0.0f;
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int e = 0; e < 8; ++e) sum = fmaf((float)w[i][r][e], h[i][e], sum);
      acc[r] = fmaf(weight, sum, acc[r]);
    }
  }
#pragma unroll
  for (int r = 0; r < ROWS; ++r) acc[r] = wave_sum(acc[r]);
  if (lane == 0)
#pragma unroll
    for (int r = 0; r < ROWS; ++r) partial[wave][r] = acc[r];
  __syncthreads();
  if (threadIdx.x < ROWS && first + threadIdx.x < a.width) {
    float total = 0.0f;
#pragma unroll
    for (int w = 0; w < kDownWaves; ++w) total += partial[w][threadIdx.x];
    a.stream[first + threadIdx.x] += total;
  }
}

}  // namespace

bool dense_gemv_ok(const DenseGemvArgs &a) { return a.k <= kGemvMaxK; }

hipError_t launch_dense_gemv(const DenseGemvArgs &a, hipStream_t stream) {
  return a.f32 ? pick_gemv<float>(a, stream) : pick_gemv<__bf16>(a, stream);
}

hipError_t launch_moe_gemv_up(const MoeGemvArgs &a, hipStream_t stream) {
  const uint32_t bytes = ((a.width + 7) / 8) * 32 + (a.experts + 2 * a.top) * 4;
  if (bytes > 60 * 1024) return hipErrorInvalidValue;
  const uint32_t widest = std::max(a.ff, a.shared_ff);
  const dim3 grid((widest + kUpOutputs * kWaves - 1) / (kUpOutputs * kWaves), a.top + (a.shared_ff ? 1 : 0));
  const bool small = a.width % 4 == 0 && a.width <= 4096;
  if (a.width % 8 != 0) moe_gemv_up_kernel<false, Staging::kNormed><<<grid, 256, bytes, stream>>>(a);
  else if (small) moe_gemv_up_kernel<true, Staging::kNormedShort><<<grid, 256, bytes, stream>>>(a);
  else moe_gemv_up_kernel<true, Staging::kNormed><<<grid, 256, bytes, stream>>>(a);
  return hipGetLastError();
}

hipError_t launch_moe_gemv_down(const MoeGemvArgs &a, hipStream_t stream) {
  const uint32_t bytes = (a.experts + 2 * a.top) * 4;
  const bool vec = a.ff % 8 == 0 && a.shared_ff % 8 == 0;
  constexpr int ROWS = 8;
  const uint32_t grid = (a.width + ROWS - 1) / ROWS;
  if (vec) moe_gemv_down_kernel<ROWS, true><<<grid, kDownWaves * 64, bytes, stream>>>(a);
  else moe_gemv_down_kernel<ROWS, false><<<grid, kDownWaves * 64, bytes, stream>>>(a);
  return hipGetLastError();
}

}  // namespace llmopt
