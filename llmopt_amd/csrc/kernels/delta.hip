// The gated delta rule with a decay per head and key channel.
//
//   S <- diag(g_t) S,   u_t = beta_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t
//
// (per head, S [dim][vdim] in float32, q and k of unit length), and behind it the norm of every head's output
// and its gate.
//
// One token (delta_step_kernel): a workgroup per head.  The low-rank products for decay and gate, the unit
// norms, the state's pass through registers, the output's norm and gate are one launch.
//
// Many tokens: chunks of 64.  With L_t the running sum of log g per channel from the chunk's start and S the
// incoming state,
//   N_ij = beta_i sum_c k_ic k_jc exp(L_ic - L_jc)   (j < i)       (I + N) U = beta (V - (K exp L) S)
//   A_ij = sum_c q_ic k_jc exp(L_ic - L_jc)          (j <= i)      O = (Q exp L) S + A U
//   S <- diag(exp L_end) S + (K exp(L_end - L))^T U
//  * delta_keys_kernel: convolution, silu and unit length of queries and keys;
//  * delta_chunk_kernel, a workgroup per chunk and head: all that does not need the state - A, the triangular
//    solves W = (I + N)^-1 beta K exp L and V' = (I + N)^-1 beta V (then U = V' - W S), and the decayed
//    operands.  The exponents are never split around a distant reference: between sub-blocks of 16 tokens the
//    reference is the later block's start (both factors at most 1), inside one the difference itself is taken;
//  * delta_state_kernel: the serial part, from chunk to chunk, the state in matrix-core accumulators;
//  * delta_output_kernel: the outputs of all chunks at once, with their norm and gate.
// Everything but the convolution's inputs and v keeps float32 accuracy: operands enter the bfloat16 matrix
// cores as a high and a low part.  Position 0 starts from a zero state and zero history.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr int Q = (int)kDeltaChunk, kBlock = 16;
constexpr int kSlice = 64, kSliceStride = kSlice + 4;  // channels of a pass through LDS
constexpr int kKeyTokens = 8;
constexpr float kUnitEpsilon = 1e-6f;

__device__ __forceinline__ float bf16_at(const uint16_t *p, size_t i) {
  return (float)reinterpret_cast<const __bf16 *>(p)[i];
}

// Operands of float32 accuracy in memory: float as it is, bf16 as a plane of high and one of low parts.
template <typename T>
constexpr int kPlanes = sizeof(T) == 4 ? 1 : 2;

template <typename T>
__device__ __forceinline__ WideFrag<T> load_wide(const T *p, size_t plane);
template <>
__device__ __forceinline__ WideFrag<float> load_wide<float>(const float *p, size_t) {
  return {*reinterpret_cast<const f32x8 *>(p)};
}
template <>
__device__ __forceinline__ WideFrag<__bf16> load_wide<__bf16>(const __bf16 *p, size_t plane) {
  return {*reinterpret_cast<const bf16x8 *>(p), *reinterpret_cast<const bf16x8 *>(p + plane)};
}
template <typename T, int N>
__device__ __forceinline__ void store_wide(T *p, size_t plane, const float (&v)[N]) {
  typedef T xn __attribute__((ext_vector_type(N)));
  xn high, low;
#pragma unroll
  for (int i = 0; i < N; ++i) {
    high[i] = (T)v[i];
    low[i] = (T)(v[i] - (float)high[i]);
  }
  *reinterpret_cast<xn *>(p) = high;
  if (kPlanes<T> == 2) *reinterpret_cast<xn *>(p + plane) = low;
}
template <typename T>
__device__ __forceinline__ void store_wide_one(T *p, size_t plane, float v) {
  const T high = (T)v;
  *p = high;
  if (kPlanes<T> == 2) p[plane] = (T)(v - (float)high);
}

// Per chunk and head, np: dim to a multiple of 32, ep: vdim to a multiple of 16.
struct DeltaWorkspace {
  float *queries, *keys;  // [m][kv_heads][dim]
  void *w, *qd;           // wide [chunks][heads][planes][Q][np]: W, Q exp L
  void *kt;               // wide [chunks][heads][planes][np][Q]: (K exp(L_end - L))^T
  float *solved;          // [chunks][heads][ep][Q]: V'^T
  float *kd;              // [chunks][heads][Q][np]: K exp L
  float *end;             // [chunks][heads][np]: exp L_end
  float *scores;          // [chunks][heads][Q][Q]: A
  void *u;                // wide [chunks][heads][planes][ep][Q]: U^T
  void *states;           // wide [chunks][heads][planes][ep][np] in operand order: every chunk's incoming state
  uint32_t chunks, channels, np, ep;
  size_t bytes;
};

DeltaWorkspace layout(const DeltaArgs &a) {
  DeltaWorkspace w = {};
  w.chunks = (a.m + Q - 1) / Q;
  w.channels = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
  w.np = (a.dim + 31) / 32 * 32;
  w.ep = (a.vdim + 15) / 16 * 16;
  uint8_t *base = static_cast<uint8_t *>(a.workspace);
  size_t at = 0;
  auto take = [&](size_t values) {
    void *p = base ? base + at : nullptr;
    at += (values * 4 + 255) & ~(size_t)255;
    return p;
  };
  const size_t keys = (size_t)a.m * a.kv_heads * a.dim, each = (size_t)w.chunks * a.heads;
  w.queries = static_cast<float *>(take(keys));
  w.keys = static_cast<float *>(take(keys));
  w.w = take(each * Q * w.np);
  w.qd = take(each * Q * w.np);
  w.kt = take(each * Q * w.np);
  w.solved = static_cast<float *>(take(each * Q * w.ep));
  w.kd = static_cast<float *>(take(each * Q * w.np));
  w.end = static_cast<float *>(take(each * w.np));
  w.scores = static_cast<float *>(take(each * Q * Q));
  w.u = take(each * Q * w.ep);
  w.states = take(each * w.ep * w.np);
  w.bytes = at;
  return w;
}

// ---- one token ---------------------------------------------------------------------------------------

constexpr int kStepThreads = 512;

// A thread owns VEC columns of the state and every `groups`-th row, R of them in registers (R == 0: any number,
// read twice).
template <int VEC, int R>
__global__ __launch_bounds__(kStepThreads) void delta_step_kernel(DeltaArgs a) {
  typedef float vec __attribute__((ext_vector_type(VEC)));
  extern __shared__ float ranks[];  // decay_in, gate_in
  __shared__ float key[kDeltaMaxWidth], query[kDeltaMaxWidth], decay[kDeltaMaxWidth], gate[kDeltaMaxWidth];
  __shared__ __attribute__((aligned(16))) float written[kDeltaMaxWidth], partial[2][kStepThreads * VEC];
  __shared__ float sums[8], product;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const uint32_t head = blockIdx.x, group = head / (a.heads / a.kv_heads);
  const uint32_t columns = a.vdim / VEC, groups = kStepThreads / columns;
  const uint32_t column = tid % columns * VEC, first = tid / columns;
  const bool fresh = a.step[kStatePosition] == 0;
  float *state = a.state + ((size_t)a.step[kStateSlot] * a.heads + head) * a.dim * a.vdim;

  vec s[R > 0 ? R : 1];
  auto row_at = [&](int i) { return first + groups * i; };
  const bool owner = first < groups;
  if (R > 0) {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const uint32_t r = row_at(i);
      s[i] = 0.0f;
      if (owner && !fresh && r < a.dim) s[i] = *reinterpret_cast<const vec *>(state + (size_t)r * a.vdim + column);
    }
  }
  for (uint32_t i = tid; i < a.decay_rank + a.gate_rank; i += kStepThreads)
    ranks[i] = i < a.decay_rank ? a.decay_in[i] : a.gate_in[i - a.decay_rank];
  const float rate = expf(bf16_at(a.a_log, head)), beta = sigmoid_f32(a.row_beta[head]);

  // unit lengths: wave 0 the query, wave 1 the key
  if (wave < 2) {
    const float *source = a.row + (size_t)(wave == 0 ? 0 : a.kv_heads * a.dim) + (size_t)group * a.dim;
    float *target = wave == 0 ? query : key, v[kDeltaMaxWidth / 64], sum = 0.0f;
#pragma unroll
    for (int i = 0; i < (int)kDeltaMaxWidth / 64; ++i) {
      v[i] = lane + 64 * i < a.dim ? source[lane + 64 * i] : 0.0f;
      sum += v[i] * v[i];
    }
    float scale = 1.0f / sqrtf(wave_sum(sum) + kUnitEpsilon);
    if (wave == 0) scale /= sqrtf((float)a.dim);
#pragma unroll
    for (int i = 0; i < (int)kDeltaMaxWidth / 64; ++i)
      if (lane + 64 * i < a.dim) target[lane + 64 * i] = v[i] * scale;
  }
  __syncthreads();
  if (wave == 0) {
    float sum = 0.0f;
    for (uint32_t c = lane; c < a.dim; c += 64) sum += key[c] * query[c];
    sum = wave_sum(sum);
    if (lane == 0) product = sum;
  }
  // decay and gate: sixteen lanes a row of the low-rank products
  const int part = tid & 15;
  for (uint32_t r = tid >> 4; r < a.dim + a.vdim; r += kStepThreads / 16) {
    const bool is_decay = r < a.dim;
    const uint32_t rank = is_decay ? a.decay_rank : a.gate_rank;
    const uint32_t n = is_decay ? head * a.dim + r : head * a.vdim + (r - a.dim);
    const __bf16 *w = reinterpret_cast<const __bf16 *>(is_decay ? a.w_decay : a.w_gate) + (size_t)n * rank;
    const float *x = is_decay ? ranks : ranks + a.decay_rank;
    float sum = 0.0f;
    for (uint32_t k = part * 8; k < rank; k += 128) {
      const bf16x8 piece = load_piece(w + k, (int)rank - (int)k, rank % 8 == 0);
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (k + e < rank) sum = fmaf((float)piece[e], x[k + e], sum);
    }
#pragma unroll
    for (int mask = 8; mask >= 1; mask >>= 1) sum += __shfl_xor(sum, mask, 64);
    if (part == 0) {
      if (is_decay) decay[r] = expf(-rate * softplus_f32(sum + bf16_at(a.dt_bias, n)));
      else gate[r - a.dim] = sigmoid_f32(sum);
    }
  }
  __syncthreads();

  vec from_key = 0.0f, from_query = 0.0f;
  if (owner) {
    if (R > 0) {
#pragma unroll
      for (int i = 0; i < R; ++i) {
        const uint32_t r = row_at(i);
        if (r >= a.dim) continue;
        s[i] *= decay[r];
        from_key += s[i] * key[r];
        from_query += s[i] * query[r];
      }
    } else if (!fresh) {
      for (uint32_t r = first; r < a.dim; r += groups) {
        const vec one = *reinterpret_cast<const vec *>(state + (size_t)r * a.vdim + column) * decay[r];
        from_key += one * key[r];
        from_query += one * query[r];
      }
    }
    *reinterpret_cast<vec *>(&partial[0][first * a.vdim + column]) = from_key;
    *reinterpret_cast<vec *>(&partial[1][first * a.vdim + column]) = from_query;
  }
  __syncthreads();
  float out = 0.0f;
  if (tid < (int)a.vdim) {
    float read = 0.0f;
    for (uint32_t g = 0; g < groups; ++g) {
      read += partial[0][g * a.vdim + tid];
      out += partial[1][g * a.vdim + tid];
    }
    const float v = a.row[2 * (size_t)a.kv_heads * a.dim + (size_t)head * a.vdim + tid];
    const float u = beta * (v - read);
    written[tid] = u;
    out = fmaf(product, u, out);
  }
  const float square = wave_sum(out * out);
  if (lane == 0) sums[wave] = square;
  __syncthreads();
  if (tid < (int)a.vdim) {
    float total = 0.0f;
#pragma unroll
    for (int i = 0; i < kStepThreads / 64; ++i) total += sums[i];
    const float inverse = 1.0f / sqrtf(total / (float)a.vdim + a.epsilon);
    a.out_row[(size_t)head * a.vdim + tid] = out * inverse * bf16_at(a.norm, tid) * gate[tid] * a.out_scale;
  }
  if (!owner) return;
  const vec u = *reinterpret_cast<const vec *>(&written[column]);
  if (R > 0) {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const uint32_t r = row_at(i);
      if (r < a.dim) *reinterpret_cast<vec *>(state + (size_t)r * a.vdim + column) = s[i] + key[r] * u;
    }
  } else {
    for (uint32_t r = first; r < a.dim; r += groups) {
      vec *p = reinterpret_cast<vec *>(state + (size_t)r * a.vdim + column);
      *p = (fresh ? vec(0.0f) : *p * decay[r]) + key[r] * u;
    }
  }
}

// ---- many tokens ----------------------------------------------------------------------------------------

// The input of channel `channel` at token t of the step (negative: before it).
template <typename T>
struct ConvInput {
  const T *input;
  const float *ring;
  uint32_t m, ld, taps, channels, position;
  __device__ __forceinline__ ConvInput(const DeltaArgs &a, uint32_t channels_, uint32_t channel)
      : input(static_cast<const T *>(a.projected) + channel), m(a.m), ld(a.ld), taps(a.taps), channels(channels_),
        position(a.step[kStatePosition]) {
    ring = a.conv_state + (size_t)a.step[kStateSlot] * taps * channels + channel;
  }
  __device__ __forceinline__ float at(int t) const {
    if (t >= 0) return t < (int)m ? to_f32(input[(size_t)t * ld]) : 0.0f;
    return (int64_t)position + t >= 0 ? ring[(size_t)((position + t) % taps) * channels] : 0.0f;
  }
};

// COUNT consecutive outputs of the convolution from token t0 on, behind silu.  TAPS: its length (0: any).
template <typename T, int TAPS, int COUNT>
__device__ __forceinline__ void conv_tokens(const DeltaArgs &a, uint32_t channels, uint32_t channel, int t0,
                                            float (&out)[COUNT]) {
  const ConvInput<T> input(a, channels, channel);
  if (TAPS > 0) {
    constexpr int BEFORE = TAPS > 0 ? TAPS - 1 : 0;
    float window[COUNT + BEFORE];
#pragma unroll
    for (int i = 0; i < COUNT + BEFORE; ++i) window[i] = input.at(t0 + i - BEFORE);
#pragma unroll
    for (int i = 0; i < COUNT; ++i) out[i] = 0.0f;
#pragma unroll
    for (int tap = 0; tap < TAPS; ++tap) {
      const float weight = bf16_at(a.conv, (size_t)channel * TAPS + tap);
#pragma unroll
      for (int i = 0; i < COUNT; ++i) out[i] = fmaf(weight, window[i + tap], out[i]);
    }
  } else {
#pragma unroll
    for (int i = 0; i < COUNT; ++i) out[i] = 0.0f;
    for (uint32_t tap = 0; tap < a.taps; ++tap) {
      const float weight = bf16_at(a.conv, (size_t)channel * a.taps + tap);
#pragma unroll
      for (int i = 0; i < COUNT; ++i) out[i] = fmaf(weight, input.at(t0 + i - (int)(a.taps - 1 - tap)), out[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < COUNT; ++i) out[i] = silu_f32(out[i]);
}

// A wave: kKeyTokens tokens of one head's query (blockIdx.z 0) or key (1), lane l its channels l + 64 i.
template <typename T, int PARTS, int TAPS>
__global__ __launch_bounds__(256) void delta_keys_kernel(DeltaArgs a, DeltaWorkspace w) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const uint32_t t0 = (blockIdx.x * 4 + wave) * kKeyTokens, group = blockIdx.y, which = blockIdx.z;
  if (t0 >= a.m) return;
  float v[PARTS][kKeyTokens], sum[kKeyTokens];
#pragma unroll
  for (int t = 0; t < kKeyTokens; ++t) sum[t] = 0.0f;
#pragma unroll
  for (int i = 0; i < PARTS; ++i) {
    const uint32_t c = lane + 64 * i;
    if (c >= a.dim) continue;
    conv_tokens<T, TAPS>(a, w.channels, (which * a.kv_heads + group) * a.dim + c, (int)t0, v[i]);
#pragma unroll
    for (int t = 0; t < kKeyTokens; ++t) sum[t] = fmaf(v[i][t], v[i][t], sum[t]);
  }
  float *out = which == 0 ? w.queries : w.keys;
#pragma unroll
  for (int t = 0; t < kKeyTokens; ++t) {
    float scale = 1.0f / sqrtf(wave_sum(sum[t]) + kUnitEpsilon);
    if (which == 0) scale /= sqrtf((float)a.dim);
    if (t0 + t >= a.m) continue;
#pragma unroll
    for (int i = 0; i < PARTS; ++i)
      if (lane + 64 * i < a.dim) out[((size_t)(t0 + t) * a.kv_heads + group) * a.dim + lane + 64 * i] = v[i][t] * scale;
  }
}

template <typename T, int TAPS>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaArgs a, DeltaWorkspace w) {
  __shared__ __attribute__((aligned(16))) float lds_k[Q * kSliceStride], lds_q[Q * kSliceStride], lds_l[Q * kSliceStride];
  __shared__ float lds_total[4][kSlice], lds_beta[Q];
  float *lds_n = lds_k;  // N, once the slices are done
  const uint32_t chunk = blockIdx.x, head = blockIdx.y, group = head / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, column = lane & 15, quad = lane >> 4;
  const size_t each = (size_t)chunk * a.heads + head;
  const uint32_t np = w.np, t_first = chunk * Q;
  const size_t plane = (size_t)Q * np;
  T *qd = static_cast<T *>(w.qd) + each * kPlanes<T> * plane, *kt = static_cast<T *>(w.kt) + each * kPlanes<T> * plane;
  T *w_out = static_cast<T *>(w.w) + each * kPlanes<T> * plane;
  float *kd = w.kd + each * plane;
  const float rate = expf(bf16_at(a.a_log, head));
  if (tid < Q) lds_beta[tid] = t_first + tid < a.m ? sigmoid_f32(a.beta[(size_t)(t_first + tid) * a.heads + head]) : 0.0f;

  f32x4 acc_k[3], acc_q[3];
  float own_k[4], own_q[4];
#pragma unroll
  for (int j = 0; j < 3; ++j) acc_k[j] = acc_q[j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
  for (int r = 0; r < 4; ++r) own_k[r] = own_q[r] = 0.0f;

  for (uint32_t s0 = 0; s0 < np; s0 += kSlice) {
    if (s0 > 0) __syncthreads();
    // thread: channel c, the sixteen tokens of block `wave`
    const uint32_t c = s0 + lane;
    float log_decay[kBlock], k[kBlock], q[kBlock];
    const float bias = c < a.dim ? bf16_at(a.dt_bias, (size_t)head * a.dim + c) : 0.0f;
#pragma unroll
    for (int i = 0; i < kBlock; ++i) {
      const uint32_t t = t_first + wave * kBlock + i;
      const bool real = t < a.m && c < a.dim;
      log_decay[i] = real ? a.decay[(size_t)t * a.heads * a.dim + (size_t)head * a.dim + c] : 0.0f;
      k[i] = real ? w.keys[((size_t)t * a.kv_heads + group) * a.dim + c] : 0.0f;
      q[i] = real ? w.queries[((size_t)t * a.kv_heads + group) * a.dim + c] : 0.0f;
    }
    float prefix[kBlock], running = 0.0f;
#pragma unroll
    for (int i = 0; i < kBlock; ++i) {
      const bool real = t_first + wave * kBlock + i < a.m && c < a.dim;
      log_decay[i] = real ? -rate * softplus_f32(log_decay[i] + bias) : 0.0f;
      running += log_decay[i];
      prefix[i] = running;
      const int at = (wave * kBlock + i) * kSliceStride + lane;
      lds_k[at] = k[i];
      lds_q[at] = q[i];
      lds_l[at] = running;
    }
    lds_total[wave][lane] = running;
    __syncthreads();
    if (c < np) {
      float before = 0.0f, after = 0.0f;
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        if (b < wave) before += lds_total[b][lane];
        if (b > wave) after += lds_total[b][lane];
      }
      float behind[kBlock];
#pragma unroll
      for (int i = kBlock - 1; i >= 0; --i) {
        behind[i] = k[i] * __expf(after);
        after += log_decay[i];
      }
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        float eight[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) eight[e] = behind[half * 8 + e];
        store_wide<T>(kt + (size_t)c * Q + wave * kBlock + half * 8, plane, eight);
      }
#pragma unroll
      for (int i = 0; i < kBlock; ++i) {
        const float from_start = __expf(before + prefix[i]);
        const size_t at = (size_t)(wave * kBlock + i) * np + c;
        store_wide_one<T>(qd + at, plane, q[i] * from_start);
        kd[at] = k[i] * from_start;
      }
      if (wave == 3) w.end[each * np + c] = __expf(before + running);
    }

    // products with the blocks before this wave's one
    const int row = (wave * kBlock + column) * kSliceStride;
#pragma unroll
    for (int step = 0; step < kSlice / 32; ++step) {
      if (s0 + step * 32 >= np) continue;
      const int at = step * 32 + quad * 8;
      WideFrag<T> later_k, later_q;
      float between[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float factor = __expf(lds_l[row + at + e]);
        later_k.set(e, lds_k[row + at + e] * factor);
        later_q.set(e, lds_q[row + at + e] * factor);
        between[e] = 0.0f;
      }
#pragma unroll
      for (int j = 2; j >= 0; --j) {
        if (j >= wave) continue;
        const int other = (j * kBlock + column) * kSliceStride;
        WideFrag<T> earlier;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float total = lds_total[j][at + e];
          earlier.set(e, lds_k[other + at + e] * __expf(total - lds_l[other + at + e] + between[e]));
          between[e] += total;
        }
        acc_k[j] = mma_wide_both(earlier, later_k, acc_k[j]);
        acc_q[j] = mma_wide_both(earlier, later_q, acc_q[j]);
      }
    }
    // inside the block: token `column` against tokens quad * 4 .. + 3
    const int valid = min(kSlice, (int)(np - s0));
    for (int at = 0; at < valid; at += 4) {
      const f32x4 li = *reinterpret_cast<const f32x4 *>(lds_l + row + at);
      const f32x4 ki = *reinterpret_cast<const f32x4 *>(lds_k + row + at);
      const f32x4 qi = *reinterpret_cast<const f32x4 *>(lds_q + row + at);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int other = (wave * kBlock + quad * 4 + r) * kSliceStride + at;
        const f32x4 lj = *reinterpret_cast<const f32x4 *>(lds_l + other), kj = *reinterpret_cast<const f32x4 *>(lds_k + other);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float weighted = kj[e] * __expf(fminf(li[e] - lj[e], 0.0f));  // (positive: a later token, not used)
          own_k[r] = fmaf(ki[e], weighted, own_k[r]);
          own_q[r] = fmaf(qi[e], weighted, own_q[r]);
        }
      }
    }
  }
  __syncthreads();

  // N to LDS, A to memory; rows are the later token
  {
    const int i = wave * kBlock + column;
    const float beta = lds_beta[i];
    float *scores = w.scores + each * Q * Q + (size_t)i * Q;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f32x4 n = {0.0f, 0.0f, 0.0f, 0.0f}, s = n;
      if (j < 3 && j < wave) {
        n = acc_k[j < 3 ? j : 0];
        s = acc_q[j < 3 ? j : 0];
      } else if (j == wave) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int other = quad * 4 + r;
          n[r] = other < column ? own_k[r] : 0.0f;
          s[r] = other <= column ? own_q[r] : 0.0f;
        }
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) n[r] *= beta;
      *reinterpret_cast<f32x4 *>(lds_n + i * kSliceStride + j * kBlock + quad * 4) = n;
      *reinterpret_cast<f32x4 *>(scores + j * kBlock + quad * 4) = s;
    }
  }
  __syncthreads();

  // forward substitution, a thread a column of the right-hand sides
  for (uint32_t n = tid; n < a.vdim + np; n += 256) {
    float x[Q];
    const bool value = n < a.vdim;
    if (value) {
      conv_tokens<T, TAPS>(a, w.channels, 2 * a.kv_heads * a.dim + head * a.vdim + n, (int)t_first, x);
    } else {
#pragma unroll
      for (int i = 0; i < Q; ++i) x[i] = kd[(size_t)i * np + (n - a.vdim)];
    }
#pragma unroll
    for (int i = 0; i < Q; ++i) {
      x[i] *= lds_beta[i];
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const f32x4 row = *reinterpret_cast<const f32x4 *>(lds_n + i * kSliceStride + j);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j + e < i) x[i] = fmaf(-row[e], x[j + e], x[i]);
      }
    }
    if (value) {
      float *target = w.solved + (each * w.ep + n) * Q;
#pragma unroll
      for (int i = 0; i < Q; i += 4) *reinterpret_cast<f32x4 *>(target + i) = f32x4{x[i], x[i + 1], x[i + 2], x[i + 3]};
    } else {
#pragma unroll
      for (int i = 0; i < Q; ++i) store_wide_one<T>(w_out + (size_t)i * np + (n - a.vdim), plane, x[i]);
    }
  }
}

__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

template <typename T, int NT>
struct DeltaOperands {
  WideFrag<T> w[2 * NT];   // W: the wave's 16 tokens, 32 channels each
  WideFrag<T> k[NT][2];    // decayed K^T: the wave's channel tiles, 32 tokens each
  f32x4 solved;            // V': four tokens of the lane's column
  f32x4 end[NT];
};

// The serial part: a workgroup owns 16 value columns of one head; its waves the channel tiles wave + 4 t of the
// state (dim <= 64 NT) and 16 tokens of U.
template <typename T, int NT>
__global__ __launch_bounds__(256, 1) void delta_state_kernel(DeltaArgs a, DeltaWorkspace w) {
  constexpr int SS = NT * 64 + 16 / (int)sizeof(T), SU = Q + 16 / (int)sizeof(T);
  __shared__ __attribute__((aligned(16))) T lds_s[kPlanes<T>][16 * SS];
  __shared__ __attribute__((aligned(16))) T lds_u[kPlanes<T>][16 * SU];
  const uint32_t head = blockIdx.x, v0 = blockIdx.y * 16, np = w.np;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const uint32_t slot = a.step[kStateSlot], v = v0 + column, v_row = min(v, a.vdim - 1);
  const bool fresh = a.step[kStatePosition] == 0;
  float *saved = a.state + ((size_t)slot * a.heads + head) * a.dim * a.vdim + v_row;
  const size_t plane = (size_t)Q * np;

  f32x4 state[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t c = (wave + 4 * t) * 16 + quad * 4 + r;
      state[t][r] = !fresh && c < a.dim ? saved[(size_t)c * a.vdim] : 0.0f;
    }

  auto load = [&](DeltaOperands<T, NT> &o, uint32_t chunk) {
    const size_t each = (size_t)chunk * a.heads + head;
    const T *w_in = static_cast<const T *>(w.w) + each * kPlanes<T> * plane + (size_t)(wave * 16 + column) * np + quad * 8;
    const T *kt = static_cast<const T *>(w.kt) + each * kPlanes<T> * plane;
#pragma unroll
    for (int s = 0; s < 2 * NT; ++s)
      if (s * 32 < (int)np) o.w[s] = load_wide<T>(w_in + s * 32, plane);
    o.solved = *reinterpret_cast<const f32x4 *>(w.solved + (each * w.ep + v_row) * Q + wave * 16 + quad * 4);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const uint32_t tile = (wave + 4 * t) * 16;
      if (tile >= np) continue;
      o.end[t] = *reinterpret_cast<const f32x4 *>(w.end + each * np + tile + quad * 4);
#pragma unroll
      for (int s = 0; s < 2; ++s) o.k[t][s] = load_wide<T>(kt + (size_t)(tile + column) * Q + s * 32 + quad * 8, plane);
    }
  };
  auto step = [&](const DeltaOperands<T, NT> &o, uint32_t chunk) {
    const size_t each = (size_t)chunk * a.heads + head;
    const size_t state_plane = (size_t)w.ep * np;
    T *states = static_cast<T *>(w.states) + each * kPlanes<T> * state_plane + (size_t)v0 * np;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const uint32_t c = (wave + 4 * t) * 16;
      if (c >= np) continue;
      const float four[4] = {state[t][0], state[t][1], state[t][2], state[t][3]};
      store_wide<T>(&lds_s[0][column * SS + c + quad * 4], 16 * SS, four);
      // [16 columns][32 channels] blocks, lane (channel / 8) * 16 + column holding eight channels
      store_wide<T>(states + c / 32 * 512 + ((c / 16 % 2 * 2 + quad / 2) * 16 + column) * 8 + quad % 2 * 4, state_plane, four);
    }
    lds_barrier();
    f32x4 read = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int s = 0; s < 2 * NT; ++s)
      if (s * 32 < (int)np) {
        const WideFrag<T> fs = load_wide<T>(&lds_s[0][column * SS + s * 32 + quad * 8], 16 * SS);
        read = mma_wide_both(o.w[s], fs, read);
      }
    float u[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) u[r] = o.solved[r] - read[r];
    store_wide<T>(&lds_u[0][column * SU + wave * 16 + quad * 4], 16 * SU, u);
    store_wide<T>(static_cast<T *>(w.u) + each * kPlanes<T> * w.ep * Q + (size_t)v * Q + wave * 16 + quad * 4,
                  (size_t)w.ep * Q, u);
    lds_barrier();
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if ((wave + 4 * t) * 16 >= (int)np) continue;
#pragma unroll
      for (int r = 0; r < 4; ++r) state[t][r] *= o.end[t][r];
    }
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const WideFrag<T> fu = load_wide<T>(&lds_u[0][column * SU + s * 32 + quad * 8], 16 * SU);
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if ((wave + 4 * t) * 16 < (int)np) state[t] = mma_wide_both(o.k[t][s], fu, state[t]);
    }
  };

  if (NT <= 2) {  // operands a chunk ahead
    DeltaOperands<T, NT> ring[2];
    load(ring[0], 0);
    for (uint32_t chunk = 0; chunk < w.chunks; chunk += 2) {
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        if (chunk + i >= w.chunks) break;
        load(ring[(i + 1) % 2], min(chunk + i + 1, w.chunks - 1));
        __builtin_amdgcn_sched_barrier(0);  // the requests stay ahead of the arithmetic
        step(ring[i], chunk + i);
      }
    }
  } else {
    DeltaOperands<T, NT> now;
    for (uint32_t chunk = 0; chunk < w.chunks; ++chunk) {
      load(now, chunk);
      step(now, chunk);
    }
  }
  if (v < a.vdim)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const uint32_t c = (wave + 4 * t) * 16 + quad * 4 + r;
        if (c < a.dim) saved[(size_t)c * a.vdim] = state[t][r];
      }
}

// The parallel part: a workgroup per chunk and head, 16 tokens a wave, all value columns, so that a head's norm
// stays in the wave.  The workgroups behind the chunks' ones: the step's last inputs into the convolution's ring.
template <typename T, int STEPS, int NE>
__global__ __launch_bounds__(256) void delta_output_kernel(DeltaArgs a, DeltaWorkspace w) {
  const uint32_t chunk = blockIdx.x, head = blockIdx.y, np = w.np;
  if (chunk >= w.chunks) {
    if (head > 0) return;
    const uint32_t t = a.m - 1 - (chunk - w.chunks), position = a.step[kStatePosition] + t;
    float *ring = a.conv_state + ((size_t)a.step[kStateSlot] * a.taps + position % a.taps) * w.channels;
    const T *input = static_cast<const T *>(a.projected) + (size_t)t * a.ld;
    for (uint32_t c = threadIdx.x; c < w.channels; c += 256) ring[c] = to_f32(input[c]);
    return;
  }
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const size_t each = (size_t)chunk * a.heads + head, plane = (size_t)Q * np, state_plane = (size_t)w.ep * np;
  const int token = wave * 16 + column;
  const uint32_t row = chunk * Q + token;
  const T *qd = static_cast<const T *>(w.qd) + each * kPlanes<T> * plane + (size_t)token * np + quad * 8;
  WideFrag<T> fq[STEPS], weight[2];
#pragma unroll
  for (int s = 0; s < STEPS; ++s)
    if (s * 32 < (int)np) fq[s] = load_wide<T>(qd + s * 32, plane);
  const float *scores = w.scores + each * Q * Q + (size_t)token * Q + quad * 8;
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const f32x8 eight = *reinterpret_cast<const f32x8 *>(scores + s * 32);
#pragma unroll
    for (int e = 0; e < 8; ++e) weight[s].set(e, eight[e]);
  }
  f32x4 out[NE];
  float square = 0.0f;
#pragma unroll
  for (int t = 0; t < NE; ++t) {
    out[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    if (t * 16 >= (int)a.vdim) continue;
    const T *states = static_cast<const T *>(w.states) + each * kPlanes<T> * state_plane + (size_t)t * 16 * np + lane * 8;
#pragma unroll
    for (int s = 0; s < STEPS; ++s)
      if (s * 32 < (int)np) out[t] = mma_wide_both(load_wide<T>(states + s * 512, state_plane), fq[s], out[t]);
    const T *u = static_cast<const T *>(w.u) + each * kPlanes<T> * w.ep * Q + (size_t)(t * 16 + column) * Q + quad * 8;
#pragma unroll
    for (int s = 0; s < 2; ++s)
      if (s * 32 <= wave * 16 + 15)  // the others come later than all of the wave's tokens
        out[t] = mma_wide_both(load_wide<T>(u + s * 32, (size_t)w.ep * Q), weight[s], out[t]);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (t * 16 + quad * 4 + r < (int)a.vdim) square = fmaf(out[t][r], out[t][r], square);
  }
  square += __shfl_xor(square, 16, 64);
  square += __shfl_xor(square, 32, 64);
  const float scale = a.out_scale / sqrtf(square / (float)a.vdim + a.epsilon);
  if (row >= a.m) return;
  const T *gate = static_cast<const T *>(a.gate) + ((size_t)row * a.heads + head) * a.vdim;
  T *target = static_cast<T *>(a.out) + (size_t)row * a.ld_out + (size_t)head * a.vdim;
  typedef T x4 __attribute__((ext_vector_type(4)));
  const bool vec = a.vdim % 4 == 0 && a.ld_out % 4 == 0 && reinterpret_cast<size_t>(a.out) % sizeof(x4) == 0;
#pragma unroll
  for (int t = 0; t < NE; ++t) {
    const uint32_t v = t * 16 + quad * 4;
    if (v >= a.vdim) continue;
    if (vec) {
      const x4 g = *reinterpret_cast<const x4 *>(gate + v);
      x4 packed;
#pragma unroll
      for (int r = 0; r < 4; ++r) packed[r] = (T)(out[t][r] * scale * bf16_at(a.norm, v + r) * sigmoid_f32(to_f32(g[r])));
      *reinterpret_cast<x4 *>(target + v) = packed;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (v + r < a.vdim)
          target[v + r] = (T)(out[t][r] * scale * bf16_at(a.norm, v + r) * sigmoid_f32(to_f32(gate[v + r])));
    }
  }
}

template <typename T, int STEPS>
hipError_t run_output(const DeltaArgs &a, const DeltaWorkspace &w, hipStream_t stream) {
  const dim3 grid(w.chunks + std::min(a.m, a.taps), a.heads);
  if (w.ep <= 64) delta_output_kernel<T, STEPS, 4><<<grid, 256, 0, stream>>>(a, w);
  else if (w.ep <= 128) delta_output_kernel<T, STEPS, 8><<<grid, 256, 0, stream>>>(a, w);
  else delta_output_kernel<T, STEPS, 16><<<grid, 256, 0, stream>>>(a, w);
  return hipGetLastError();
}

template <typename T, int NT>
hipError_t run_scan(const DeltaArgs &a, const DeltaWorkspace &w, hipStream_t stream) {
  delta_state_kernel<T, NT><<<dim3(a.heads, w.ep / 16), 256, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  return run_output<T, 2 * NT>(a, w, stream);
}

template <typename T, int TAPS>
hipError_t run_chunks(const DeltaArgs &a, const DeltaWorkspace &w, hipStream_t stream) {
  const dim3 key_grid((a.m + 4 * kKeyTokens - 1) / (4 * kKeyTokens), a.kv_heads, 2);
  if (a.dim <= 64) delta_keys_kernel<T, 1, TAPS><<<key_grid, 256, 0, stream>>>(a, w);
  else if (a.dim <= 128) delta_keys_kernel<T, 2, TAPS><<<key_grid, 256, 0, stream>>>(a, w);
  else delta_keys_kernel<T, 4, TAPS><<<key_grid, 256, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  delta_chunk_kernel<T, TAPS><<<dim3(w.chunks, a.heads), 256, 0, stream>>>(a, w);
  return hipGetLastError();
}

template <typename T>
hipError_t run_prefill(const DeltaArgs &a, hipStream_t stream) {
  const DeltaWorkspace w = layout(a);
  hipError_t status = a.taps == 4 ? run_chunks<T, 4>(a, w, stream) : run_chunks<T, 0>(a, w, stream);
  if (status != hipSuccess) return status;
  if (w.np <= 64) return run_scan<T, 1>(a, w, stream);
  if (w.np <= 128) return run_scan<T, 2>(a, w, stream);
  return run_scan<T, 4>(a, w, stream);
}

template <int VEC>
hipError_t run_step(const DeltaArgs &a, hipStream_t stream) {
  const uint32_t groups = kStepThreads / (a.vdim / VEC), rows = (a.dim + groups - 1) / groups;
  const uint32_t bytes = (a.decay_rank + a.gate_rank) * 4;
  if (rows <= 8) delta_step_kernel<VEC, 8><<<a.heads, kStepThreads, bytes, stream>>>(a);
  else if (rows <= 32 && VEC == 4) delta_step_kernel<VEC, VEC == 4 ? 32 : 0><<<a.heads, kStepThreads, bytes, stream>>>(a);
  else delta_step_kernel<VEC, 0><<<a.heads, kStepThreads, bytes, stream>>>(a);
  return hipGetLastError();
}

}  // namespace

size_t delta_workspace_bytes(const DeltaArgs &a) {
  DeltaArgs sized = a;
  sized.workspace = nullptr;
  return layout(sized).bytes;
}

hipError_t launch_delta_step(const DeltaArgs &a, hipStream_t stream) {
  return a.vdim % 4 == 0 ? run_step<4>(a, stream) : run_step<1>(a, stream);
}

hipError_t launch_delta_prefill(const DeltaArgs &a, hipStream_t stream) {
  return a.f32 ? run_prefill<float>(a, stream) : run_prefill<__bf16>(a, stream);
}

}  // namespace llmopt
