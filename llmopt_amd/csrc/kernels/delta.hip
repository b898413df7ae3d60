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
//  * delta_chunk_kernel, a workgroup per chunk and head: convolutions, unit lengths, decays, and all that does not
//    need the state - A, the triangular solves W = (I + N)^-1 beta K exp L and V' = (I + N)^-1 beta V (then
//    U = V' - W S), and the decayed operands.  The exponents are never split around a distant reference: between
//    sub-blocks of 16 tokens the reference is the later block's start (both factors at most 1), inside one it is
//    half the block's decay, or the difference itself is taken where that could overflow.  (I + N)^-1 is formed in
//    float32: the four diagonal blocks by substitution, the others from them on the float32 matrix cores;
//  * delta_state_kernel: the serial part, from chunk to chunk, the state in matrix-core accumulators;
//  * delta_output_kernel: the outputs of all chunks at once, with their norm and gate.
// Everything but the convolutions' inputs and v keeps float32 accuracy: operands enter the bfloat16 matrix
// cores as a high and a low part.  Position 0 starts from a zero state and zero history.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr int Q = (int)kDeltaChunk, kBlock = 16;
constexpr int kSlice = 64, kSliceStride = kSlice + 4;  // channels of a pass through LDS
constexpr float kSafeLog = -120.0f;  // decay of a block whose halves neither overflow nor vanish
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
// Matrices that become matrix-core operands lie in operand order: blocks of 16 rows and 32 contraction indices, lane
// (index / 8) * 16 + row of a block holding eight of them, so that an operand is one contiguous kilobyte.
// `row`, `k` of a matrix with K (a multiple of 32) contraction indices:
__device__ __forceinline__ uint32_t operand_at(uint32_t row, uint32_t k, uint32_t K) {
  return ((row >> 4) * (K >> 5) + (k >> 5)) * 512 + (((k >> 3) & 3) * 16 + (row & 15)) * 8 + (k & 7);
}

// Per chunk and head, np: dim to 64, 128 or 256 (the kernels' own sizes: no load of theirs is conditional), ep: vdim to a
// multiple of 16.
struct DeltaWorkspace {
  void *w, *qd;           // wide operands [chunks][heads][planes][Q][np]: W, Q exp L
  void *kt;               // wide operand [chunks][heads][planes][np][Q]: (K exp(L_end - L))^T
  float *solved;          // [chunks][heads][ep / 16][4][64 lanes][4]: V' as products leave it
  void *kd;               // wide operand [chunks][heads][planes][np][Q]: (K exp L)^T
  void *v;                // operand [chunks][heads][ep][Q]: V^T
  float *end;             // [chunks][heads][np]: exp L_end
  float *scores;          // [chunks][heads][Q][Q]: A
  void *u;                // wide operand [chunks][heads][planes][ep][Q]: U^T
  void *states;           // wide operand [chunks][heads][planes][ep][np]: every chunk's incoming S^T
  uint32_t chunks, channels, np, ep;
  size_t bytes;
};

DeltaWorkspace layout(const DeltaArgs &a) {
  DeltaWorkspace w = {};
  w.chunks = (a.m + Q - 1) / Q;
  w.channels = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
  w.np = a.dim <= 64 ? 64 : a.dim <= 128 ? 128 : 256;
  w.ep = (a.vdim + 15) / 16 * 16;
  uint8_t *base = static_cast<uint8_t *>(a.workspace);
  size_t at = 0;
  auto take = [&](size_t values) {
    void *p = base ? base + at : nullptr;
    at += (values * 4 + 255) & ~(size_t)255;
    return p;
  };
  const size_t each = (size_t)w.chunks * a.heads;
  w.w = take(each * Q * w.np);
  w.qd = take(each * Q * w.np);
  w.kt = take(each * Q * w.np);
  w.solved = static_cast<float *>(take(each * Q * w.ep));
  w.kd = take(each * Q * w.np);
  w.v = take(each * Q * w.ep);
  w.end = static_cast<float *>(take(each * w.np));
  w.scores = static_cast<float *>(take(each * Q * Q));
  w.u = take(each * Q * w.ep);
  w.states = take(each * w.ep * w.np);
  w.bytes = at;
  return w;
}

// ---- one token ---------------------------------------------------------------------------------------

constexpr int kStepThreads = 512, kRowsAhead = 8;

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
      s[i] = *reinterpret_cast<const vec *>(state + min(r, a.dim - 1) * a.vdim + column);
      if (fresh || r >= a.dim) s[i] = 0.0f;
    }
  }
  // rows of the low-rank products, all on their way at once where they are short
  const int part = tid & 15;
  auto row_rank = [&](uint32_t r) { return r < a.dim ? a.decay_rank : a.gate_rank; };
  auto row_weights = [&](uint32_t r) {
    return reinterpret_cast<const __bf16 *>(r < a.dim ? a.w_decay + ((size_t)head * a.dim + r) * a.decay_rank
                                                      : a.w_gate + ((size_t)head * a.vdim + (r - a.dim)) * a.gate_rank);
  };
  const bool ahead = a.decay_rank <= 128 && a.gate_rank <= 128 && (a.decay_rank | a.gate_rank) % 8 == 0 &&
                     a.dim + a.vdim <= kRowsAhead * (kStepThreads / 16);
  bf16x8 pieces[kRowsAhead];
  if (ahead) {
#pragma unroll
    for (int i = 0; i < kRowsAhead; ++i) {
      const uint32_t r = min((uint32_t)((tid >> 4) + i * (kStepThreads / 16)), a.dim + a.vdim - 1);
      pieces[i] = load_piece(row_weights(r) + part * 8, (int)row_rank(r) - part * 8, true);
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
#pragma unroll 1
    for (uint32_t c = lane; c < a.dim; c += 64) sum += key[c] * query[c];
    sum = wave_sum(sum);
    if (lane == 0) product = sum;
  }
  // decay and gate: sixteen lanes a row of the low-rank products
  auto finish = [&](uint32_t r, float sum) {
#pragma unroll
    for (int mask = 8; mask >= 1; mask >>= 1) sum += __shfl_xor(sum, mask, 64);
    if (part != 0 || r >= a.dim + a.vdim) return;
    if (r < a.dim) decay[r] = expf(-rate * softplus_f32(sum + bf16_at(a.dt_bias, (size_t)head * a.dim + r)));
    else gate[r - a.dim] = sigmoid_f32(sum);
  };
  if (ahead) {
    f32x8 x[2];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      x[0][e] = part * 8 + e < a.decay_rank ? ranks[part * 8 + e] : 0.0f;
      x[1][e] = part * 8 + e < a.gate_rank ? ranks[a.decay_rank + part * 8 + e] : 0.0f;
    }
#pragma unroll
    for (int i = 0; i < kRowsAhead; ++i) {
      const uint32_t r = (tid >> 4) + i * (kStepThreads / 16);
      float sum = 0.0f;
#pragma unroll
      for (int e = 0; e < 8; ++e) sum = fmaf((float)pieces[i][e], r < a.dim ? x[0][e] : x[1][e], sum);
      finish(r, sum);
    }
  } else {
    for (uint32_t r = tid >> 4; r < a.dim + a.vdim; r += kStepThreads / 16) {
      const uint32_t rank = row_rank(r);
      const __bf16 *w = row_weights(r);
      const float *x = r < a.dim ? ranks : ranks + a.decay_rank;
      float sum = 0.0f;
      for (uint32_t k = part * 8; k < rank; k += 128) {
        const bf16x8 piece = load_piece(w + k, (int)rank - (int)k, rank % 8 == 0);
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (k + e < rank) sum = fmaf((float)piece[e], x[k + e], sum);
      }
      finish(r, sum);
    }
  }
  __syncthreads();

  vec from_key = 0.0f, from_query = 0.0f;
  if (owner) {
    if (R > 0) {
#pragma unroll
      for (int i = 0; i < R; ++i) {
        const uint32_t r = min(row_at(i), a.dim - 1);  // (zeros behind the last row)
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
#pragma unroll 4
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

// COUNT consecutive outputs of the convolution of one channel from token t0 of the step on, behind silu.  TAPS: its
// length, at most COUNT + 1 (0: any).  t0 is a multiple of COUNT and the same in a whole wave; inputs before the step
// come from the ring, those behind its end are zero.  All loads of a channel are requested before the first is used.
template <typename T, int TAPS, int COUNT>
__device__ __forceinline__ void conv_tokens(const DeltaArgs &a, uint32_t channels, uint32_t channel, int t0,
                                            float (&out)[COUNT]) {
  const T *input = static_cast<const T *>(a.projected) + channel;
  const uint32_t position = a.step[kStatePosition];
  const float *ring = a.conv_state + (size_t)a.step[kStateSlot] * a.taps * channels + channel;
  const int last = (int)a.m - 1;
  auto before = [&](int t) {  // t < 0
    return (int64_t)position + t >= 0 ? ring[(size_t)((position + t) % a.taps) * channels] : 0.0f;
  };
#pragma unroll
  for (int i = 0; i < COUNT; ++i) out[i] = 0.0f;
  if (TAPS > 0) {
    constexpr int BEFORE = TAPS > 0 ? TAPS - 1 : 0;
    static_assert(BEFORE <= COUNT, "only the first block of a step reaches behind it");
    T raw[COUNT + BEFORE];
#pragma unroll
    for (int i = 0; i < COUNT + BEFORE; ++i) raw[i] = input[(size_t)(uint32_t)min(max(t0 + i - BEFORE, 0), last) * a.ld];
    float window[COUNT + BEFORE];
#pragma unroll
    for (int i = 0; i < COUNT + BEFORE; ++i) window[i] = t0 + i - BEFORE <= last ? to_f32(raw[i]) : 0.0f;
    if (t0 == 0) {
#pragma unroll
      for (int i = 0; i < BEFORE; ++i) window[i] = before(i - BEFORE);
    }
#pragma unroll
    for (int tap = 0; tap < TAPS; ++tap) {
      const float weight = bf16_at(a.conv, (size_t)channel * TAPS + tap);
#pragma unroll
      for (int i = 0; i < COUNT; ++i) out[i] = fmaf(weight, window[i + tap], out[i]);
    }
  } else {
    for (uint32_t tap = 0; tap < a.taps; ++tap) {
      const float weight = bf16_at(a.conv, (size_t)channel * a.taps + tap);
      const int first = t0 - (int)(a.taps - 1 - tap);
#pragma unroll
      for (int i = 0; i < COUNT; ++i) {
        const float now = to_f32(input[(size_t)(uint32_t)min(max(first + i, 0), last) * a.ld]);
        const float value = first + i < 0 ? before(first + i) : first + i <= last ? now : 0.0f;
        out[i] = fmaf(weight, value, out[i]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < COUNT; ++i) out[i] *= __builtin_amdgcn_rcpf(1.0f + __expf(-out[i]));
}

// a b for 16 x 16 blocks in float32.  a: the lane's four consecutive values of row lane % 16; b and the result: rows
// 4 (lane / 16) .. + 3 of column lane % 16.
__device__ __forceinline__ f32x4 block_product(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
  for (int s = 0; s < 4; ++s) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[s], b[s], c, 0, 0, 0);
  return c;
}

// SLICES: dim <= 64 SLICES.  Wherever a thread owns a channel or value column it has the sixteen tokens of block `wave`.
template <typename T, int SLICES, int TAPS>
__global__ __launch_bounds__(256, SLICES <= 2 ? 2 : 1) void delta_chunk_kernel(DeltaArgs a, DeltaWorkspace w) {
  __shared__ __attribute__((aligned(16))) float lds_k[Q * kSliceStride], lds_q[Q * kSliceStride], lds_l[Q * kSliceStride];
  __shared__ __attribute__((aligned(16))) float lds_total[4][kSlice], lds_beta[Q];
  float *lds_n = lds_q, *lds_t = lds_k;  // N and (I + N)^-1, once the slices are done
  const uint32_t chunk = blockIdx.x, head = blockIdx.y, group = head / (a.heads / a.kv_heads);
  const int tid = threadIdx.x, lane = tid & 63, column = lane & 15, quad = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const size_t each = (size_t)chunk * a.heads + head;
  constexpr uint32_t np = SLICES * kSlice;
  constexpr size_t plane = (size_t)Q * np;
  const uint32_t t_first = chunk * Q, t_wave = t_first + wave * kBlock;
  T *qd = static_cast<T *>(w.qd) + each * kPlanes<T> * plane, *kt = static_cast<T *>(w.kt) + each * kPlanes<T> * plane;
  T *kd = static_cast<T *>(w.kd) + each * kPlanes<T> * plane, *w_out = static_cast<T *>(w.w) + each * kPlanes<T> * plane;
  T *values = static_cast<T *>(w.v) + each * w.ep * Q;
  const float rate = expf(bf16_at(a.a_log, head));
  if (tid < Q) lds_beta[tid] = t_first + tid < a.m ? sigmoid_f32(a.beta[(size_t)(t_first + tid) * a.heads + head]) : 0.0f;

  // queries and keys: convolution, silu, unit length
  float k[SLICES][kBlock], q[SLICES][kBlock];
#pragma unroll
  for (int s = 0; s < SLICES; ++s) {
    const uint32_t c = s * kSlice + lane;
    const uint32_t channel = group * a.dim + min(c, a.dim - 1);
    conv_tokens<T, TAPS>(a, w.channels, channel, (int)t_wave, q[s]);
    conv_tokens<T, TAPS>(a, w.channels, a.kv_heads * a.dim + channel, (int)t_wave, k[s]);
    if (c >= a.dim) {
#pragma unroll
      for (int i = 0; i < kBlock; ++i) q[s][i] = k[s][i] = 0.0f;
    }
  }
  const float query_scale = 1.0f / sqrtf((float)a.dim);
#pragma unroll
  for (int i = 0; i < kBlock; ++i) {
    float qq = 0.0f, kk = 0.0f;
#pragma unroll
    for (int s = 0; s < SLICES; ++s) {
      qq = fmaf(q[s][i], q[s][i], qq);
      kk = fmaf(k[s][i], k[s][i], kk);
    }
    const bool real = t_wave + i < a.m;
    qq = wave_sum(qq);
    kk = wave_sum(kk);
    const float q_scale = real ? query_scale * __builtin_amdgcn_rsqf(qq + kUnitEpsilon) : 0.0f;
    const float k_scale = real ? __builtin_amdgcn_rsqf(kk + kUnitEpsilon) : 0.0f;
#pragma unroll
    for (int s = 0; s < SLICES; ++s) {
      q[s][i] *= q_scale;
      k[s][i] *= k_scale;
    }
  }

  f32x4 acc_k[3], acc_q[3], own_k, own_q;
#pragma unroll
  for (int j = 0; j < 3; ++j) acc_k[j] = acc_q[j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  own_k = own_q = f32x4{0.0f, 0.0f, 0.0f, 0.0f};

#pragma unroll
  for (int slice = 0; slice < SLICES; ++slice) {
    const uint32_t s0 = slice * kSlice;
    if (slice > 0) __syncthreads();
    const uint32_t c = s0 + lane;
    float log_decay[kBlock], prefix[kBlock], running = 0.0f;
    const float bias = c < a.dim ? bf16_at(a.dt_bias, (size_t)head * a.dim + c) : 0.0f;
#pragma unroll
    for (int i = 0; i < kBlock; ++i)
      log_decay[i] = a.decay[((size_t)min(t_wave + i, a.m - 1) * a.heads + head) * a.dim + min(c, a.dim - 1)];
#pragma unroll
    for (int i = 0; i < kBlock; ++i) {
      log_decay[i] = t_wave + i < a.m && c < a.dim ? -rate * softplus_fast_f32(log_decay[i] + bias) : 0.0f;
      running += log_decay[i];
      prefix[i] = running;
      const int at = (wave * kBlock + i) * kSliceStride + lane;
      lds_k[at] = k[slice][i];
      lds_q[at] = q[slice][i];
      lds_l[at] = running;
    }
    lds_total[wave][lane] = running;
    __syncthreads();
    {
      float before = 0.0f, after = 0.0f;
#pragma unroll
      for (int b = 0; b < 4; ++b) {
        if (b < wave) before += lds_total[b][lane];
        if (b > wave) after += lds_total[b][lane];
      }
      if (wave == 3) w.end[each * np + c] = __expf(before + running);
      float decayed[kBlock];
      auto store_column = [&](T *target) {
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          float eight[8];
#pragma unroll
          for (int e = 0; e < 8; ++e) eight[e] = decayed[half * 8 + e];
          store_wide<T>(target + operand_at(c, wave * kBlock + half * 8, Q), plane, eight);
        }
      };
#pragma unroll
      for (int i = kBlock - 1; i >= 0; --i) {
        decayed[i] = k[slice][i] * __expf(after);
        after += log_decay[i];
      }
      store_column(kt);
#pragma unroll
      for (int i = 0; i < kBlock; ++i) decayed[i] = k[slice][i] * __expf(before + prefix[i]);
      store_column(kd);
    }

    // products with the blocks before this wave's one, and inside it
    const int row = (wave * kBlock + column) * kSliceStride;
    const bool safe = __all(lds_total[wave][lane] > kSafeLog);
#pragma unroll
    for (int step = 0; step < kSlice / 32; ++step) {
      const int at = step * 32 + quad * 8;
      WideFrag<T> later_k, later_q, earlier;
      f32x8 l, kv, qv;
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        const f32x4 l4 = *reinterpret_cast<const f32x4 *>(lds_l + row + at + half * 4);
        const f32x4 k4 = *reinterpret_cast<const f32x4 *>(lds_k + row + at + half * 4);
        const f32x4 q4 = *reinterpret_cast<const f32x4 *>(lds_q + row + at + half * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          l[half * 4 + e] = l4[e];
          kv[half * 4 + e] = k4[e];
          qv[half * 4 + e] = q4[e];
        }
      }
      if (safe) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float from_middle = l[e] - 0.5f * lds_total[wave][at + e];
          const float up = __expf(from_middle);
          later_k.set(e, kv[e] * up);
          later_q.set(e, qv[e] * up);
          earlier.set(e, kv[e] * __expf(-from_middle));
        }
        own_k = mma_wide_both(earlier, later_k, own_k);
        own_q = mma_wide_both(earlier, later_q, own_q);
      }
      float between[8];  // the decay of the blocks between
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const float factor = __expf(l[e]);
        qv[e] *= factor;
        later_k.set(e, kv[e] * factor);
        later_q.set(e, qv[e]);
        between[e] = 0.0f;
      }
#pragma unroll
      for (int j = 2; j >= 0; --j) {
        if (j >= wave) continue;
        const int other = (j * kBlock + column) * kSliceStride + at;
#pragma unroll
        for (int half = 0; half < 2; ++half) {
          const f32x4 l4 = *reinterpret_cast<const f32x4 *>(lds_l + other + half * 4);
          const f32x4 k4 = *reinterpret_cast<const f32x4 *>(lds_k + other + half * 4);
          const f32x4 total = *reinterpret_cast<const f32x4 *>(&lds_total[j][at + half * 4]);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            earlier.set(half * 4 + e, k4[e] * __expf(total[e] - l4[e] + between[half * 4 + e]));
            between[half * 4 + e] += total[e];
          }
        }
        acc_k[j] = mma_wide_both(earlier, later_k, acc_k[j]);
        acc_q[j] = mma_wide_both(earlier, later_q, acc_q[j]);
      }
      float eight[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) eight[e] = qv[e] * __expf(between[e]);
      store_wide<T>(qd + operand_at(wave * kBlock + column, s0 + at, np), plane, eight);
    }
    if (!safe) {  // token `column` against tokens quad * 4 .. + 3
      for (int at = 0; at < kSlice; ++at) {
        const float li = lds_l[row + at], ki = lds_k[row + at], qi = lds_q[row + at];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int other = (wave * kBlock + quad * 4 + r) * kSliceStride + at;
          const float weighted = lds_k[other] * __expf(fminf(li - lds_l[other], 0.0f));  // (positive: a later token, not used)
          own_k[r] = fmaf(ki, weighted, own_k[r]);
          own_q[r] = fmaf(qi, weighted, own_q[r]);
        }
      }
    }
  }
  // values: convolution and silu
  for (uint32_t n = lane; n < w.ep; n += 64) {
    float v[kBlock];
    if (n < a.vdim) {
      conv_tokens<T, TAPS>(a, w.channels, 2 * a.kv_heads * a.dim + head * a.vdim + n, (int)t_wave, v);
    } else {
#pragma unroll
      for (int i = 0; i < kBlock; ++i) v[i] = 0.0f;
    }
#pragma unroll
    for (int half = 0; half < 2; ++half) {
      Frag<T> eight;
#pragma unroll
      for (int e = 0; e < 8; ++e) eight[e] = (T)v[half * 8 + e];
      *reinterpret_cast<Frag<T> *>(values + operand_at(n, wave * kBlock + half * 8, Q)) = eight;
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

  // the inverse's diagonal block `wave`, a lane a column
  {
    const float *n = lds_n + wave * kBlock * kSliceStride + wave * kBlock;
    float *t = lds_t + wave * kBlock * kSliceStride + wave * kBlock;
    float x[kBlock];
#pragma unroll
    for (int i = 0; i < kBlock; ++i) {
      x[i] = i == column ? 1.0f : 0.0f;
#pragma unroll
      for (int j = 0; j < i; j += 4) {
        const f32x4 four = *reinterpret_cast<const f32x4 *>(n + i * kSliceStride + j);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (j + e < i) x[i] = fmaf(-four[e], x[j + e], x[i]);
      }
      if (quad == 0) t[i * kSliceStride + column] = x[i];
    }
  }
  __syncthreads();
  // block column `wave` below the diagonal: T_ij = -T_ii sum_(j <= k < i) N_ik T_kj
  {
    f32x4 t[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (i < wave) continue;
      if (i == wave) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          t[i][r] = lds_t[(i * kBlock + quad * 4 + r) * kSliceStride + i * kBlock + column];
        continue;
      }
      f32x4 sum = {0.0f, 0.0f, 0.0f, 0.0f};
      const int at = (i * kBlock + column) * kSliceStride + quad * 4;
#pragma unroll
      for (int j = 0; j < i; ++j)
        if (j >= wave) sum = block_product(*reinterpret_cast<const f32x4 *>(lds_n + at + j * kBlock), t[j], sum);
      const f32x4 own = *reinterpret_cast<const f32x4 *>(lds_t + at + i * kBlock);
      t[i] = block_product(-own, sum, f32x4{0.0f, 0.0f, 0.0f, 0.0f});
#pragma unroll
      for (int r = 0; r < 4; ++r)
        lds_t[(i * kBlock + quad * 4 + r) * kSliceStride + wave * kBlock + column] = t[i][r];
    }
  }
  __syncthreads();
  // times the write strengths: what the wave's tokens take from the chunk's tokens
  WideFrag<T> solve[2];
  const int token = wave * kBlock + column;
#pragma unroll
  for (int s = 0; s < 2; ++s)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int j = s * 32 + quad * 8 + e;
      solve[s].set(e, j <= token ? lds_t[token * kSliceStride + j] * lds_beta[j] : 0.0f);
    }
  const f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f};
  for (uint32_t tile = 0; tile < w.ep; tile += 16) {
    const T *v = values + tile * Q + lane * 8;
    f32x4 x = mma_wide(solve[0], *reinterpret_cast<const Frag<T> *>(v), zero);
    if (wave >= 2) x = mma_wide(solve[1], *reinterpret_cast<const Frag<T> *>(v + 512), x);
    *reinterpret_cast<f32x4 *>(w.solved + (each * w.ep + tile) * Q + wave * 256 + lane * 4) = x;
  }
  for (uint32_t tile = 0; tile < np; tile += 16) {
    const T *keys = kd + tile * Q + lane * 8;
    f32x4 x = mma_wide_both(load_wide<T>(keys, plane), solve[0], zero);
    if (wave >= 2) x = mma_wide_both(load_wide<T>(keys + 512, plane), solve[1], x);
    const float four[4] = {x[0], x[1], x[2], x[3]};
    store_wide<T>(w_out + operand_at(token, tile + quad * 4, np), plane, four);
  }
}

__device__ __forceinline__ void lds_barrier() {
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}

// step(ring[i], chunk) for every chunk in turn, their operands requested DEPTH - 1 chunks ahead.  (The loop has one exit:
// with one behind every step the compiler waits for all requests at the loop's head.)
template <int DEPTH, typename Operands, typename Load, typename Step>
__device__ __forceinline__ void walk_chunks(uint32_t chunks, Operands (&ring)[DEPTH], Load load, Step step) {
#pragma unroll
  for (int i = 0; i < DEPTH - 1; ++i) load(ring[i], min((uint32_t)i, chunks - 1));
  uint32_t chunk = 0;
  for (; chunk + DEPTH <= chunks; chunk += DEPTH) {
#pragma unroll
    for (int i = 0; i < DEPTH; ++i) {
      load(ring[(i + DEPTH - 1) % DEPTH], min(chunk + i + DEPTH - 1, chunks - 1));
      __builtin_amdgcn_sched_barrier(0);  // the requests stay ahead of the arithmetic
      step(ring[i], chunk + i);
    }
  }
#pragma unroll
  for (int i = 0; i < DEPTH - 1; ++i)
    if (chunk + i < chunks) step(ring[i], chunk + i);
}

// The serial part: a workgroup owns 16 value columns of one head.  Waves 0 .. 3 hold the state, the channel tiles
// wave + 4 t each (dim <= 64 NT), and waves 4 .. 7 compute U, 16 tokens each; state and U pass through LDS.  Each half
// keeps its operands DEPTH - 1 chunks ahead in registers, which one wave could not hold for both.
template <typename T, int NT>
__global__ __launch_bounds__(512) void delta_state_kernel(DeltaArgs a, DeltaWorkspace w) {
  constexpr uint32_t np = NT * 64;
  constexpr size_t plane = (size_t)Q * np;
  constexpr int SS = NT * 64 + 16 / (int)sizeof(T), SU = Q + 16 / (int)sizeof(T), DEPTH = NT <= 2 ? 3 : 2;
  __shared__ __attribute__((aligned(16))) T lds_s[kPlanes<T>][16 * SS];
  __shared__ __attribute__((aligned(16))) T lds_u[kPlanes<T>][16 * SU];
  const uint32_t head = blockIdx.x, v0 = blockIdx.y * 16;
  const int role = __builtin_amdgcn_readfirstlane(threadIdx.x >> 8);
  const int wave = __builtin_amdgcn_readfirstlane((threadIdx.x >> 6) & 3);
  const int lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const uint32_t v = v0 + column, v_row = min(v, a.vdim - 1);
  const size_t heads = a.heads;

  if (role == 1) {
    struct Operands {
      WideFrag<T> w[2 * NT];  // W: the wave's 16 tokens, 32 channels each
      f32x4 solved;           // V': four tokens of the lane's column
    } ring[DEPTH];
    auto load = [&](Operands &o, uint32_t chunk) {
      const size_t each = (size_t)chunk * heads + head;
      const T *w_in = static_cast<const T *>(w.w) + each * kPlanes<T> * plane + wave * 16 * np + lane * 8;
#pragma unroll
      for (int s = 0; s < 2 * NT; ++s) o.w[s] = load_wide<T>(w_in + s * 512, plane);
      o.solved = *reinterpret_cast<const f32x4 *>(w.solved + (each * w.ep + v0) * Q + wave * 256 + lane * 4);
    };
    auto step = [&](const Operands &o, uint32_t chunk) {
      lds_barrier();  // the state is there
      f32x4 read[2];
      read[0] = read[1] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int s = 0; s < 2 * NT; ++s) {
        const WideFrag<T> fs = load_wide<T>(&lds_s[0][column * SS + s * 32 + quad * 8], 16 * SS);
        read[s % 2] = mma_wide_both(o.w[s], fs, read[s % 2]);
      }
      float u[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) u[r] = o.solved[r] - (read[0][r] + read[1][r]);
      store_wide<T>(&lds_u[0][column * SU + wave * 16 + quad * 4], 16 * SU, u);
      lds_barrier();  // U is there
      store_wide<T>(static_cast<T *>(w.u) + ((size_t)chunk * heads + head) * kPlanes<T> * w.ep * Q +
                        operand_at(v, wave * 16 + quad * 4, Q),
                    (size_t)w.ep * Q, u);
    };
    walk_chunks<DEPTH>(w.chunks, ring, load, step);
    return;
  }

  const bool fresh = a.step[kStatePosition] == 0;
  float *saved = a.state + ((size_t)a.step[kStateSlot] * heads + head) * a.dim * a.vdim + v_row;
  f32x4 state[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t c = (wave + 4 * t) * 16 + quad * 4 + r;
      state[t][r] = !fresh && c < a.dim ? saved[(size_t)c * a.vdim] : 0.0f;
    }
  struct Operands {
    WideFrag<T> k[NT][2];  // decayed K^T: the wave's channel tiles, 32 tokens each
    f32x4 end[NT];
  } ring[DEPTH];
  auto load = [&](Operands &o, uint32_t chunk) {
    const size_t each = (size_t)chunk * heads + head;
    const T *kt = static_cast<const T *>(w.kt) + each * kPlanes<T> * plane + wave * 16 * Q + lane * 8;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      o.end[t] = *reinterpret_cast<const f32x4 *>(w.end + each * np + (wave + 4 * t) * 16 + quad * 4);
#pragma unroll
      for (int s = 0; s < 2; ++s) o.k[t][s] = load_wide<T>(kt + t * 64 * Q + s * 512, plane);
    }
  };
  auto step = [&](const Operands &o, uint32_t chunk) {
    const size_t state_plane = (size_t)w.ep * np;
    T *states = static_cast<T *>(w.states) + ((size_t)chunk * heads + head) * kPlanes<T> * state_plane;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const float four[4] = {state[t][0], state[t][1], state[t][2], state[t][3]};
      store_wide<T>(&lds_s[0][column * SS + (wave + 4 * t) * 16 + quad * 4], 16 * SS, four);
    }
    lds_barrier();
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const float four[4] = {state[t][0], state[t][1], state[t][2], state[t][3]};
      store_wide<T>(states + operand_at(v, (wave + 4 * t) * 16 + quad * 4, np), state_plane, four);
#pragma unroll
      for (int r = 0; r < 4; ++r) state[t][r] *= o.end[t][r];
    }
    lds_barrier();
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const WideFrag<T> fu = load_wide<T>(&lds_u[0][column * SU + s * 32 + quad * 8], 16 * SU);
#pragma unroll
      for (int t = 0; t < NT; ++t) state[t] = mma_wide_both(o.k[t][s], fu, state[t]);
    }
  };
  walk_chunks<DEPTH>(w.chunks, ring, load, step);
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
  constexpr uint32_t np = STEPS * 32;
  const uint32_t chunk = blockIdx.x, head = blockIdx.y;
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
  const T *qd = static_cast<const T *>(w.qd) + each * kPlanes<T> * plane + wave * 16 * np + lane * 8;
  WideFrag<T> fq[STEPS], weight[2];
#pragma unroll
  for (int s = 0; s < STEPS; ++s) fq[s] = load_wide<T>(qd + s * 512, plane);
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
    for (int s = 0; s < STEPS; ++s) out[t] = mma_wide_both(load_wide<T>(states + s * 512, state_plane), fq[s], out[t]);
    const T *u = static_cast<const T *>(w.u) + each * kPlanes<T> * w.ep * Q + t * 16 * Q + lane * 8;
#pragma unroll
    for (int s = 0; s < 2; ++s)
      if (s * 32 <= wave * 16 + 15)  // the others come later than all of the wave's tokens
        out[t] = mma_wide_both(load_wide<T>(u + s * 512, (size_t)w.ep * Q), weight[s], out[t]);
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
  delta_state_kernel<T, NT><<<dim3(a.heads, w.ep / 16), 512, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  return run_output<T, 2 * NT>(a, w, stream);
}

template <typename T, int TAPS>
hipError_t run_chunks(const DeltaArgs &a, const DeltaWorkspace &w, hipStream_t stream) {
  const dim3 grid(w.chunks, a.heads);
  if (a.dim <= 64) delta_chunk_kernel<T, 1, TAPS><<<grid, 256, 0, stream>>>(a, w);
  else if (a.dim <= 128) delta_chunk_kernel<T, 2, TAPS><<<grid, 256, 0, stream>>>(a, w);
  else delta_chunk_kernel<T, 4, TAPS><<<grid, 256, 0, stream>>>(a, w);
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
  else if (rows <= 16 && VEC == 4) delta_step_kernel<VEC, VEC == 4 ? 16 : 0><<<a.heads, kStepThreads, bytes, stream>>>(a);
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
