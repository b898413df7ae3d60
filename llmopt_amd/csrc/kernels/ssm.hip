// The Mamba-2 recurrence (state-space duality form).
//
//   S_t = exp(-a dt_t) S_(t-1) + dt_t b_t x_t^T,   y_t = S_t^T c_t + d x_t      (per head, S in float32)
//
// One token (ssm_step_kernel): a wave per row of the transposed state [vdim][state_size], lanes along the
// state; the convolution, the softplus and their bookkeeping ran in the projection's epilogue.
//
// Many tokens: chunks of 64.  Within a chunk
//   y_i = exp(L_i) S c_i + sum_{j <= i} (c_i . b_j) exp(L_i - L_j) dt_j x_j + d x_i
//   S  <- exp(L_63) S + sum_j exp(L_63 - L_j) dt_j b_j x_j^T
// with L the running sum of -a dt from the chunk's start, all as matrix products:
//  * ssm_conv_kernel: convolution and silu; leaves x and b transposed per chunk (the contraction over
//    tokens reads eight consecutive tokens of one channel) and b, c row-major;
//  * ssm_prepare_kernel: softplus, the running sums (in double, kept as two floats: their differences
//    enter an exponential) and the convolution's last inputs into the ring;
//  * ssm_scores_kernel: c_i . b_j of every chunk and group, shared by the heads of the group;
//  * ssm_state_kernel: the serial part, and nothing else: the state from chunk to chunk, in registers;
//  * ssm_output_kernel: the outputs of all chunks at once, from the states the serial part left.
// Operands that must keep float32 accuracy (the state, decay-weighted inputs and scores) enter the bfloat16
// matrix cores as a high and a low part.
// The position-0 token starts from a zero state and zero history, whatever a slot held before.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr int Q = (int)kSsmChunk;
constexpr int kConvTokens = 16;

__device__ __forceinline__ float bf16_at(const uint16_t *p, size_t i) {
  return (float)reinterpret_cast<const __bf16 *>(p)[i];
}

struct SsmWorkspace {
  void *xt;       // T [chunks][inner][Q]
  void *bt;       // T [chunks][groups * np][Q]
  void *b, *c;    // T [chunks * Q][groups * np]
  float *dt;      // [chunks][heads][Q]
  float *sum;     // [chunks][heads][2][Q] (high parts, low parts)
  float *tail;    // [chunks][heads][Q]: dt times the decay to the chunk's end
  float *scores;  // [chunks][groups][Q][Q]
  void *states;   // T [chunks][heads][planes][vdim to 16][np]: every chunk's incoming state, in operand order
  uint32_t chunks, inner, np;
  size_t bytes;
};

size_t aligned(size_t bytes) { return (bytes + 255) & ~(size_t)255; }

SsmWorkspace layout(const SsmArgs &a) {
  SsmWorkspace w = {};
  w.chunks = (a.m + Q - 1) / Q;
  w.inner = a.heads * a.vdim;
  w.np = (a.state_size + 31) / 32 * 32;
  const size_t element = a.f32 ? 4 : 2, tokens = (size_t)w.chunks * Q;
  uint8_t *base = static_cast<uint8_t *>(a.workspace);
  size_t at = 0;
  auto take = [&](size_t bytes) {
    void *p = base ? base + at : nullptr;
    at += aligned(bytes);
    return p;
  };
  w.xt = take(tokens * w.inner * element);
  w.bt = take(tokens * a.groups * w.np * element);
  w.b = take(tokens * a.groups * w.np * element);
  w.c = take(tokens * a.groups * w.np * element);
  w.dt = static_cast<float *>(take(tokens * a.heads * 4));
  w.sum = static_cast<float *>(take(tokens * a.heads * 8));
  w.tail = static_cast<float *>(take(tokens * a.heads * 4));
  w.scores = static_cast<float *>(take((size_t)w.chunks * a.groups * Q * Q * 4));
  w.states = take((size_t)w.chunks * a.heads * ((a.vdim + 15) / 16 * 16) * w.np * 4);  // two bf16 planes or one f32
  w.bytes = at;
  return w;
}

// ---- one token ---------------------------------------------------------------------------------------

constexpr int kStepRows = 4;  // state rows of a wave

__global__ __launch_bounds__(256) void ssm_step_kernel(SsmArgs a) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const uint32_t inner = a.heads * a.vdim, n = a.state_size;
  const uint32_t first = (blockIdx.x * 4 + wave) * kStepRows;
  if (first >= inner) return;
  const bool fresh = a.step[kStatePosition] == 0;
  float *state = a.ssm_state + ((size_t)a.step[kStateSlot] * inner + first) * n;
  const float *x = a.row + inner, *b = x + inner, *c = b + a.groups * n, *dt = c + a.groups * n;
  float y[kStepRows], decay[kStepRows], gain[kStepRows];
  uint32_t group[kStepRows];
#pragma unroll
  for (int r = 0; r < kStepRows; ++r) {
    const uint32_t row = min(first + r, inner - 1), head = row / a.vdim;
    decay[r] = fresh ? 0.0f : expf(-expf(bf16_at(a.a_log, head)) * dt[head]);
    gain[r] = dt[head] * x[row];
    group[r] = head / (a.heads / a.groups);
    y[r] = 0.0f;
  }
  for (uint32_t k = lane; k < n; k += 64) {
    float s[kStepRows];
#pragma unroll
    for (int r = 0; r < kStepRows; ++r) s[r] = fresh || first + r >= inner ? 0.0f : state[(size_t)r * n + k];
#pragma unroll
    for (int r = 0; r < kStepRows; ++r) {
      s[r] = fmaf(decay[r], s[r], gain[r] * b[group[r] * n + k]);
      if (first + r < inner) state[(size_t)r * n + k] = s[r];
      y[r] = fmaf(s[r], c[group[r] * n + k], y[r]);
    }
  }
#pragma unroll
  for (int r = 0; r < kStepRows; ++r) y[r] = wave_sum(y[r]);
#pragma unroll
  for (int r = 0; r < kStepRows; ++r)
    if (lane == r && first + r < inner) {
      const uint32_t row = first + r;
      a.gated[row] = (y[r] + bf16_at(a.d_skip, row / a.vdim) * x[row]) * silu_f32(a.row[row]);
    }
}

// ---- many tokens ----------------------------------------------------------------------------------------

// TAPS: the convolution's length (0: any length, its inputs read once per tap).
template <typename T, int TAPS>
__global__ __launch_bounds__(256) void ssm_conv_kernel(SsmArgs a, SsmWorkspace w) {
  const uint32_t n = a.state_size, channels = w.inner + 2 * a.groups * n;
  const uint32_t padded = w.inner + 2 * a.groups * w.np;
  const uint32_t p = blockIdx.x * 256 + threadIdx.x;  // channel, the b and c groups padded to np
  if (p >= padded) return;
  const uint32_t t0 = blockIdx.y * kConvTokens;
  // which channel of the convolution this is
  uint32_t channel = p, within = 0, which = 0;  // which: 0 x, 1 b, 2 c
  bool real = true;
  if (p >= w.inner) {
    const uint32_t q = p - w.inner, bc = a.groups * w.np;
    which = 1 + q / bc;
    within = q % bc;
    const uint32_t g = within / w.np, k = within % w.np;
    real = k < n;
    channel = w.inner + (which - 1) * a.groups * n + g * n + k;
  }
  const uint32_t ld = w.inner + channels;
  const T *input = static_cast<const T *>(a.projected) + w.inner + channel;
  const uint32_t position = a.step[kStatePosition];
  const float *ring = a.conv_state + (size_t)a.step[kStateSlot] * a.taps * channels + channel;
  T out[kConvTokens];
  if (real) {
    const float bias = bf16_at(a.conv_bias, channel);
    float sum[kConvTokens];
#pragma unroll
    for (int i = 0; i < kConvTokens; ++i) sum[i] = bias;
    // the input of token t (negative: before the step)
    auto at = [&](int t) {
      if (t >= 0) return t < (int)a.m ? to_f32(input[(size_t)t * ld]) : 0.0f;
      return (int64_t)position + t >= 0 ? ring[(size_t)((position + t) % a.taps) * channels] : 0.0f;
    };
    if (TAPS > 0) {
      float window[kConvTokens + TAPS - 1];
#pragma unroll
      for (int i = 0; i < kConvTokens + TAPS - 1; ++i) window[i] = at((int)t0 + i - (TAPS - 1));
#pragma unroll
      for (int tap = 0; tap < TAPS; ++tap) {
        const float weight = bf16_at(a.conv, (size_t)channel * TAPS + tap);
#pragma unroll
        for (int i = 0; i < kConvTokens; ++i) sum[i] = fmaf(weight, window[i + tap], sum[i]);
      }
    } else {
      for (uint32_t tap = 0; tap < a.taps; ++tap) {
        const float weight = bf16_at(a.conv, (size_t)channel * a.taps + tap);
#pragma unroll
        for (int i = 0; i < kConvTokens; ++i) sum[i] = fmaf(weight, at((int)t0 + i - (int)(a.taps - 1 - tap)), sum[i]);
      }
    }
#pragma unroll
    for (int i = 0; i < kConvTokens; ++i) out[i] = t0 + i < a.m ? (T)silu_f32(sum[i]) : (T)0.0f;
  } else {
#pragma unroll
    for (int i = 0; i < kConvTokens; ++i) out[i] = (T)0.0f;
  }
  const uint32_t chunk = t0 / Q, j = t0 % Q;
  if (which != 2) {
    T *target = which == 0 ? static_cast<T *>(w.xt) + ((size_t)chunk * w.inner + p) * Q + j
                           : static_cast<T *>(w.bt) + ((size_t)chunk * a.groups * w.np + within) * Q + j;
    Frag<T> lo, hi;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      lo[i] = out[i];
      hi[i] = out[8 + i];
    }
    reinterpret_cast<Frag<T> *>(target)[0] = lo;
    reinterpret_cast<Frag<T> *>(target)[1] = hi;
  }
  if (which != 0) {
    T *target = static_cast<T *>(which == 1 ? w.b : w.c) + (size_t)t0 * a.groups * w.np + within;
#pragma unroll
    for (int i = 0; i < kConvTokens; ++i) target[(size_t)i * a.groups * w.np] = out[i];
  }
}

// Blocks [0, chunks * ceil(heads / 4)): softplus and running sums, a wave a head and a lane a token.  The
// blocks behind: the step's last `taps` convolution inputs into the ring.
template <typename T>
__global__ __launch_bounds__(256) void ssm_prepare_kernel(SsmArgs a, SsmWorkspace w) {
  const uint32_t head_blocks = (a.heads + 3) / 4;
  if (blockIdx.x < w.chunks * head_blocks) {
    const uint32_t chunk = blockIdx.x / head_blocks, head = blockIdx.x % head_blocks * 4 + (threadIdx.x >> 6);
    if (head >= a.heads) return;
    const int j = threadIdx.x & 63;
    const uint32_t t = chunk * Q + j;
    const float bias = bf16_at(a.dt_bias, head);
    const float step = t < a.m ? softplus_f32(a.dt[(size_t)t * a.heads + head] + bias) : 0.0f;
    double running = -(double)expf(bf16_at(a.a_log, head)) * (double)step;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const double before = __shfl_up(running, d, 64);
      if (j >= d) running += before;
    }
    const double end = __shfl(running, 63, 64);
    const size_t at = (size_t)chunk * a.heads + head;
    const float high = (float)running;
    w.dt[at * Q + j] = step;
    w.tail[at * Q + j] = step * __expf((float)(end - running));
    w.sum[at * 2 * Q + j] = high;
    w.sum[at * 2 * Q + Q + j] = (float)(running - (double)high);
    return;
  }
  const uint32_t channels = w.inner + 2 * a.groups * a.state_size;
  const uint32_t t = a.m - 1 - (blockIdx.x - w.chunks * head_blocks), position = a.step[kStatePosition] + t;
  float *ring = a.conv_state + ((size_t)a.step[kStateSlot] * a.taps + position % a.taps) * channels;
  const T *input = static_cast<const T *>(a.projected) + (size_t)t * (w.inner + channels) + w.inner;
  for (uint32_t c = threadIdx.x; c < channels; c += 256) ring[c] = to_f32(input[c]);
}

template <typename T>
__global__ __launch_bounds__(256) void ssm_scores_kernel(SsmArgs a, SsmWorkspace w) {
  const uint32_t chunk = blockIdx.x, group = blockIdx.y;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const size_t ld = (size_t)a.groups * w.np;
  const T *b = static_cast<const T *>(w.b) + (size_t)chunk * Q * ld + group * w.np + quad * 8;
  const T *c = static_cast<const T *>(w.c) + (size_t)chunk * Q * ld + group * w.np + quad * 8;
  float *scores = w.scores + ((size_t)chunk * a.groups + group) * Q * Q;
  f32x4 acc[4];
#pragma unroll
  for (int t = 0; t < 4; ++t) acc[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
  for (uint32_t k = 0; k < w.np; k += 32) {
    const Frag<T> fc = *reinterpret_cast<const Frag<T> *>(c + (size_t)(wave * 16 + column) * ld + k);
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      if (t > wave) continue;
      const Frag<T> fb = *reinterpret_cast<const Frag<T> *>(b + (size_t)(t * 16 + column) * ld + k);
      acc[t] = mma(fb, fc, acc[t]);
    }
  }
#pragma unroll
  for (int t = 0; t < 4; ++t)
    *reinterpret_cast<f32x4 *>(scores + (wave * 16 + column) * Q + t * 16 + quad * 4) = acc[t];
}

// A chunk's incoming state as the matrix cores take it: float as it is, bf16 as a high and a low plane, in
// operand order: [16 state rows][32 columns] blocks, lane (column / 8) * 16 + row holding eight columns, so
// that an operand is one contiguous load and the serial part stores whole lines.
template <typename T>
constexpr int kStatePlanes = sizeof(T) == 4 ? 1 : 2;
template <typename T>
__device__ __forceinline__ T *state_block(const SsmArgs &a, const SsmWorkspace &w, uint32_t chunk, uint32_t head,
                                          int plane, uint32_t v0) {
  const size_t rows = (a.vdim + 15) & ~15u;
  return static_cast<T *>(w.states) +
         ((((size_t)chunk * a.heads + head) * kStatePlanes<T> + plane) * rows + v0) * w.np;
}

template <typename T, int NT>
struct StateOperands {
  Frag<T> x[2];      // x^T of the 16 state rows, 32 tokens each
  Frag<T> b[NT][2];  // b^T of the wave's state columns
  f32x8 tail[2];
  float end;
};

// The serial part: a workgroup owns 16 state rows of one head, its waves the 16-column tiles wave + 4 t
// (state_size <= 64 NT); the chunks' incoming states go to the workspace.  No exchange between waves.
template <typename T, int NT>
__global__ __launch_bounds__(256, 1) void ssm_state_kernel(SsmArgs a, SsmWorkspace w) {
  const uint32_t head = blockIdx.x, v0 = blockIdx.y * 16, group = head / (a.heads / a.groups);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const uint32_t n = a.state_size, slot = a.step[kStateSlot];
  const bool fresh = a.step[kStatePosition] == 0;
  const size_t ld = (size_t)a.groups * w.np;
  // lane: state row v, columns k .. k + 3 of every tile; rows beyond the head's end repeat its last one
  const uint32_t v = v0 + column, v_row = min(v, a.vdim - 1);
  float *saved = a.ssm_state + (((size_t)slot * a.heads + head) * a.vdim + v_row) * n;

  f32x4 state[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t k = (wave + 4 * t) * 16 + quad * 4 + r;
      state[t][r] = !fresh && k < n ? saved[k] : 0.0f;
    }

  auto load = [&](StateOperands<T, NT> &o, uint32_t chunk) {
    const T *x = static_cast<const T *>(w.xt) + ((size_t)chunk * w.inner + head * a.vdim + v_row) * Q + quad * 8;
    const float *tail = w.tail + ((size_t)chunk * a.heads + head) * Q + quad * 8;
    o.end = w.sum[((size_t)chunk * a.heads + head) * 2 * Q + Q - 1];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      o.x[s] = *reinterpret_cast<const Frag<T> *>(x + s * 32);
      o.tail[s] = *reinterpret_cast<const f32x8 *>(tail + s * 32);
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if ((wave + 4 * t) * 16 < (int)w.np)
          o.b[t][s] = *reinterpret_cast<const Frag<T> *>(
              static_cast<const T *>(w.bt) +
              ((size_t)chunk * ld + group * w.np + (wave + 4 * t) * 16 + column) * Q + s * 32 + quad * 8);
    }
  };
  auto step = [&](const StateOperands<T, NT> &o, uint32_t chunk) {
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const uint32_t k = (wave + 4 * t) * 16;
      if (k >= w.np) continue;
      typedef T x4 __attribute__((ext_vector_type(4)));
      x4 high, low;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        high[r] = (T)state[t][r];
        low[r] = (T)(state[t][r] - (float)high[r]);
      }
      const uint32_t at = k / 32 * 512 + ((k / 16 % 2 * 2 + quad / 2) * 16 + column) * 8 + quad % 2 * 4;
      *reinterpret_cast<x4 *>(state_block<T>(a, w, chunk, head, 0, v0) + at) = high;
      if (kStatePlanes<T> == 2) *reinterpret_cast<x4 *>(state_block<T>(a, w, chunk, head, 1, v0) + at) = low;
    }
    const float carry = __expf(o.end);
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) state[t][r] *= carry;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      WideFrag<T> fx;
#pragma unroll
      for (int e = 0; e < 8; ++e) fx.set(e, to_f32(o.x[s][e]) * o.tail[s][e]);
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if ((wave + 4 * t) * 16 < (int)w.np) state[t] = mma_wide_b(o.b[t][s], fx, state[t]);
    }
  };

  // operands two chunks ahead
  StateOperands<T, NT> ring[3];
  load(ring[0], 0);
  load(ring[1], min(1u, w.chunks - 1));
  for (uint32_t chunk = 0; chunk < w.chunks; chunk += 3) {
#pragma unroll
    for (int i = 0; i < 3; ++i) {
      if (chunk + i >= w.chunks) break;
      load(ring[(i + 2) % 3], min(chunk + i + 2, w.chunks - 1));
      __builtin_amdgcn_sched_barrier(0);  // the requests stay ahead of the arithmetic
      step(ring[i], chunk + i);
    }
  }
  if (v < a.vdim)
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const uint32_t k = (wave + 4 * t) * 16 + quad * 4 + r;
        if (k < n) saved[k] = state[t][r];
      }
}

// The parallel part: a workgroup per chunk and head, 16 tokens a wave.  y^T of 16 state rows: the incoming
// state against c, scaled by the decay since the chunk's start, and x^T against the weighted scores of the
// chunk's earlier tokens (the skip connection is one more weight on the token's own input).
template <typename T, int STEPS>
__global__ __launch_bounds__(256) void ssm_output_kernel(SsmArgs a, SsmWorkspace w) {
  const uint32_t chunk = blockIdx.x, head = blockIdx.y, group = head / (a.heads / a.groups);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const size_t ld = (size_t)a.groups * w.np;
  const int token = wave * 16 + column;  // of the lane's output column
  const uint32_t row = chunk * Q + token;
  const size_t at = (size_t)chunk * a.heads + head;
  const float *dt = w.dt + at * Q, *sum = w.sum + at * 2 * Q;
  const float *score = w.scores + (((size_t)chunk * a.groups + group) * Q + token) * Q;
  const T *c = static_cast<const T *>(w.c) + (size_t)row * ld + group * w.np + quad * 8;
  const float skip = bf16_at(a.d_skip, head);
  Frag<T> fc[STEPS];
#pragma unroll
  for (int s = 0; s < STEPS; ++s)
    if (s * 32 < (int)w.np) fc[s] = *reinterpret_cast<const Frag<T> *>(c + s * 32);
  const float own_high = sum[token], own_low = sum[Q + token];
  WideFrag<T> weight[2];
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const int j0 = s * 32 + quad * 8;
    const f32x8 sc = *reinterpret_cast<const f32x8 *>(score + j0), d = *reinterpret_cast<const f32x8 *>(dt + j0);
    const f32x8 high = *reinterpret_cast<const f32x8 *>(sum + j0), low = *reinterpret_cast<const f32x8 *>(sum + Q + j0);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float decayed = __expf((own_high - high[e]) + (own_low - low[e])) * d[e];
      const int j = j0 + e;
      weight[s].set(e, j > token ? 0.0f : fmaf(sc[e], decayed, j == token ? skip : 0.0f));
    }
  }
  const float scale = __expf(own_high);
  for (uint32_t v0 = blockIdx.z * 16; v0 < a.vdim; v0 += gridDim.z * 16) {
    const uint32_t v_row = min(v0 + column, a.vdim - 1);
    f32x4 high = {0.0f, 0.0f, 0.0f, 0.0f}, low = high, within = high;
#pragma unroll
    for (int s = 0; s < STEPS; ++s)
      if (s * 32 < (int)w.np) {
        high = mma(reinterpret_cast<const Frag<T> *>(state_block<T>(a, w, chunk, head, 0, v0))[s * 64 + lane], fc[s], high);
        if (kStatePlanes<T> == 2)
          low = mma(reinterpret_cast<const Frag<T> *>(state_block<T>(a, w, chunk, head, 1, v0))[s * 64 + lane], fc[s], low);
      }
    const T *x = static_cast<const T *>(w.xt) + ((size_t)chunk * w.inner + head * a.vdim + v_row) * Q + quad * 8;
#pragma unroll
    for (int s = 0; s < 2; ++s)
      if (s * 32 <= wave * 16 + 15)  // the others come later than all of the wave's tokens
        within = mma_wide_b(*reinterpret_cast<const Frag<T> *>(x + s * 32), weight[s], within);
    if (row >= a.m) continue;
    T *out = static_cast<T *>(a.y) + (size_t)row * w.inner + head * a.vdim + v0 + quad * 4;
    typedef T x4 __attribute__((ext_vector_type(4)));
    x4 y;
#pragma unroll
    for (int r = 0; r < 4; ++r) y[r] = (T)fmaf(scale, high[r] + low[r], within[r]);
    if (a.vdim % 4 == 0) {
      if (v0 + quad * 4 < a.vdim) *reinterpret_cast<x4 *>(out) = y;
    } else {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (v0 + quad * 4 + r < a.vdim) out[r] = y[r];
    }
  }
}

template <typename T, int NT>
hipError_t run_scan(const SsmArgs &a, const SsmWorkspace &w, hipStream_t stream) {
  ssm_state_kernel<T, NT><<<dim3(a.heads, (a.vdim + 15) / 16), 256, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  const uint32_t blocks = (a.vdim + 15) / 16;
  const uint32_t parts = std::min<uint32_t>(blocks, std::max<uint32_t>(1, 1024 / std::max<uint32_t>(1, w.chunks * a.heads)));
  ssm_output_kernel<T, 2 * NT><<<dim3(w.chunks, a.heads, parts), 256, 0, stream>>>(a, w);
  return hipGetLastError();
}

template <typename T>
hipError_t run_prefill(const SsmArgs &a, hipStream_t stream) {
  const SsmWorkspace w = layout(a);
  const uint32_t padded = w.inner + 2 * a.groups * w.np;
  const dim3 conv_grid((padded + 255) / 256, w.chunks * Q / kConvTokens);
  if (a.taps == 4) ssm_conv_kernel<T, 4><<<conv_grid, 256, 0, stream>>>(a, w);
  else if (a.taps == 3) ssm_conv_kernel<T, 3><<<conv_grid, 256, 0, stream>>>(a, w);
  else ssm_conv_kernel<T, 0><<<conv_grid, 256, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  ssm_prepare_kernel<T><<<w.chunks * ((a.heads + 3) / 4) + std::min(a.m, a.taps), 256, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  ssm_scores_kernel<T><<<dim3(w.chunks, a.groups), 256, 0, stream>>>(a, w);
  if (hipError_t status = hipGetLastError()) return status;
  if (w.np <= 64) return run_scan<T, 1>(a, w, stream);
  if (w.np <= 128) return run_scan<T, 2>(a, w, stream);
  if (w.np <= 256) return run_scan<T, 4>(a, w, stream);
  return hipErrorInvalidValue;
}

}  // namespace

size_t ssm_workspace_bytes(const SsmArgs &a) {
  SsmArgs sized = a;
  sized.workspace = nullptr;
  return layout(sized).bytes;
}

hipError_t launch_ssm_step(const SsmArgs &a, hipStream_t stream) {
  const uint32_t rows = a.heads * a.vdim, per = 4 * kStepRows;
  ssm_step_kernel<<<(rows + per - 1) / per, 256, 0, stream>>>(a);
  return hipGetLastError();
}

hipError_t launch_ssm_prefill(const SsmArgs &a, hipStream_t stream) {
  return a.f32 ? run_prefill<float>(a, stream) : run_prefill<__bf16>(a, stream);
}

}  // namespace llmopt
