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
//  * ssm_scan_kernel: a workgroup owns 16 state rows of one head and walks the chunks, its slice of the
//    state in registers.  Operands that must keep float32 accuracy (the state, the decay-weighted
//    inputs) enter the bfloat16 matrix cores as a high and a low part.
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

// What a wave reads of one chunk, requested a chunk ahead.
template <typename T, int NT>
struct ChunkOperands {
  Frag<T> c[2 * NT];     // c rows of the wave's 16 tokens, np / 32 steps (np <= 64 NT)
  Frag<T> x[2];          // x^T of the 16 state rows, 32 tokens each
  Frag<T> b[NT][2];      // b^T of the wave's state columns
  f32x8 score[2], dt[2], tail[2], high[2];
  f32x8 low[sizeof(T) == 4 ? 2 : 1];  // bf16 does without the running sums' low parts
  float own_high, own_low, end;
};

// NT: 16-column tiles of the state a wave owns (state_size <= 64 NT).
template <typename T, int NT>
__global__ __launch_bounds__(256, 1) void ssm_scan_kernel(SsmArgs a, SsmWorkspace w) {
  constexpr int STRIDE = 64 * NT + 4;
  __shared__ __attribute__((aligned(16))) float states[2][16 * STRIDE];
  const uint32_t head = blockIdx.x, v0 = blockIdx.y * 16, group = head / (a.heads / a.groups);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, column = lane & 15, quad = lane >> 4;
  const uint32_t n = a.state_size, slot = a.step[kStateSlot];
  const bool fresh = a.step[kStatePosition] == 0;
  const size_t ld = (size_t)a.groups * w.np;
  const int token = wave * 16 + column;  // the token of the lane's output column
  // state rows beyond the head's end repeat its last one and are not stored
  const uint32_t v_row = min(v0 + column, a.vdim - 1);
  float *saved = a.ssm_state + ((size_t)slot * a.heads + head) * a.vdim * n;
  const float skip = bf16_at(a.d_skip, head);

  f32x4 state[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t v = v0 + quad * 4 + r, k = (wave + 4 * t) * 16 + column;
      state[t][r] = !fresh && v < a.vdim && k < n ? saved[(size_t)v * n + k] : 0.0f;
    }

  auto load = [&](ChunkOperands<T, NT> &o, uint32_t chunk) {
    const T *c = static_cast<const T *>(w.c) + ((size_t)chunk * Q + token) * ld + group * w.np + quad * 8;
#pragma unroll
    for (int s = 0; s < 2 * NT; ++s)
      if (s * 32 < (int)w.np) o.c[s] = *reinterpret_cast<const Frag<T> *>(c + s * 32);
    const T *x = static_cast<const T *>(w.xt) + ((size_t)chunk * w.inner + head * a.vdim + v_row) * Q + quad * 8;
    const float *score = w.scores + (((size_t)chunk * a.groups + group) * Q + token) * Q + quad * 8;
    const float *dt = w.dt + ((size_t)chunk * a.heads + head) * Q;
    const float *tail = w.tail + ((size_t)chunk * a.heads + head) * Q;
    const float *sum = w.sum + ((size_t)chunk * a.heads + head) * 2 * Q;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      o.x[s] = *reinterpret_cast<const Frag<T> *>(x + s * 32);
      o.score[s] = *reinterpret_cast<const f32x8 *>(score + s * 32);
      o.dt[s] = *reinterpret_cast<const f32x8 *>(dt + s * 32 + quad * 8);
      o.tail[s] = *reinterpret_cast<const f32x8 *>(tail + s * 32 + quad * 8);
      o.high[s] = *reinterpret_cast<const f32x8 *>(sum + s * 32 + quad * 8);
      if (sizeof(T) == 4) o.low[s] = *reinterpret_cast<const f32x8 *>(sum + Q + s * 32 + quad * 8);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const uint32_t k = (wave + 4 * t) * 16 + column;
        if ((wave + 4 * t) * 16 < (int)w.np)
          o.b[t][s] = *reinterpret_cast<const Frag<T> *>(
              static_cast<const T *>(w.bt) + ((size_t)chunk * ld + group * w.np + k) * Q + s * 32 + quad * 8);
      }
    }
    o.own_high = sum[token];
    o.own_low = sum[Q + token];
    o.end = sum[Q - 1];
  };

  auto step = [&](const ChunkOperands<T, NT> &o, uint32_t chunk) {
    float *lds = states[chunk & 1];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) lds[(quad * 4 + r) * STRIDE + (wave + 4 * t) * 16 + column] = state[t][r];
    __syncthreads();
    // y^T: rows = state rows, column = the lane's token
    f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
    for (int s = 0; s < 2 * NT; ++s)
      if (s * 32 < (int)w.np) {
        WideFrag<T> fs;
        const float *row = lds + column * STRIDE + s * 32 + quad * 8;
        const f32x4 lo = *reinterpret_cast<const f32x4 *>(row), hi = *reinterpret_cast<const f32x4 *>(row + 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          fs.set(e, lo[e]);
          fs.set(4 + e, hi[e]);
        }
        y = mma_wide(fs, o.c[s], y);
      }
    const float scale = __expf(o.own_high);
#pragma unroll
    for (int r = 0; r < 4; ++r) y[r] *= scale;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      if (s * 32 > wave * 16 + 15) continue;  // all of these tokens come later
      WideFrag<T> fp;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int j = s * 32 + quad * 8 + e;
        const float weight = __expf(sizeof(T) == 4 ? (o.own_high - o.high[s][e]) + (o.own_low - o.low[s][e])
                                              : o.own_high - o.high[s][e]) * o.dt[s][e];
        // the skip connection is one more weight on the token's own input
        fp.set(e, j > token ? 0.0f : fmaf(o.score[s][e], weight, j == token ? skip : 0.0f));
      }
      y = mma_wide_b(o.x[s], fp, y);
    }
    // the new state
    const float carry = __expf(o.end);
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) state[t][r] *= carry;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      WideFrag<T> fx;
#pragma unroll
      for (int e = 0; e < 8; ++e)
        fx.set(e, to_f32(o.x[s][e]) * o.tail[s][e]);
#pragma unroll
      for (int t = 0; t < NT; ++t)
        if ((wave + 4 * t) * 16 < (int)w.np) state[t] = mma_wide(fx, o.b[t][s], state[t]);
    }
    const uint32_t row = chunk * Q + token;
    if (row < a.m) {
      T *out = static_cast<T *>(a.y) + (size_t)row * w.inner + head * a.vdim;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const uint32_t v = v0 + quad * 4 + r;
        if (v < a.vdim) out[v] = (T)y[r];
      }
    }
  };

  ChunkOperands<T, NT> even, odd;
  load(even, 0);
  for (uint32_t chunk = 0; chunk < w.chunks; chunk += 2) {
    if (chunk + 1 < w.chunks) load(odd, chunk + 1);
    __builtin_amdgcn_sched_barrier(0);  // the requests stay ahead of the arithmetic
    step(even, chunk);
    if (chunk + 1 < w.chunks) {
      if (chunk + 2 < w.chunks) load(even, chunk + 2);
      __builtin_amdgcn_sched_barrier(0);
      step(odd, chunk + 1);
    }
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t v = v0 + quad * 4 + r, k = (wave + 4 * t) * 16 + column;
      if (v < a.vdim && k < n) saved[(size_t)v * n + k] = state[t][r];
    }
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
  const dim3 grid(a.heads, (a.vdim + 15) / 16);
  if (w.np <= 64) ssm_scan_kernel<T, 1><<<grid, 256, 0, stream>>>(a, w);
  else if (w.np <= 128) ssm_scan_kernel<T, 2><<<grid, 256, 0, stream>>>(a, w);
  else if (w.np <= 256) ssm_scan_kernel<T, 4><<<grid, 256, 0, stream>>>(a, w);
  else return hipErrorInvalidValue;
  return hipGetLastError();
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
