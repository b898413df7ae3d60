// Grouped-query attention over chunks of positions, with a tanh cap on the scores and a learned sink in
// the softmax denominator.
//
//   score(i, j) = cap tanh(scale q_i . k_j / cap),  visible when j <= i and i / chunk == j / chunk
//   out_i = sum_j exp(score) v_j / (sum_j exp(score) + exp(sink))
//
// Keys and values live in a ring per sequence slot and head: position p in row p % capacity, capacity >=
// chunk, so that a ring of one chunk holds everything later tokens can see.
//
//  * chunk_prefill_kernel: a portion of a prompt.  Four waves walk the keys of 64 * QT query rows of one
//    head, 64 keys a stage through LDS; keys before the portion come from the ring, the others from the
//    portion's own rows.  S^T = K Q^T leaves every lane four consecutive keys of one query row, which is
//    the B operand of O^T += V^T P^T up to a permutation of the contraction index that the V^T operand
//    follows: probabilities never leave their lane.  Caps of at most kFixedMaxCap bound the exponent, so
//    the running maximum (and the rescaling) is dropped for a constant one.
//  * chunk_decode_kernel: one token.  A workgroup takes kSplitKeys keys of one key / value head for all
//    query heads on it; chunk_merge_kernel joins the splits when the ring is longer than one.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr int kStageKeys = 64;
constexpr uint32_t kSplitKeys = 128;
constexpr float kFixedMaxCap = 40.0f;

__device__ __forceinline__ uint32_t chunk_start(uint32_t position, uint32_t chunk) {
  return chunk ? position - position % chunk : 0;
}

__device__ __forceinline__ float capped(float s, float scale, float cap, float inverse_cap) {
  s *= scale;
  return cap > 0.0f ? cap * tanh_f32(s * inverse_cap) : s;
}

template <typename T, int ND, int NE, int QT>
__global__ __launch_bounds__(256) void chunk_prefill_kernel(ChunkAttentionArgs a) {
  constexpr int DP = ND * 32, EP = NE * 16;
  constexpr int PAD = 16 / (int)sizeof(T);
  constexpr int SK = DP + PAD, SV = kStageKeys + PAD;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  T *lds_k = reinterpret_cast<T *>(lds);
  T *lds_v = lds_k + kStageKeys * SK;  // [EP][SV], transposed

  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, column = lane & 15, quad = lane >> 4;
  const uint32_t head = blockIdx.y, group = head / (a.heads / a.kv_heads);
  const uint32_t tile = gridDim.x - 1 - blockIdx.x;  // longest rows first
  const uint32_t p0 = a.state[kStatePosition], slot = a.state[kStateSlot];
  const uint32_t row_first = tile * 64 * QT;
  const uint32_t row_end = min(row_first + 64 * QT, a.m);
  const uint32_t ld = a.heads * a.dim + a.kv_heads * (a.dim + a.vdim);
  const T *qkv = static_cast<const T *>(a.qkv);
  const T *fresh_k = qkv + a.heads * a.dim + group * a.dim;
  const T *fresh_v = qkv + a.heads * a.dim + a.kv_heads * a.dim + group * a.vdim;
  const size_t ring = ((size_t)slot * a.kv_heads + group) * a.cache.capacity;
  const T *cache_k = static_cast<const T *>(a.cache.keys) + ring * a.dim;
  const T *cache_v = static_cast<const T *>(a.cache.values) + ring * a.vdim;
  const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0;

  // queries of this wave: operand columns
  Frag<T> fq[QT][ND];
  uint32_t low[QT], query[QT];  // visible positions of the lane's row: low .. query
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const uint32_t r = min(row_first + (wave * QT + t) * 16 + column, a.m - 1);
    query[t] = p0 + r;
    low[t] = chunk_start(query[t], a.cache.chunk);
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      const int k = d * 32 + quad * 8;
      fq[t][d] = load_piece(qkv + (size_t)r * ld + head * a.dim + k, (int)a.dim - k, vec);
    }
  }
  const uint32_t wave_last = p0 + min(row_first + (wave + 1) * QT * 16 - 1, a.m - 1);
  const uint32_t wave_low = chunk_start(p0 + min(row_first + wave * QT * 16, a.m - 1), a.cache.chunk);

  const bool has_sink = a.sink != nullptr;
  const float sink = has_sink ? (float)reinterpret_cast<const __bf16 *>(a.sink)[head] : 0.0f;
  const bool fixed = a.softcap > 0.0f && a.softcap <= kFixedMaxCap;
  const float inverse_cap = a.softcap > 0.0f ? 1.0f / a.softcap : 0.0f;
  float top[QT], total[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    top[t] = has_sink ? (fixed ? fmaxf(sink, 0.0f) : sink) : (fixed ? 0.0f : -1e30f);
    total[t] = has_sink && quad == 0 ? __expf(sink - top[t]) : 0.0f;
  }
  f32x4 out[NE][QT];
#pragma unroll
  for (int e = 0; e < NE; ++e)
#pragma unroll
    for (int t = 0; t < QT; ++t) out[e][t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};

  const uint32_t last = p0 + row_end - 1;
  const uint32_t key_begin = chunk_start(p0 + row_first, a.cache.chunk);
  for (uint32_t base = key_begin; base <= last; base += kStageKeys) {
    __syncthreads();
#pragma unroll
    for (int i = 0; i < ND; ++i) {
      const int index = i * 256 + tid, row = index / (ND * 4), piece = (index % (ND * 4)) * 8;
      const uint32_t j = min(base + row, last);
      const T *source = j < p0 ? cache_k + (size_t)(j % a.cache.capacity) * a.dim : fresh_k + (size_t)(j - p0) * ld;
      *reinterpret_cast<Frag<T> *>(lds_k + row * SK + piece) = load_piece(source + piece, (int)a.dim - piece, vec);
    }
#pragma unroll
    for (int i = 0; i < (NE + 3) / 4; ++i) {
      const int index = i * 256 + tid, pair = index & 31, piece = (index >> 5) * 8;
      if (piece < EP) {
        Frag<T> two[2];
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          const uint32_t j = min(base + pair * 2 + h, last);
          const T *source =
              j < p0 ? cache_v + (size_t)(j % a.cache.capacity) * a.vdim : fresh_v + (size_t)(j - p0) * ld;
          two[h] = load_piece(source + piece, (int)a.vdim - piece, vec);
        }
        typedef T x2 __attribute__((ext_vector_type(2)));
#pragma unroll
        for (int e = 0; e < 8; ++e)
          *reinterpret_cast<x2 *>(lds_v + (piece + e) * SV + pair * 2) = x2{two[0][e], two[1][e]};
      }
    }
    __syncthreads();
    if (base > wave_last || base + kStageKeys <= wave_low) continue;

    f32x4 score[4][QT];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
      for (int t = 0; t < QT; ++t) score[kt][t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int d = 0; d < ND; ++d) {
        const Frag<T> fk = *reinterpret_cast<const Frag<T> *>(lds_k + (kt * 16 + column) * SK + d * 32 + quad * 8);
#pragma unroll
        for (int t = 0; t < QT; ++t) score[kt][t] = mma(fk, fq[t][d], score[kt][t]);
      }
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      float best = top[t];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const uint32_t j = base + kt * 16 + quad * 4 + r;
          const bool seen = j >= low[t] && j <= query[t];
          const float s = seen ? capped(score[kt][t][r], a.scale, a.softcap, inverse_cap) : -INFINITY;
          score[kt][t][r] = s;
          if (!fixed) best = fmaxf(best, s);
        }
      if (!fixed) {
        best = fmaxf(best, __shfl_xor(best, 16, 64));
        best = fmaxf(best, __shfl_xor(best, 32, 64));
        const float alpha = __expf(top[t] - best);
        top[t] = best;
        total[t] *= alpha;
#pragma unroll
        for (int e = 0; e < NE; ++e)
#pragma unroll
          for (int r = 0; r < 4; ++r) out[e][t][r] *= alpha;
      }
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float p = __expf(score[kt][t][r] - top[t]);
          score[kt][t][r] = p;
          total[t] += p;
        }
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      Frag<T> fp[QT];
#pragma unroll
      for (int t = 0; t < QT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          fp[t][r] = (T)score[2 * ks][t][r];
          fp[t][4 + r] = (T)score[2 * ks + 1][t][r];
        }
#pragma unroll
      for (int e = 0; e < NE; ++e) {
        typedef T x4 __attribute__((ext_vector_type(4)));
        const T *row = lds_v + (e * 16 + column) * SV + ks * 32 + quad * 4;
        const x4 first = *reinterpret_cast<const x4 *>(row), second = *reinterpret_cast<const x4 *>(row + 16);
        const Frag<T> fv = __builtin_shufflevector(first, second, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
        for (int t = 0; t < QT; ++t) out[e][t] = mma(fv, fp[t], out[e][t]);
      }
    }
  }

#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float sum = total[t];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    const float inverse = 1.0f / sum;
    const uint32_t r = row_first + (wave * QT + t) * 16 + column;
    if (r >= a.m) continue;
    T *target = static_cast<T *>(a.out) + (size_t)r * a.heads * a.vdim + head * a.vdim;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const uint32_t c = e * 16 + quad * 4;
      typedef T x4 __attribute__((ext_vector_type(4)));
      if (vec && c < a.vdim) {
        x4 packed;
#pragma unroll
        for (int i = 0; i < 4; ++i) packed[i] = (T)(out[e][t][i] * inverse);
        *reinterpret_cast<x4 *>(target + c) = packed;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (c + i < a.vdim) target[c + i] = (T)(out[e][t][i] * inverse);
      }
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void chunk_cache_write_kernel(ChunkAttentionArgs a, uint32_t first_row) {
  const uint32_t r = first_row + blockIdx.x;
  const uint32_t position = a.state[kStatePosition] + r, slot = a.state[kStateSlot];
  const uint32_t row = position % a.cache.capacity;
  const uint32_t n_k = a.kv_heads * a.dim, n_v = a.kv_heads * a.vdim;
  const T *source = static_cast<const T *>(a.qkv) + (size_t)r * (a.heads * a.dim + n_k + n_v) + a.heads * a.dim;
  T *keys = static_cast<T *>(a.cache.keys), *values = static_cast<T *>(a.cache.values);
  for (uint32_t c = threadIdx.x; c < n_k + n_v; c += 256) {
    if (c < n_k)
      keys[(((size_t)slot * a.kv_heads + c / a.dim) * a.cache.capacity + row) * a.dim + c % a.dim] = source[c];
    else
      values[(((size_t)slot * a.kv_heads + (c - n_k) / a.vdim) * a.cache.capacity + row) * a.vdim + (c - n_k) % a.vdim] =
          source[c];
  }
}

// PIECES: 64-wide parts of a key row.  Partial results [heads][splits][vdim + 2] (sum, maximum, total).
template <typename T, int PIECES>
__global__ __launch_bounds__(256) void chunk_decode_kernel(ChunkAttentionArgs a, uint32_t splits) {
  extern __shared__ __attribute__((aligned(16))) float shared[];
  const uint32_t position = a.state[kStatePosition], slot = a.state[kStateSlot];
  const uint32_t group = blockIdx.x, split = blockIdx.y, per = a.heads / a.kv_heads;
  const uint32_t low = chunk_start(position, a.cache.chunk);
  const uint32_t begin = low + split * kSplitKeys;
  if (begin > position) return;
  const uint32_t keys = min(kSplitKeys, position + 1 - begin);
  const uint32_t dim8 = (a.dim + 7) & ~7u;
  float *q = shared;                    // [per][dim8]
  float *scores = q + per * dim8;       // [per][kSplitKeys]
  float *stats = scores + per * kSplitKeys;  // [per][2]
  float *reduce = stats + 2 * per;      // [256][9]
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0;
  const size_t ring = ((size_t)slot * a.kv_heads + group) * a.cache.capacity;
  const T *cache_k = static_cast<const T *>(a.cache.keys) + ring * a.dim;
  const T *cache_v = static_cast<const T *>(a.cache.values) + ring * a.vdim;

  // eight lanes a key, 32 keys a pass; all of a split's keys are requested at once
  const int sub = tid & 7;
  Frag<T> k[kSplitKeys / 32][PIECES];
#pragma unroll
  for (int pass = 0; pass < (int)kSplitKeys / 32; ++pass) {
    const uint32_t j = begin + min((uint32_t)(pass * 32 + (tid >> 3)), keys - 1);
    const T *row = cache_k + (size_t)(j % a.cache.capacity) * a.dim;
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
      const int c = (p * 8 + sub) * 8;
      k[pass][p] = load_piece(row + c, (int)a.dim - c, vec);
    }
  }
  for (uint32_t i = tid; i < per * dim8; i += 256) {
    const uint32_t h = i / dim8, c = i % dim8;
    q[i] = c < a.dim ? to_f32(static_cast<const T *>(a.qkv)[(group * per + h) * a.dim + c]) : 0.0f;
  }
  __syncthreads();
  const float inverse_cap = a.softcap > 0.0f ? 1.0f / a.softcap : 0.0f;
  for (uint32_t h = 0; h < per; ++h) {
    float dot[kSplitKeys / 32];
#pragma unroll
    for (int pass = 0; pass < (int)kSplitKeys / 32; ++pass) dot[pass] = 0.0f;
#pragma unroll
    for (int p = 0; p < PIECES; ++p) {
      const uint32_t c = (p * 8 + sub) * 8;
      if (c >= dim8) continue;
      const f32x4 lo = *reinterpret_cast<const f32x4 *>(q + h * dim8 + c);
      const f32x4 hi = *reinterpret_cast<const f32x4 *>(q + h * dim8 + c + 4);
#pragma unroll
      for (int pass = 0; pass < (int)kSplitKeys / 32; ++pass)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          dot[pass] = fmaf(to_f32(k[pass][p][e]), lo[e], dot[pass]);
          dot[pass] = fmaf(to_f32(k[pass][p][4 + e]), hi[e], dot[pass]);
        }
    }
#pragma unroll
    for (int pass = 0; pass < (int)kSplitKeys / 32; ++pass) {
      float s = dot[pass];
      s += __shfl_xor(s, 1, 64);
      s += __shfl_xor(s, 2, 64);
      s += __shfl_xor(s, 4, 64);
      const uint32_t index = pass * 32 + (tid >> 3);
      if (sub == 0)
        scores[h * kSplitKeys + index] = index < keys ? capped(s, a.scale, a.softcap, inverse_cap) : -INFINITY;
    }
  }
  __syncthreads();
  for (uint32_t h = wave; h < per; h += 4) {
    float *row = scores + h * kSplitKeys;
    const float s0 = row[lane], s1 = row[64 + lane];
    const float best = wave_max(fmaxf(s0, s1));
    const float e0 = __expf(s0 - best), e1 = __expf(s1 - best);
    row[lane] = e0;
    row[64 + lane] = e1;
    const float sum = wave_sum(e0 + e1);
    if (lane == 0) {
      stats[2 * h] = best;
      stats[2 * h + 1] = sum;
    }
  }
  __syncthreads();
  const uint32_t pieces = (a.vdim + 7) / 8, subsets = 256 / pieces;
  const uint32_t piece = tid % pieces, subset = tid / pieces;
  constexpr int HEADS = 4;
  for (uint32_t h0 = 0; h0 < per; h0 += HEADS) {
    float acc[HEADS][8];
#pragma unroll
    for (int h = 0; h < HEADS; ++h)
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[h][e] = 0.0f;
    if (subset < subsets)
#pragma unroll 4
      for (uint32_t i = subset; i < keys; i += subsets) {
        const T *row = cache_v + (size_t)((begin + i) % a.cache.capacity) * a.vdim;
        const Frag<T> v = load_piece(row + piece * 8, (int)a.vdim - (int)piece * 8, vec);
#pragma unroll
        for (int h = 0; h < HEADS; ++h) {
          const float p = scores[min(h0 + h, per - 1) * kSplitKeys + i];
#pragma unroll
          for (int e = 0; e < 8; ++e) acc[h][e] = fmaf(p, to_f32(v[e]), acc[h][e]);
        }
      }
#pragma unroll
    for (int h = 0; h < HEADS; ++h) {
      if (h0 + h >= per) break;
      const uint32_t head = group * per + h0 + h;
      __syncthreads();
#pragma unroll
      for (int e = 0; e < 8; ++e) reduce[tid * 9 + e] = acc[h][e];
      __syncthreads();
      for (uint32_t c = tid; c < a.vdim; c += 256) {
        float sum = 0.0f;
        for (uint32_t s = 0; s < subsets; ++s) sum += reduce[(s * pieces + c / 8) * 9 + c % 8];
        const float best = stats[2 * (h0 + h)], total = stats[2 * (h0 + h) + 1];
        if (splits == 1) {
          const float sink = a.sink ? (float)reinterpret_cast<const __bf16 *>(a.sink)[head] : -INFINITY;
          const float top = fmaxf(best, sink);
          const float mine = __expf(best - top);
          static_cast<T *>(a.out)[head * a.vdim + c] = (T)(sum * mine / (total * mine + __expf(sink - top)));
        } else {
          float *partial = static_cast<float *>(a.workspace) + ((size_t)head * splits + split) * (a.vdim + 2);
          partial[c] = sum;
          if (c == 0) {
            partial[a.vdim] = best;
            partial[a.vdim + 1] = total;
          }
        }
      }
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void chunk_merge_kernel(ChunkAttentionArgs a, uint32_t splits) {
  const uint32_t head = blockIdx.x, position = a.state[kStatePosition];
  const uint32_t live = min(splits, (position - chunk_start(position, a.cache.chunk)) / kSplitKeys + 1);
  const uint32_t stride = a.vdim + 2;
  const float *partial = static_cast<const float *>(a.workspace) + (size_t)head * splits * stride;
  const float sink = a.sink ? (float)reinterpret_cast<const __bf16 *>(a.sink)[head] : -INFINITY;
  float top = sink;
  for (uint32_t s = 0; s < live; ++s) top = fmaxf(top, partial[s * stride + a.vdim]);
  float total = __expf(sink - top);
  for (uint32_t s = 0; s < live; ++s)
    total += partial[s * stride + a.vdim + 1] * __expf(partial[s * stride + a.vdim] - top);
  for (uint32_t c = threadIdx.x; c < a.vdim; c += 256) {
    float sum = 0.0f;
    for (uint32_t s = 0; s < live; ++s)
      sum = fmaf(partial[s * stride + c], __expf(partial[s * stride + a.vdim] - top), sum);
    static_cast<T *>(a.out)[head * a.vdim + c] = (T)(sum / total);
  }
}

uint32_t decode_splits(const ChunkAttentionArgs &a) {
  const uint32_t longest = a.cache.chunk ? std::min(a.cache.chunk, a.cache.capacity) : a.cache.capacity;
  return (longest + kSplitKeys - 1) / kSplitKeys;
}

uint32_t decode_lds_bytes(const ChunkAttentionArgs &a) {
  const uint32_t per = a.heads / a.kv_heads, dim8 = (a.dim + 7) & ~7u;
  return (per * dim8 + per * kSplitKeys + 2 * per + 256 * 9) * 4;
}

template <typename T, int PIECES>
hipError_t run_decode(const ChunkAttentionArgs &a, hipStream_t stream) {
  static bool allowed[kMaxDevices] = {};
  const uint32_t splits = decode_splits(a), bytes = decode_lds_bytes(a);
  if (bytes > 64 * 1024)
    if (hipError_t status = allow_dynamic_lds(reinterpret_cast<const void *>(chunk_decode_kernel<T, PIECES>),
                                              160 * 1024, allowed))
      return status;
  chunk_decode_kernel<T, PIECES><<<dim3(a.kv_heads, splits), 256, bytes, stream>>>(a, splits);
  if (hipError_t status = hipGetLastError()) return status;
  if (splits > 1) chunk_merge_kernel<T><<<a.heads, 256, 0, stream>>>(a, splits);
  return hipGetLastError();
}

template <typename T, int ND, int NE>
hipError_t run_prefill(const ChunkAttentionArgs &a, hipStream_t stream) {
  constexpr int QT = sizeof(T) == 2 && ND <= 4 && NE <= 8 ? 2 : 1;
  constexpr int PAD = 16 / (int)sizeof(T);
  constexpr int bytes = (kStageKeys * (ND * 32 + PAD) + NE * 16 * (kStageKeys + PAD)) * (int)sizeof(T);
  static bool allowed[kMaxDevices] = {};
  if (bytes > 64 * 1024)
    if (hipError_t status = allow_dynamic_lds(reinterpret_cast<const void *>(chunk_prefill_kernel<T, ND, NE, QT>),
                                              bytes, allowed))
      return status;
  const dim3 grid((a.m + 64 * QT - 1) / (64 * QT), a.heads);
  chunk_prefill_kernel<T, ND, NE, QT><<<grid, 256, bytes, stream>>>(a);
  return hipGetLastError();
}

template <typename T, int ND>
hipError_t pick_value_width(const ChunkAttentionArgs &a, hipStream_t stream) {
  if (a.vdim <= 32) return run_prefill<T, ND, 2>(a, stream);
  if (a.vdim <= 64) return run_prefill<T, ND, 4>(a, stream);
  if (a.vdim <= 128) return run_prefill<T, ND, 8>(a, stream);
  return run_prefill<T, ND, 16>(a, stream);
}

template <typename T>
hipError_t pick_attention(const ChunkAttentionArgs &a, hipStream_t stream) {
  if (a.m == 1) {
    if (a.dim <= 64) return run_decode<T, 1>(a, stream);
    if (a.dim <= 128) return run_decode<T, 2>(a, stream);
    return run_decode<T, 4>(a, stream);
  }
  if (a.dim <= 64) return pick_value_width<T, 2>(a, stream);
  if (a.dim <= 128) return pick_value_width<T, 4>(a, stream);
  return pick_value_width<T, 8>(a, stream);
}

}  // namespace

size_t chunk_attention_workspace_bytes(const ChunkAttentionArgs &a) {
  if (a.m != 1) return 0;
  const uint32_t splits = decode_splits(a);
  return splits > 1 ? (size_t)a.heads * splits * (a.vdim + 2) * 4 : 0;
}

bool chunk_attention_ok(const ChunkAttentionArgs &a) {
  return a.dim <= 256 && a.vdim <= 256 && decode_lds_bytes(a) <= 160 * 1024;
}

hipError_t launch_chunk_attention(const ChunkAttentionArgs &a, hipStream_t stream) {
  return a.f32 ? pick_attention<float>(a, stream) : pick_attention<__bf16>(a, stream);
}

hipError_t launch_chunk_cache_write(const ChunkAttentionArgs &a, hipStream_t stream) {
  const uint32_t first = a.m > a.cache.capacity ? a.m - a.cache.capacity : 0;
  if (a.f32) chunk_cache_write_kernel<float><<<a.m - first, 256, 0, stream>>>(a, first);
  else chunk_cache_write_kernel<__bf16><<<a.m - first, 256, 0, stream>>>(a, first);
  return hipGetLastError();
}

}  // namespace llmopt
