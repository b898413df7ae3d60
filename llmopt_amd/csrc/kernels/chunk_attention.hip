// Grouped-query attention over chunks of positions or a sliding window, with a tanh cap on the scores and a
// learned sink in the softmax denominator (both optional).
//
//   score(i, j) = cap tanh(scale q_i . k_j / cap),  visible when j <= i and i / chunk == j / chunk,
//                                                   or when 0 <= i - j < window
//   out_i = sum_j exp(score) v_j / (sum_j exp(score) + exp(sink))
//
// Keys and values live in a ring per sequence slot and head: position p in row p % capacity, capacity >=
// chunk or window, so that a ring of one holds everything later tokens can see.
//
//  * chunk_prefill_kernel: a portion of a prompt.  Four waves walk the keys of 64 * QT query rows of one
//    head, 64 keys a stage through LDS; keys before the portion come from the ring, the others from the
//    portion's own rows.  S^T = K Q^T leaves every lane four consecutive keys of one query row, which is
//    the B operand of O^T += V^T P^T up to a permutation of the contraction index that the V^T operand
//    follows: probabilities never leave their lane (bf16: as a high and a low part, so that the weights keep
//    float32 accuracy in the product).  Caps of at most kFixedMaxCap bound the exponent, so
//    the running maximum (and the rescaling) is dropped for a constant one.
//  * chunk_decode_kernel: one token.  A workgroup takes kSplitKeys keys of one key / value head for all
//    query heads on it, which are the operand columns; chunk_merge_kernel joins the splits when the ring is
//    longer than one.  Over a raw float32 row it norms and rotates the group's queries and the token's own
//    key first (in LDS) and leaves key and value in the ring; the own key and value never come from there.
//  * rotate_heads_kernel: the same norm and rotation for a portion of a prompt, in place.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr int kStageKeys = 64;
constexpr uint32_t kSplitKeys = 128;
constexpr float kFixedMaxCap = 40.0f;
constexpr float kLog2e = 1.4426950408889634f;

// The first position that `position` sees; never falls from one position to the next.
__device__ __forceinline__ uint32_t first_seen(uint32_t position, const ChunkCache &cache) {
  if (cache.span == 0) return 0;
  if (cache.sliding) return position + 1 > cache.span ? position + 1 - cache.span : 0;
  return position - position % cache.span;
}

// Values of four keys (rows of the stage) at the lane's column: what the V^T operand takes.  bf16: the
// transposing LDS read - in a group of 16 lanes, lane 4 q + c receives element c of the 8-byte pieces named
// by lanes q, 4 + q, 8 + q and 12 + q, so lane 4 e + q names (key e, columns 4 q ..).
typedef short s16x4 __attribute__((ext_vector_type(4)));
typedef __attribute__((address_space(3))) s16x4 *lds_piece_t;
__device__ __forceinline__ bf16x4 four_keys(const __bf16 *stage, int stride, int lane) {
  const __bf16 *piece = stage + ((lane & 15) >> 2) * stride + (lane & 3) * 4;
  return __builtin_bit_cast(bf16x4, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_piece_t)piece));
}
__device__ __forceinline__ f32x4 four_keys(const float *stage, int stride, int lane) {
  f32x4 v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = stage[i * stride + (lane & 15)];
  return v;
}

__device__ __forceinline__ float exp2_raw(float x) { return __builtin_amdgcn_exp2f(x); }

template <typename T, int NE>
constexpr int value_stride() { return NE * 16 + 32 / (int)sizeof(T); }

template <typename T, int ND, int NE>
constexpr int prefill_lds_bytes() {
  return kStageKeys * (ND * 32 + 16 / (int)sizeof(T) + value_stride<T, NE>()) * (int)sizeof(T);
}

template <typename T, int ND, int NE, int QT, bool FIXED>
__global__ __launch_bounds__(256, ND * 2 + NE <= 16 || sizeof(T) == 2 ? 2 : 1) void chunk_prefill_kernel(ChunkAttentionArgs a) {
  constexpr int DP = ND * 32, EP = NE * 16;
  constexpr int SK = DP + 16 / (int)sizeof(T), SV = value_stride<T, NE>();
  constexpr int K_LOADS = kStageKeys * DP / 8 / 256, V_PIECES = EP / 8;
  constexpr int V_LOADS = (kStageKeys * V_PIECES + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  T *lds_k = reinterpret_cast<T *>(lds);
  T *lds_v = lds_k + kStageKeys * SK;

  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, column = lane & 15, quad = lane >> 4;
  // heads of one key / value head follow each other kv_heads apart, so that they share an XCD's L2 when
  // kv_heads is a multiple of the eight XCDs; the longest rows of all heads come first
  const uint32_t per = a.heads / a.kv_heads, group = blockIdx.x % a.kv_heads;
  const uint32_t head = group * per + blockIdx.x / a.kv_heads;
  const uint32_t tile = gridDim.y - 1 - blockIdx.y;
  const uint32_t p0 = a.state[kStatePosition], slot = a.state[kStateSlot];
  const uint32_t row_first = tile * 64 * QT;
  const uint32_t row_end = min(row_first + 64 * QT, a.m);
  const uint32_t ld = a.ld;
  const T *qkv = static_cast<const T *>(a.qkv);
  const T *fresh_k = qkv + a.heads * a.dim + group * a.dim;
  const T *fresh_v = qkv + a.heads * a.dim + a.kv_heads * a.dim + group * a.vdim;
  const size_t ring = ((size_t)slot * a.kv_heads + group) * a.cache.capacity;
  const T *cache_k = static_cast<const T *>(a.cache.keys) + ring * a.dim;
  const T *cache_v = static_cast<const T *>(a.cache.values) + ring * a.vdim;
  const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0 && ld % 8 == 0;

  // queries of this wave: operand columns
  Frag<T> fq[QT][ND];
  uint32_t low[QT], query[QT];  // visible positions of the lane's row: low .. query
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const uint32_t r = min(row_first + (wave * QT + t) * 16 + column, a.m - 1);
    query[t] = p0 + r;
    low[t] = first_seen(query[t], a.cache);
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      const int k = d * 32 + quad * 8;
      fq[t][d] = load_piece(qkv + (size_t)r * ld + head * a.dim + k, (int)a.dim - k, vec);
    }
  }
  const uint32_t wave_first = p0 + min(row_first + wave * QT * 16, a.m - 1);
  const uint32_t wave_last = p0 + min(row_first + (wave + 1) * QT * 16 - 1, a.m - 1);
  const uint32_t wave_low = first_seen(wave_first, a.cache);
  const uint32_t wave_low_last = first_seen(wave_last, a.cache);

  // Exponents are taken to base two.  capped: score = cap tanh(scale s / cap), with
  // tanh z = 1 - 2 / (1 + e^(2 z)); fixed: the cap bounds it, and the maximum is a constant.
  const bool has_sink = a.sink != nullptr, capped = a.softcap > 0.0f;
  const float sink = has_sink ? (float)reinterpret_cast<const __bf16 *>(a.sink)[head] * kLog2e : 0.0f;
  const float cap = a.softcap * kLog2e;
  const float inner = capped ? 2.0f * a.scale / a.softcap * kLog2e : a.scale * kLog2e;
  float top[QT], total[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    top[t] = has_sink ? (FIXED ? fmaxf(sink, 0.0f) : sink) : (FIXED ? 0.0f : -1e30f);
    total[t] = has_sink && quad == 0 ? exp2_raw(sink - top[t]) : 0.0f;
  }
  f32x4 out[NE][QT];
#pragma unroll
  for (int e = 0; e < NE; ++e)
#pragma unroll
    for (int t = 0; t < QT; ++t) out[e][t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};

  const uint32_t last = p0 + row_end - 1;
  const uint32_t key_begin = first_seen(p0 + row_first, a.cache);

  // a stage travels global -> registers while the one before it is multiplied
  Frag<T> reg_k[K_LOADS], reg_v[V_LOADS];
  auto fetch = [&](uint32_t base) {
#pragma unroll
    for (int i = 0; i < K_LOADS; ++i) {
      const int index = i * 256 + tid, row = index / (DP / 8), piece = (index % (DP / 8)) * 8;
      const uint32_t j = min(base + row, last);
      const T *source = j < p0 ? cache_k + (size_t)(j % a.cache.capacity) * a.dim : fresh_k + (size_t)(j - p0) * ld;
      reg_k[i] = load_piece(source + piece, (int)a.dim - piece, vec);
    }
#pragma unroll
    for (int i = 0; i < V_LOADS; ++i) {
      const int index = i * 256 + tid, row = min(index / V_PIECES, kStageKeys - 1), piece = (index % V_PIECES) * 8;
      const uint32_t j = min(base + row, last);
      const T *source = j < p0 ? cache_v + (size_t)(j % a.cache.capacity) * a.vdim : fresh_v + (size_t)(j - p0) * ld;
      reg_v[i] = load_piece(source + piece, (int)a.vdim - piece, vec);
    }
  };
  auto stash = [&] {
#pragma unroll
    for (int i = 0; i < K_LOADS; ++i) {
      const int index = i * 256 + tid;
      *reinterpret_cast<Frag<T> *>(lds_k + index / (DP / 8) * SK + (index % (DP / 8)) * 8) = reg_k[i];
    }
#pragma unroll
    for (int i = 0; i < V_LOADS; ++i) {
      const int index = i * 256 + tid;
      if (index < kStageKeys * V_PIECES)
        *reinterpret_cast<Frag<T> *>(lds_v + index / V_PIECES * SV + (index % V_PIECES) * 8) = reg_v[i];
    }
  };

  fetch(key_begin);
  for (uint32_t base = key_begin; base <= last; base += kStageKeys) {
    __syncthreads();
    stash();
    __syncthreads();
    if (base + kStageKeys <= last) fetch(base + kStageKeys);
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
      __builtin_amdgcn_sched_barrier(0);  // operands of one key tile at a time: registers
    }
    const bool whole = base >= wave_low_last && base + kStageKeys - 1 <= wave_first;  // no border in this stage
    auto seen = [&](int t, int kt, int r) {
      const uint32_t j = base + kt * 16 + quad * 4 + r;
      return j >= low[t] && j <= query[t];
    };
    if (FIXED) {
#pragma unroll
      for (int t = 0; t < QT; ++t) {
        const float high = cap - top[t];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float tail = __builtin_amdgcn_rcpf(1.0f + exp2_raw(score[kt][t][r] * inner));
            score[kt][t][r] = exp2_raw(fmaf(-2.0f * cap, tail, high));
          }
        if (!whole) {
#pragma unroll
          for (int kt = 0; kt < 4; ++kt)
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (!seen(t, kt, r)) score[kt][t][r] = 0.0f;
        }
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) total[t] += score[kt][t][r];
      }
    } else {
#pragma unroll
      for (int t = 0; t < QT; ++t) {
        float best = top[t];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            float s = score[kt][t][r] * inner;
            if (capped) s = fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + exp2_raw(s)), cap);
            if (!whole && !seen(t, kt, r)) s = -INFINITY;
            score[kt][t][r] = s;
            best = fmaxf(best, s);
          }
        best = fmaxf(best, __shfl_xor(best, 16, 64));
        best = fmaxf(best, __shfl_xor(best, 32, 64));
        const float alpha = exp2_raw(top[t] - best);
        top[t] = best;
        total[t] *= alpha;
#pragma unroll
        for (int e = 0; e < NE; ++e)
#pragma unroll
          for (int r = 0; r < 4; ++r) out[e][t][r] *= alpha;
#pragma unroll
        for (int kt = 0; kt < 4; ++kt)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            score[kt][t][r] = exp2_raw(score[kt][t][r] - best);
            total[t] += score[kt][t][r];
          }
      }
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      WideFrag<T> fp[QT];  // the weights keep float32 accuracy
#pragma unroll
      for (int t = 0; t < QT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          fp[t].set(r, score[2 * ks][t][r]);
          fp[t].set(4 + r, score[2 * ks + 1][t][r]);
        }
#pragma unroll
      for (int e = 0; e < NE; ++e) {
        const T *keys = lds_v + (ks * 32 + quad * 4) * SV + e * 16;
        const auto first = four_keys(keys, SV, lane), second = four_keys(keys + 16 * SV, SV, lane);
        const Frag<T> fv = __builtin_shufflevector(first, second, 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
        for (int t = 0; t < QT; ++t) out[e][t] = mma_wide_b(fv, fp[t], out[e][t]);
        if (e % 4 == 3) __builtin_amdgcn_sched_barrier(0);
      }
    }
  }

#pragma unroll
  for (int t = 0; t < QT; ++t) {
    float sum = total[t];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    const float inverse = a.out_scale / sum;
    const uint32_t r = row_first + (wave * QT + t) * 16 + column;
    if (r >= a.m) continue;
    T *target = static_cast<T *>(a.out) + (size_t)r * a.ld_out + head * a.vdim;
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const uint32_t c = e * 16 + quad * 4;
      typedef T x4 __attribute__((ext_vector_type(4)));
      if (vec && a.ld_out % 4 == 0 && c < a.vdim) {
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
  const T *source = static_cast<const T *>(a.qkv) + (size_t)r * a.ld + a.heads * a.dim;
  T *keys = static_cast<T *>(a.cache.keys), *values = static_cast<T *>(a.cache.values);
  for (uint32_t c = threadIdx.x; c < n_k + n_v; c += 256) {
    if (c < n_k)
      keys[(((size_t)slot * a.kv_heads + c / a.dim) * a.cache.capacity + row) * a.dim + c % a.dim] = source[c];
    else
      values[(((size_t)slot * a.kv_heads + (c - n_k) / a.vdim) * a.cache.capacity + row) * a.vdim + (c - n_k) % a.vdim] =
          source[c];
  }
}

// One token: the query heads of one key / value head are the operand columns (16 at a time), a wave takes 32
// keys of the workgroup's 128; all keys and values of a split are requested before the first is used.  The
// values pass through a wave's own LDS rows on the way to their transposed operand.  Partial results
// [heads][splits][vdim + 2] (weighted sum, maximum, total), or the output when there is one split.
template <typename T, int NE>
constexpr int decode_lds_floats() {
  return 4 * 32 * value_stride<T, NE>() * (int)sizeof(T) / 4 + 2 * 4 * 16;
}

// Cosine and sine of every rotated pair at one position.
struct Turn {
  float cosine, sine;
};
__device__ __forceinline__ void fill_turns(const HeadRotation &r, uint32_t position, Turn *turns) {
  for (uint32_t c = threadIdx.x; c < r.dims / 2; c += 256) turn(position, r.frequencies[c], turns[c].cosine, turns[c].sine);
}

// Norm and rotation of head vectors, a wave a vector, lane l holding components l + 64 i.
template <int PARTS>
struct HeadVector {
  float v[PARTS];
  // exchange(v, partner, half): every rotated component's partner, c + half or c - half.
  template <typename Exchange>
  __device__ __forceinline__ void norm_and_rotate(const HeadRotation &r, const uint16_t *norm, uint32_t dim,
                                                  const Turn *turns, int lane, Exchange exchange) {
    float sum = 0.0f;
#pragma unroll
    for (int i = 0; i < PARTS; ++i) sum += v[i] * v[i];
    const float inverse = 1.0f / sqrtf(wave_sum(sum) / (float)dim + r.epsilon);
    float partner[PARTS];
    const uint32_t half = r.dims / 2;
#pragma unroll
    for (int i = 0; i < PARTS; ++i) {
      const uint32_t c = lane + 64 * i;
      v[i] *= inverse * (c < dim ? (float)reinterpret_cast<const __bf16 *>(norm)[c] : 0.0f);
    }
    exchange(v, partner, half);
#pragma unroll
    for (int i = 0; i < PARTS; ++i) {
      const uint32_t c = lane + 64 * i;
      if (c >= r.dims) continue;
      const Turn t = turns[c < half ? c : c - half];
      v[i] = c < half ? v[i] * t.cosine - partner[i] * t.sine : v[i] * t.cosine + partner[i] * t.sine;
    }
  }
};

// The partner of every rotated component through `row`, floats of the wave's own in LDS.
template <int PARTS>
struct ThroughLds {
  float *row;
  uint32_t dims;
  int lane;
  __device__ __forceinline__ void operator()(const float (&v)[PARTS], float (&partner)[PARTS], uint32_t half) const {
#pragma unroll
    for (int i = 0; i < PARTS; ++i) row[lane + 64 * i] = v[i];
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < PARTS; ++i) {
      const uint32_t c = lane + 64 * i;
      partner[i] = c < dims ? row[c < half ? c + half : c - half] : 0.0f;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // read before the row is written again
    __builtin_amdgcn_wave_barrier();
  }
};

// A workgroup a row; its waves take vectors 0 .. heads + kv_heads - 1 (the queries, then the keys) in turn, the next one
// requested ahead.
template <typename T, int PARTS>
__global__ __launch_bounds__(256) void rotate_heads_kernel(ChunkAttentionArgs a) {
  __shared__ float rows[4][PARTS * 64];
  __shared__ Turn turns[PARTS * 32];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const uint32_t r = blockIdx.x, vectors = a.heads + a.kv_heads;
  T *row = const_cast<T *>(static_cast<const T *>(a.qkv)) + (size_t)r * a.ld;
  T ahead[PARTS];
  auto request = [&](uint32_t vector) {
#pragma unroll
    for (int i = 0; i < PARTS; ++i)
      if (lane + 64 * i < a.dim) ahead[i] = row[(size_t)vector * a.dim + lane + 64 * i];
  };
  request(min((uint32_t)wave, vectors - 1));
  fill_turns(a.rotation, a.state[kStatePosition] + r, turns);
  __syncthreads();
  for (uint32_t vector = wave; vector < vectors; vector += 4) {
    HeadVector<PARTS> h;
#pragma unroll
    for (int i = 0; i < PARTS; ++i) h.v[i] = lane + 64 * i < a.dim ? to_f32(ahead[i]) : 0.0f;
    request(min(vector + 4, vectors - 1));
    h.norm_and_rotate(a.rotation, vector < a.heads ? a.rotation.q_norm : a.rotation.k_norm, a.dim, turns, lane,
                      ThroughLds<PARTS>{rows[wave], a.rotation.dims, lane});
#pragma unroll
    for (int i = 0; i < PARTS; ++i)
      if (lane + 64 * i < a.dim) row[(size_t)vector * a.dim + lane + 64 * i] = (T)h.v[i];
  }
}

// LDS of a decode workgroup that starts from a raw row: queries [16][ND * 32 + pad], the own key, the own
// value, a float row for every wave, the position's turns.
template <typename T, int ND, int NE>
constexpr int raw_row_lds_bytes() {
  return (17 * (ND * 32 + 16 / (int)sizeof(T)) + NE * 16) * (int)sizeof(T) + 4 * (ND <= 2 ? 64 : ND * 32) * 4 +
         ND * 16 * (int)sizeof(Turn);
}

template <typename T, int ND, int NE, bool RAW>
__global__ __launch_bounds__(256) void chunk_decode_kernel(ChunkAttentionArgs a, uint32_t splits) {
  constexpr int EP = NE * 16, SV = value_stride<T, NE>(), V_PIECES = EP / 8;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const uint32_t position = a.state[kStatePosition], slot = a.state[kStateSlot];
  const uint32_t group = blockIdx.x, split = blockIdx.y, per = a.heads / a.kv_heads;
  const uint32_t begin = first_seen(position, a.cache) + split * kSplitKeys;
  if (begin > position) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, column = lane & 15, quad = lane >> 4;
  // a wave's own rows: the values [32][SV], then its sums [16][EP] in their place
  constexpr int OWN = 32 * SV * (int)sizeof(T);
  static_assert(16 * EP * 4 <= OWN, "the sums fit the values' place");
  T *lds_v = reinterpret_cast<T *>(lds + wave * OWN);
  float *lds_top = reinterpret_cast<float *>(lds + 4 * OWN), *lds_total = lds_top + 4 * 16;  // [4][16] each
  const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0;
  const size_t ring = ((size_t)slot * a.kv_heads + group) * a.cache.capacity;
  const T *cache_k = static_cast<const T *>(a.cache.keys) + ring * a.dim;
  const T *cache_v = static_cast<const T *>(a.cache.values) + ring * a.vdim;
  const uint32_t wave_begin = begin + wave * 32;

  Frag<T> fk[2][ND], reg_v[NE];
#pragma unroll
  for (int kt = 0; kt < 2; ++kt) {
    const T *row = cache_k + (size_t)(min(wave_begin + kt * 16 + column, position) % a.cache.capacity) * a.dim;
#pragma unroll
    for (int d = 0; d < ND; ++d) fk[kt][d] = load_piece(row + d * 32 + quad * 8, (int)a.dim - (d * 32 + quad * 8), vec);
  }
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int index = i * 64 + lane, row = index / V_PIECES, piece = (index % V_PIECES) * 8;
    const uint32_t j = min(wave_begin + row, position) % a.cache.capacity;
    reg_v[i] = load_piece(cache_v + (size_t)j * a.vdim + piece, (int)a.vdim - piece, vec);
  }
  const bool capped = a.softcap > 0.0f;
  const float cap = a.softcap * kLog2e;
  const float inner = capped ? 2.0f * a.scale / a.softcap * kLog2e : a.scale * kLog2e;

  // a raw row: the first sixteen queries and the own key and value
  constexpr int SQ = ND * 32 + 16 / (int)sizeof(T), PARTS = ND <= 2 ? 1 : ND / 2;
  T *lds_q = reinterpret_cast<T *>(lds + decode_lds_floats<T, NE>() * 4), *own_k = lds_q + 16 * SQ, *own_v = own_k + SQ;
  float *exchange = reinterpret_cast<float *>(own_v + EP) + wave * PARTS * 64;
  Turn *turns = reinterpret_cast<Turn *>(reinterpret_cast<float *>(own_v + EP) + 4 * PARTS * 64);
  auto stage_vectors = [&](uint32_t h0, uint32_t count, bool key) {
    for (uint32_t n = wave; n < count + (key ? 1 : 0); n += 4) {
      const bool query = n < count;
      const float *source = a.row + (query ? (size_t)(group * per + h0 + n) * a.dim : (size_t)(a.heads + group) * a.dim);
      HeadVector<PARTS> h;
#pragma unroll
      for (int i = 0; i < PARTS; ++i) h.v[i] = lane + 64 * i < a.dim ? source[lane + 64 * i] : 0.0f;
      h.norm_and_rotate(a.rotation, query ? a.rotation.q_norm : a.rotation.k_norm, a.dim, turns, lane,
                        ThroughLds<PARTS>{exchange, a.rotation.dims, lane});
      T *target = query ? lds_q + n * SQ : own_k;
#pragma unroll
      for (int i = 0; i < PARTS; ++i)
        if (lane + 64 * i < ND * 32) target[lane + 64 * i] = (T)h.v[i];  // (zeros behind the head's end)
    }
  };
  if (RAW) {
    fill_turns(a.rotation, position, turns);
    __syncthreads();
    stage_vectors(0, min(16u, per), true);
    const float *value = a.row + (size_t)(a.heads + a.kv_heads) * a.dim + (size_t)group * a.vdim;
    for (uint32_t c = tid; c < EP; c += 256) own_v[c] = (T)(c < a.vdim ? value[c] : 0.0f);
    __syncthreads();
    if (begin + kSplitKeys > position) {  // this workgroup's keys end with the own one
      const size_t at = ring + position % a.cache.capacity;
      for (uint32_t c = tid; c < a.dim; c += 256) static_cast<T *>(a.cache.keys)[at * a.dim + c] = own_k[c];
      for (uint32_t c = tid; c < a.vdim; c += 256) static_cast<T *>(a.cache.values)[at * a.vdim + c] = own_v[c];
    }
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
      if (wave_begin + kt * 16 + column >= position)
#pragma unroll
        for (int d = 0; d < ND; ++d) fk[kt][d] = *reinterpret_cast<const Frag<T> *>(own_k + d * 32 + quad * 8);
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int index = i * 64 + lane;
      if (wave_begin + index / V_PIECES >= position)
        reg_v[i] = *reinterpret_cast<const Frag<T> *>(own_v + (index % V_PIECES) * 8);
    }
  }

  for (uint32_t h0 = 0; h0 < per; h0 += 16) {
    const uint32_t head = group * per + min(h0 + column, per - 1);
    Frag<T> fq[ND];
    if (RAW && h0 > 0) {
      stage_vectors(h0, min(16u, per - h0), false);
      __syncthreads();
    }
#pragma unroll
    for (int d = 0; d < ND; ++d)
      fq[d] = RAW ? *reinterpret_cast<const Frag<T> *>(lds_q + min((uint32_t)column, per - 1 - h0) * SQ + d * 32 + quad * 8)
                  : load_piece(static_cast<const T *>(a.qkv) + (size_t)head * a.dim + d * 32 + quad * 8,
                               (int)a.dim - (d * 32 + quad * 8), vec);
    f32x4 score[2];
    float best = -1e30f;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      score[kt] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
      for (int d = 0; d < ND; ++d) score[kt] = mma(fk[kt][d], fq[d], score[kt]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float s = score[kt][r] * inner;
        if (capped) s = fmaf(-2.0f * cap, __builtin_amdgcn_rcpf(1.0f + exp2_raw(s)), cap);
        if (wave_begin + kt * 16 + quad * 4 + r > position) s = -INFINITY;
        score[kt][r] = s;
        best = fmaxf(best, s);
      }
    }
    best = fmaxf(best, __shfl_xor(best, 16, 64));
    best = fmaxf(best, __shfl_xor(best, 32, 64));
    if (quad == 0) lds_top[wave * 16 + column] = best;
#pragma unroll
    for (int i = 0; i < NE; ++i) {
      const int index = i * 64 + lane;
      *reinterpret_cast<Frag<T> *>(lds_v + index / V_PIECES * SV + (index % V_PIECES) * 8) = reg_v[i];
    }
    __syncthreads();
#pragma unroll
    for (int w = 0; w < 4; ++w) best = fmaxf(best, lds_top[w * 16 + column]);
    WideFrag<T> fp;
    float total = 0.0f;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float p = exp2_raw(score[kt][r] - best);
        total += p;
        fp.set(kt * 4 + r, p);
      }
    total += __shfl_xor(total, 16, 64);
    total += __shfl_xor(total, 32, 64);
    if (quad == 0) lds_total[wave * 16 + column] = total;
    f32x4 out[NE];
#pragma unroll
    for (int e = 0; e < NE; ++e) {
      const T *keys = lds_v + quad * 4 * SV + e * 16;
      const auto first = four_keys(keys, SV, lane), second = four_keys(keys + 16 * SV, SV, lane);
      const Frag<T> fv = __builtin_shufflevector(first, second, 0, 1, 2, 3, 4, 5, 6, 7);
      out[e] = mma_wide_b(fv, fp, f32x4{0.0f, 0.0f, 0.0f, 0.0f});
    }
    __syncthreads();  // every read of the values is done
#pragma unroll
    for (int e = 0; e < NE; ++e)
      *reinterpret_cast<f32x4 *>(lds + wave * OWN + (column * EP + e * 16 + quad * 4) * 4) = out[e];
    __syncthreads();
    const uint32_t live = min(16u, per - h0);
    for (uint32_t i = tid; i < live * EP; i += 256) {
      const uint32_t h = i / EP, c = i % EP;
      if (c >= a.vdim) continue;
      float sum = 0.0f, all = 0.0f, top = -1e30f;
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        sum += *reinterpret_cast<const float *>(lds + w * OWN + (h * EP + c) * 4);
        all += lds_total[w * 16 + h];
        top = fmaxf(top, lds_top[w * 16 + h]);
      }
      const uint32_t target = group * per + h0 + h;
      if (splits == 1) {
        if (a.sink) {
          const float sink = (float)reinterpret_cast<const __bf16 *>(a.sink)[target] * kLog2e, most = fmaxf(top, sink);
          const float mine = exp2_raw(top - most);
          sum *= mine;
          all = all * mine + exp2_raw(sink - most);
        }
        if (a.out_row) a.out_row[target * a.vdim + c] = sum / all * a.out_scale;
        else static_cast<T *>(a.out)[target * a.vdim + c] = (T)(sum / all * a.out_scale);
      } else {
        float *partial = static_cast<float *>(a.workspace) + ((size_t)target * splits + split) * (a.vdim + 2);
        partial[c] = sum;
        if (c == 0) {
          partial[a.vdim] = top;
          partial[a.vdim + 1] = all;
        }
      }
    }
    __syncthreads();
  }
}

// A workgroup a head; the splits' weights are formed once, in LDS (maxima are exponents of two).
template <typename T>
__global__ __launch_bounds__(256) void chunk_merge_kernel(ChunkAttentionArgs a, uint32_t splits) {
  extern __shared__ __attribute__((aligned(16))) float shared[];
  float *best = shared, *total = shared + splits;
  const uint32_t head = blockIdx.x, position = a.state[kStatePosition];
  const uint32_t live = min(splits, (position - first_seen(position, a.cache)) / kSplitKeys + 1);
  const uint32_t stride = a.vdim + 2;
  const float *partial = static_cast<const float *>(a.workspace) + (size_t)head * splits * stride;
  const float sink = a.sink ? (float)reinterpret_cast<const __bf16 *>(a.sink)[head] * kLog2e : -INFINITY;
  constexpr uint32_t AHEAD = 8;
  const uint32_t c = threadIdx.x;
  float first[AHEAD];  // the first splits' values on their way while the weights are formed
#pragma unroll
  for (uint32_t s = 0; s < AHEAD; ++s) first[s] = s < live && c < a.vdim ? partial[s * stride + c] : 0.0f;
  for (uint32_t s = threadIdx.x; s < live; s += 256) {
    best[s] = partial[s * stride + a.vdim];
    total[s] = partial[s * stride + a.vdim + 1];
  }
  __syncthreads();
  float top = sink;
  for (uint32_t s = 0; s < live; ++s) top = fmaxf(top, best[s]);
  float denominator = exp2_raw(sink - top), sum = 0.0f;
#pragma unroll
  for (uint32_t s = 0; s < AHEAD; ++s)
    if (s < live) {
      const float weight = exp2_raw(best[s] - top);
      denominator = fmaf(total[s], weight, denominator);
      sum = fmaf(first[s], weight, sum);
    }
#pragma unroll 8
  for (uint32_t s = AHEAD; s < live; ++s) {
    const float weight = exp2_raw(best[s] - top);
    denominator = fmaf(total[s], weight, denominator);
    if (c < a.vdim) sum = fmaf(partial[s * stride + c], weight, sum);
  }
  if (c >= a.vdim) return;
  if (a.out_row) a.out_row[head * a.vdim + c] = sum / denominator * a.out_scale;
  else static_cast<T *>(a.out)[head * a.vdim + c] = (T)(sum / denominator * a.out_scale);
}

uint32_t decode_splits(const ChunkAttentionArgs &a) {
  const uint32_t longest = a.cache.span ? std::min(a.cache.span, a.cache.capacity) : a.cache.capacity;
  return (longest + kSplitKeys - 1) / kSplitKeys;
}

template <typename T, int ND, int NE, bool RAW>
hipError_t run_decode(const ChunkAttentionArgs &a, hipStream_t stream) {
  static bool allowed[kMaxDevices] = {};
  constexpr int bytes = decode_lds_floats<T, NE>() * 4 + (RAW ? raw_row_lds_bytes<T, ND, NE>() : 0);
  const uint32_t splits = decode_splits(a);
  if (bytes > 64 * 1024)
    if (hipError_t status = allow_dynamic_lds(reinterpret_cast<const void *>(chunk_decode_kernel<T, ND, NE, RAW>), bytes, allowed))
      return status;
  chunk_decode_kernel<T, ND, NE, RAW><<<dim3(a.kv_heads, splits), 256, bytes, stream>>>(a, splits);
  if (hipError_t status = hipGetLastError()) return status;
  if (splits > 1) chunk_merge_kernel<T><<<a.heads, 256, splits * 8, stream>>>(a, splits);
  return hipGetLastError();
}

template <typename T, int ND, int NE, bool FIXED>
hipError_t run_prefill_kernel(const ChunkAttentionArgs &a, hipStream_t stream) {
  constexpr int QT = sizeof(T) == 2 && ND <= 4 && NE <= 8 ? 2 : 1;
  constexpr int bytes = prefill_lds_bytes<T, ND, NE>();
  static bool allowed[kMaxDevices] = {};
  if (bytes > 64 * 1024)
    if (hipError_t status = allow_dynamic_lds(
            reinterpret_cast<const void *>(chunk_prefill_kernel<T, ND, NE, QT, FIXED>), bytes, allowed))
      return status;
  const dim3 grid(a.heads, (a.m + 64 * QT - 1) / (64 * QT));
  chunk_prefill_kernel<T, ND, NE, QT, FIXED><<<grid, 256, bytes, stream>>>(a);
  return hipGetLastError();
}

template <typename T, int ND, int NE>
hipError_t run_prefill(const ChunkAttentionArgs &a, hipStream_t stream) {
  if (a.softcap > 0.0f && a.softcap <= kFixedMaxCap) return run_prefill_kernel<T, ND, NE, true>(a, stream);
  return run_prefill_kernel<T, ND, NE, false>(a, stream);
}

template <typename T, int ND, int NE>
hipError_t run_attention(const ChunkAttentionArgs &a, hipStream_t stream) {
  if (a.m > 1) return run_prefill<T, ND, NE>(a, stream);
  return a.row ? run_decode<T, ND, NE, true>(a, stream) : run_decode<T, ND, NE, false>(a, stream);
}

template <typename T, int ND>
hipError_t pick_value_width(const ChunkAttentionArgs &a, hipStream_t stream) {
  if (a.vdim <= 32) return run_attention<T, ND, 2>(a, stream);
  if (a.vdim <= 64) return run_attention<T, ND, 4>(a, stream);
  if (a.vdim <= 128) return run_attention<T, ND, 8>(a, stream);
  return run_attention<T, ND, 16>(a, stream);
}

template <typename T>
hipError_t pick_attention(const ChunkAttentionArgs &a, hipStream_t stream) {
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
  return a.dim <= 256 && a.vdim <= 256 && decode_splits(a) <= 8000;  // (the merge keeps two words a split in LDS)
}

hipError_t launch_chunk_attention(const ChunkAttentionArgs &a, hipStream_t stream) {
  return a.f32 ? pick_attention<float>(a, stream) : pick_attention<__bf16>(a, stream);
}

hipError_t launch_rotate_heads(const ChunkAttentionArgs &a, hipStream_t stream) {
  const dim3 grid(a.m);
  const int parts = a.dim <= 64 ? 1 : a.dim <= 128 ? 2 : 4;
  auto run = [&](auto kernel) {
    kernel<<<grid, 256, 0, stream>>>(a);
    return hipGetLastError();
  };
  if (a.f32)
    return run(parts == 1 ? rotate_heads_kernel<float, 1> : parts == 2 ? rotate_heads_kernel<float, 2> : rotate_heads_kernel<float, 4>);
  return run(parts == 1 ? rotate_heads_kernel<__bf16, 1> : parts == 2 ? rotate_heads_kernel<__bf16, 2> : rotate_heads_kernel<__bf16, 4>);
}

hipError_t launch_chunk_cache_write(const ChunkAttentionArgs &a, hipStream_t stream) {
  const uint32_t first = a.m > a.cache.capacity ? a.m - a.cache.capacity : 0;
  if (a.f32) chunk_cache_write_kernel<float><<<a.m - first, 256, 0, stream>>>(a, first);
  else chunk_cache_write_kernel<__bf16><<<a.m - first, 256, 0, stream>>>(a, first);
  return hipGetLastError();
}

}  // namespace llmopt
