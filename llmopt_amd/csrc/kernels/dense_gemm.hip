// Matrix product of many activation rows with bfloat16 weights on the matrix cores, and the small
// row-wise kernels around it (norm, embedding).
//
//   out[r, c] = sum_k x[r, k] w[c, k]       x [m, k] bf16 or f32, w bf16 [n, k], sums in float32
//
// A workgroup owns a BM x BN tile and walks K in stages of 64 staged in LDS (dense_gemm_direct_kernel for
// bf16 rows of whole stages, dense_gemm_kernel through registers for the rest).  The weights are the A
// operand and the activations the B operand: a lane then ends with four consecutive output columns of one
// row, and the epilogue stores 8 or 16 bytes at a time.
//
//  * gated: the 16-column groups of a tile alternate between the gate and the up matrix, so that both
//    values of an output element meet in one lane.
//  * routed: a tile belongs to one expert; its rows are gathered (or taken in place) from the order the
//    route plan made, and tiles that the plan did not fill end at once.
//  * workgroups are dealt to the XCDs in contiguous runs (blockIdx % 8 is the XCD), and inside a run
//    eight row tiles share a column of weight tiles: both operands are re-read from that XCD's L2.
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

constexpr int kStageK = 64;

struct GemmParams {
  DenseLinearArgs a;
  uint32_t tiles_m, tiles_n, total, per_xcd;
};

template <typename T>
constexpr int lds_stride() { return kStageK + 16 / (int)sizeof(T); }

template <typename T, int BM, int BN>
constexpr int gemm_lds_bytes() {
  return 2 * (BM * lds_stride<T>() * (int)sizeof(T) + BN * lds_stride<__bf16>() * 2);
}

template <typename T>
__device__ __forceinline__ void store4(T *out, f32x4 v, uint32_t count, bool vec) {
  if (vec && count >= 4) {
    typedef T x4 __attribute__((ext_vector_type(4)));
    x4 packed;
#pragma unroll
    for (int i = 0; i < 4; ++i) packed[i] = (T)v[i];
    *reinterpret_cast<x4 *>(out) = packed;
    return;
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (i < (int)count) out[i] = (T)v[i];
}

// kQkv: value columns of row r mixed with (or kept for) other layers.
__device__ __forceinline__ void mix_values(const DenseLinearArgs &a, uint32_t r, uint32_t c, f32x4 &v) {
  if (a.mix.mode == 0 || c + 3 < a.split) return;
  const uint32_t n_v = a.n - a.split;
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (c + i < a.n && c + i >= a.split) {
      float *first = a.mix.v_first + (size_t)r * n_v + (c + i - a.split);
      if (a.mix.mode == 1) *first = v[i];
      else v[i] = (1.0f - a.mix.lambda) * v[i] + a.mix.lambda * *first;
    }
}

// Four results of row r, columns c .. c + 3 (those below n).
template <typename T>
__device__ __forceinline__ void emit(const DenseLinearArgs &a, uint32_t r, uint32_t c, f32x4 v) {
  const uint32_t count = a.n - c;
  switch (a.epilogue) {
    case DenseEpilogue::kStore:
    case DenseEpilogue::kGated:
      store4(static_cast<T *>(a.out) + (size_t)r * a.ld_out + c, v, count, (a.ld_out & 3) == 0);
      return;
    case DenseEpilogue::kStoreF32:
      store4(a.out_f32 + (size_t)r * a.ld_f32 + c, v, count, (a.ld_f32 & 3) == 0);
      return;
    case DenseEpilogue::kAdd: {
      float *p = a.out_f32 + (size_t)r * a.ld_f32 + c;
      const float gate = a.row_gate ? sigmoid_f32(a.row_gate[(size_t)r * a.row_gate_stride]) : 1.0f;
      if (count >= 4 && (a.ld_f32 & 3) == 0) {
        f32x4 old = *reinterpret_cast<f32x4 *>(p);
#pragma unroll
        for (int i = 0; i < 4; ++i) old[i] += gate * v[i];
        *reinterpret_cast<f32x4 *>(p) = old;
        return;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (i < (int)count) p[i] += gate * v[i];
      return;
    }
    case DenseEpilogue::kQkv: {
      mix_values(a, r, c, v);
      store4(static_cast<T *>(a.out) + (size_t)r * a.ld_out + c, v, count, (a.ld_out & 3) == 0);
      return;
    }
    case DenseEpilogue::kSplit:
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (i < (int)count) {
          if (c + i < a.split) static_cast<T *>(a.out)[(size_t)r * a.ld_out + c + i] = (T)v[i];
          else a.out_f32[(size_t)r * a.ld_f32 + (c + i - a.split)] = v[i];
        }
      return;
  }
}

// Where a workgroup's tile lies; false: nothing to do.
struct TilePlace {
  uint32_t m_first, m_rows, n_first, expert;
};

template <int BM, int COLUMNS, bool ROUTED>
__device__ __forceinline__ bool place_tile(const GemmParams &p, TilePlace &t) {
  const DenseLinearArgs &a = p.a;
  t.expert = 0;
  if (ROUTED) {
    const uint32_t tile = blockIdx.y;
    t.m_rows = a.tile_rows[tile];
    if (t.m_rows == 0) return false;
    t.m_first = a.tile_first[tile];
    t.expert = a.tile_expert[tile];
    t.n_first = blockIdx.x * COLUMNS;
    return true;
  }
  const uint32_t id = (blockIdx.x & 7) * p.per_xcd + (blockIdx.x >> 3);
  if (id >= p.total) return false;
  // groups of eight row tiles walk the column tiles together
  const uint32_t group_tiles = 8 * p.tiles_n, group = id / group_tiles, within = id % group_tiles;
  const uint32_t rows_here = min(8u, p.tiles_m - group * 8);
  t.m_first = (group * 8 + within % rows_here) * BM;
  t.m_rows = min((uint32_t)BM, a.m - t.m_first);
  t.n_first = within / rows_here * COLUMNS;
  return true;
}

// GATED of the kernels: 0 no, 1 an activation of the gate alone, 2 the clamped pair.  (Apart: the epilogue's code is
// repeated for every value of a tile, and an activation more costs the large tiles a few percent.)
constexpr int kOneSided = 1, kClampedPair = 2;
template <int GATED>
__device__ __forceinline__ float gated(const DenseLinearArgs &a, float gate, float up) {
  if (GATED == kClampedPair) return gated_value(gate, up, kGateClamped, a.limit);
  return gate_activation(gate, a.activation) * up;
}

// A wave's accumulators: MT x NT groups of 16 x 16 from row `row_offset` and tile column `column_offset` on.
template <typename T, int MT, int NT, int GATED>
__device__ __forceinline__ void emit_tile(const DenseLinearArgs &a, const f32x4 (&acc)[MT][NT], uint32_t m_first,
                                          uint32_t m_rows, uint32_t n_first, uint32_t row_offset,
                                          uint32_t column_offset, int lane) {
  const int column = (lane >> 4) * 4;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const uint32_t r_in_tile = row_offset + i * 16 + (lane & 15);
    if (r_in_tile >= m_rows) continue;
    const uint32_t r = m_first + r_in_tile;
    if (GATED) {
#pragma unroll
      for (int j = 0; j < NT; j += 2) {
        const uint32_t c = n_first + column_offset / 2 + (j / 2) * 16 + column;
        if (c >= a.n) continue;
        f32x4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = gated<GATED>(a, acc[i][j][e], acc[i][j + 1][e]);
        emit<T>(a, r, c, v);
      }
    } else {
#pragma unroll
      for (int j = 0; j < NT; ++j) {
        const uint32_t c = n_first + column_offset + j * 16 + column;
        if (c < a.n) emit<T>(a, r, c, acc[i][j]);
      }
    }
  }
}

// WM x WN waves; a wave owns (BM / WM) x (BN / WN).  Two LDS stages: the next one travels global -> registers
// while this one is multiplied, one barrier a stage; LDS rows carry 16 bytes of padding, so that the sixteen
// rows an operand read touches start in different banks.
template <typename T, int BM, int BN, int WM, int GATED, bool ROUTED, bool VEC, int WAVES = 4>
__global__ __launch_bounds__(WAVES * 64) void dense_gemm_kernel(GemmParams p) {
  constexpr int WN = WAVES / WM, PASS = WAVES * 8;
  constexpr int MT = BM / WM / 16, NT = BN / WN / 16;
  constexpr int A_PIECES = BM / PASS, W_PIECES = BN / PASS;
  constexpr int SA = lds_stride<T>(), SW = lds_stride<__bf16>();
  constexpr int COLUMNS = GATED ? BN / 2 : BN;
  static_assert(!GATED || NT % 2 == 0, "gate and up of an element meet in one wave");
  extern __shared__ __attribute__((aligned(16))) char lds[];
  T *lds_a = reinterpret_cast<T *>(lds);
  __bf16 *lds_w = reinterpret_cast<__bf16 *>(lds + 2 * BM * SA * sizeof(T));
  const DenseLinearArgs &a = p.a;

  TilePlace place;
  if (!place_tile<BM, COLUMNS, ROUTED>(p, place)) return;
  const uint32_t m_first = place.m_first, m_rows = place.m_rows, n_first = place.n_first, expert = place.expert;

  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int wm = wave / WN, wn = wave % WN;
  const int piece = tid & 7, row_in_pass = tid >> 3;  // PASS rows a pass

  const T *src_a[A_PIECES];
#pragma unroll
  for (int i = 0; i < A_PIECES; ++i) {
    uint32_t r = m_first + min((uint32_t)(row_in_pass + PASS * i), m_rows - 1);
    if (ROUTED && a.row_source) r = a.row_source[r];
    src_a[i] = static_cast<const T *>(a.x) + (size_t)r * a.ldx + piece * 8;
  }
  const __bf16 *src_w[W_PIECES];
#pragma unroll
  for (int i = 0; i < W_PIECES; ++i) {
    const int r = row_in_pass + PASS * i;
    const uint16_t *matrix = a.w;
    uint32_t c = n_first + r;
    if (GATED) {
      if ((r >> 4) & 1) matrix = a.w_up;
      c = n_first + (r >> 5) * 16 + (r & 15);
    }
    c = min(c, a.n - 1);
    src_w[i] = reinterpret_cast<const __bf16 *>(matrix) + ((size_t)expert * a.n + c) * a.k + piece * 8;
  }

  Frag<T> reg_a[A_PIECES];
  bf16x8 reg_w[W_PIECES];
  auto fetch = [&](uint32_t k0) {
    const int count = (int)a.k - (int)(k0 + piece * 8);
#pragma unroll
    for (int i = 0; i < W_PIECES; ++i) reg_w[i] = load_piece(src_w[i] + k0, count, VEC);
#pragma unroll
    for (int i = 0; i < A_PIECES; ++i) reg_a[i] = load_piece(src_a[i] + k0, count, VEC);
  };
  auto stash = [&](int buffer) {
#pragma unroll
    for (int i = 0; i < A_PIECES; ++i)
      *reinterpret_cast<Frag<T> *>(lds_a + (buffer * BM + row_in_pass + PASS * i) * SA + piece * 8) = reg_a[i];
#pragma unroll
    for (int i = 0; i < W_PIECES; ++i)
      *reinterpret_cast<bf16x8 *>(lds_w + (buffer * BN + row_in_pass + PASS * i) * SW + piece * 8) = reg_w[i];
  };

  f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};

  const int stages = (int)((a.k + kStageK - 1) / kStageK);
  const int fr = lane & 15, fk = (lane >> 4) * 8;
  auto multiply = [&](int buffer) {
    const T *la = lds_a + (buffer * BM + wm * (BM / WM) + fr) * SA + fk;
    const __bf16 *lw = lds_w + (buffer * BN + wn * (BN / WN) + fr) * SW + fk;
#pragma unroll
    for (int kk = 0; kk < kStageK; kk += 32) {
      Frag<T> fa[MT];
      Frag<T> fw[NT];
#pragma unroll
      for (int j = 0; j < NT; ++j)
        fw[j] = convert_frag<T>(*reinterpret_cast<const bf16x8 *>(lw + j * 16 * SW + kk));
#pragma unroll
      for (int i = 0; i < MT; ++i) fa[i] = *reinterpret_cast<const Frag<T> *>(la + i * 16 * SA + kk);
#pragma unroll
      for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[i][j] = mma(fw[j], fa[i], acc[i][j]);
    }
  };
  fetch(0);
  stash(0);
  __syncthreads();
  for (int s = 0; s < stages; ++s) {
    if (s + 1 < stages) fetch((s + 1) * kStageK);
    multiply(s & 1);
    if (s + 1 < stages) stash((s & 1) ^ 1);
    __syncthreads();
  }

  emit_tile<T, MT, NT, GATED>(a, acc, m_first, m_rows, n_first, wm * (BM / WM), wn * (BN / WN), lane);
}

template <int BM, int COLUMNS, bool ROUTED>
GemmParams gemm_params(const DenseLinearArgs &a, dim3 *grid) {
  GemmParams p = {};
  p.a = a;
  p.tiles_n = (a.n + COLUMNS - 1) / COLUMNS;
  if (ROUTED) {
    *grid = dim3(p.tiles_n, a.tiles);
  } else {
    p.tiles_m = (a.m + BM - 1) / BM;
    p.total = p.tiles_m * p.tiles_n;
    p.per_xcd = (p.total + 7) / 8;
    *grid = dim3(p.per_xcd * 8);
  }
  return p;
}

template <typename T, int BM, int BN, int WM, int GATED, bool ROUTED, bool VEC, int WAVES = 4>
hipError_t run_gemm(const DenseLinearArgs &a, hipStream_t stream) {
  constexpr int bytes = gemm_lds_bytes<T, BM, BN>();
  static bool allowed[kMaxDevices] = {};
  if (bytes > 64 * 1024)
    if (hipError_t status = allow_dynamic_lds(
            reinterpret_cast<const void *>(dense_gemm_kernel<T, BM, BN, WM, GATED, ROUTED, VEC, WAVES>), bytes, allowed))
      return status;
  dim3 grid;
  const GemmParams p = gemm_params<BM, GATED ? BN / 2 : BN, ROUTED>(a, &grid);
  dense_gemm_kernel<T, BM, BN, WM, GATED, ROUTED, VEC, WAVES><<<grid, WAVES * 64, bytes, stream>>>(p);
  return hipGetLastError();
}

// The bf16 outputs of a wave, 16 rows at a time through its own LDS rows, so that a store covers whole lines.
template <int MT, int NT, int GATED>
__device__ __forceinline__ void emit_rows(const DenseLinearArgs &a, const f32x4 (&acc)[MT][NT], uint32_t m_first,
                                          uint32_t m_rows, uint32_t n_first, uint32_t row_offset,
                                          uint32_t column_offset, int lane, __bf16 *rows) {
  constexpr int WIDTH = (GATED ? NT / 2 : NT) * 16, STRIDE = WIDTH + 8, PIECES = WIDTH / 8;
  const uint32_t c_first = n_first + (GATED ? column_offset / 2 : column_offset);
  const uint32_t limit = a.epilogue == DenseEpilogue::kSplit ? a.split : a.n;  // columns of `out`
  const int quad = lane >> 4;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
    const uint32_t r_in_tile = row_offset + i * 16 + (lane & 15), r = m_first + r_in_tile;
#pragma unroll
    for (int j = 0; j < (GATED ? NT / 2 : NT); ++j) {
      const uint32_t c = c_first + j * 16 + quad * 4;
      f32x4 v;
      if (GATED) {
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = gated<GATED>(a, acc[i][2 * j][e], acc[i][2 * j + 1][e]);
      } else {
        v = acc[i][j];
        if (a.epilogue == DenseEpilogue::kQkv && r_in_tile < m_rows) mix_values(a, r, c, v);
        if (a.epilogue == DenseEpilogue::kSplit && r_in_tile < m_rows && c + 3 >= a.split) {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c + e >= a.split && c + e < a.n) a.out_f32[(size_t)r * a.ld_f32 + (c + e - a.split)] = v[e];
        }
      }
      bf16x4 packed;
#pragma unroll
      for (int e = 0; e < 4; ++e) packed[e] = (__bf16)v[e];
      *reinterpret_cast<bf16x4 *>(rows + (lane & 15) * STRIDE + j * 16 + quad * 4) = packed;
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // the wave's rows are whole
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int q = 0; q < (16 * PIECES + 63) / 64; ++q) {
      const int index = q * 64 + lane, row = index / PIECES, piece = index % PIECES;
      const uint32_t at = row_offset + i * 16 + row, c = c_first + piece * 8;
      if (row >= 16 || at >= m_rows || c >= limit) continue;
      const bf16x8 v = *reinterpret_cast<const bf16x8 *>(rows + row * STRIDE + piece * 8);
      __bf16 *out = static_cast<__bf16 *>(a.out) + (size_t)(m_first + at) * a.ld_out + c;
      if (c + 8 <= limit && a.ld_out % 8 == 0) {
        *reinterpret_cast<bf16x8 *>(out) = v;
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          if (c + e < limit) out[e] = v[e];
      }
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // read before the next sixteen rows are written
    __builtin_amdgcn_wave_barrier();
  }
}

// The same product for bf16 rows of a multiple of 64 values, staged by direct global -> LDS copies
// (global_load_lds_dwordx4: 64 lanes x 16 bytes to consecutive LDS addresses) a ring of STAGES stages deep:
// the copies of later stages run while a stage is multiplied, waited for by count, one barrier a stage.
// LDS rows are 128 bytes with their 16-byte pieces XOR-ed by half the row, which spreads the sixteen rows
// an operand read touches over all banks; the copies place pieces by permuting their source addresses.
__device__ __forceinline__ void copy_to_lds(const __bf16 *source, uint32_t lds_address) {
  asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off" : : "v"(source), "s"(lds_address) : "memory");
}

template <int BM, int BN, int WM, int WAVES, int STAGES, int GATED, bool ROUTED>
__global__ __launch_bounds__(WAVES * 64) void dense_gemm_direct_kernel(GemmParams p) {
  constexpr int WN = WAVES / WM;
  constexpr int MT = BM / WM / 16, NT = BN / WN / 16;
  constexpr int ROWS = BM + BN;              // LDS rows of a stage: activations, then weights
  constexpr int COPIES = ROWS / 8 / WAVES;   // 8-row copies of a wave per stage
  constexpr int COLUMNS = GATED ? BN / 2 : BN;
  static_assert(ROWS % (8 * WAVES) == 0 && (!GATED || NT % 2 == 0), "tile does not divide over the waves");
  extern __shared__ __attribute__((aligned(16))) char lds[];
  __bf16 *stage_rows = reinterpret_cast<__bf16 *>(lds);
  const DenseLinearArgs &a = p.a;
  TilePlace place;
  if (!place_tile<BM, COLUMNS, ROUTED>(p, place)) return;

  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int wm = wave / WN, wn = wave % WN;

  const __bf16 *source[COPIES];
#pragma unroll
  for (int i = 0; i < COPIES; ++i) {
    const int row = (i * WAVES + wave) * 8 + (lane >> 3);
    const int piece = (lane & 7) ^ ((row >> 1) & 7);
    if (row < BM) {
      uint32_t r = place.m_first + min((uint32_t)row, place.m_rows - 1);
      if (ROUTED && a.row_source) r = a.row_source[r];
      source[i] = static_cast<const __bf16 *>(a.x) + (size_t)r * a.ldx + piece * 8;
    } else {
      const int w_row = row - BM;
      const uint16_t *matrix = a.w;
      uint32_t c = place.n_first + w_row;
      if (GATED) {
        if ((w_row >> 4) & 1) matrix = a.w_up;
        c = place.n_first + (w_row >> 5) * 16 + (w_row & 15);
      }
      c = min(c, a.n - 1);
      source[i] = reinterpret_cast<const __bf16 *>(matrix) + ((size_t)place.expert * a.n + c) * a.k + piece * 8;
    }
  }
  const uint32_t lds_base = (uint32_t)(size_t)(__attribute__((address_space(3))) char *)lds;
  auto request = [&](int stage) {
    const uint32_t slot = lds_base + (stage % STAGES) * ROWS * 128;
#pragma unroll
    for (int i = 0; i < COPIES; ++i) copy_to_lds(source[i] + stage * kStageK, slot + (i * WAVES + wave) * 1024);
  };

  f32x4 acc[MT][NT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};

  const int stages = (int)(a.k / kStageK);
  const int fr = lane & 15, quad = lane >> 4, twist = (fr >> 1) & 7;
#pragma unroll
  for (int s = 0; s < STAGES - 1; ++s)
    if (s < stages) request(s);
  for (int s = 0; s < stages; ++s) {
    // this stage has landed once at most the copies of the STAGES - 2 later ones are under way (and this wave
    // has all it read of the stage before)
    if (s + STAGES - 2 < stages) asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" : : "n"((STAGES - 2) * COPIES) : "memory");
    else asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    // every wave is done with the stage before: its slot is free
    if (s + STAGES - 1 < stages) request(s + STAGES - 1);
    const __bf16 *rows = stage_rows + (s % STAGES) * ROWS * 64;
    const __bf16 *la = rows + (wm * (BM / WM) + fr) * 64, *lw = rows + (BM + wn * (BN / WN) + fr) * 64;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      const int at = ((kk * 4 + quad) ^ twist) * 8;
      bf16x8 fa[MT], fw[NT];
#pragma unroll
      for (int j = 0; j < NT; ++j) fw[j] = *reinterpret_cast<const bf16x8 *>(lw + j * 16 * 64 + at);
#pragma unroll
      for (int i = 0; i < MT; ++i) fa[i] = *reinterpret_cast<const bf16x8 *>(la + i * 16 * 64 + at);
#pragma unroll
      for (int i = 0; i < MT; ++i)
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[i][j] = mma(fw[j], fa[i], acc[i][j]);
    }
  }
  if (a.epilogue == DenseEpilogue::kAdd || a.epilogue == DenseEpilogue::kStoreF32) {
    emit_tile<__bf16, MT, NT, GATED>(a, acc, place.m_first, place.m_rows, place.n_first, wm * (BM / WM),
                                     wn * (BN / WN), lane);
    return;
  }
  __syncthreads();  // the stages' LDS is free
  static_assert(16 * (NT * 16 + 8) * 2 * WAVES <= STAGES * ROWS * 128, "a wave's output rows fit");
  emit_rows<MT, NT, GATED>(a, acc, place.m_first, place.m_rows, place.n_first, wm * (BM / WM), wn * (BN / WN), lane,
                           stage_rows + wave * 16 * (NT * 16 + 8));
}

template <int BM, int BN, int WM, int WAVES, int STAGES, int GATED, bool ROUTED>
hipError_t run_direct(const DenseLinearArgs &a, hipStream_t stream) {
  constexpr int bytes = STAGES * (BM + BN) * 128;
  static bool allowed[kMaxDevices] = {};
  const auto kernel = dense_gemm_direct_kernel<BM, BN, WM, WAVES, STAGES, GATED, ROUTED>;
  if (bytes > 64 * 1024)
    if (hipError_t status = allow_dynamic_lds(reinterpret_cast<const void *>(kernel), bytes, allowed)) return status;
  dim3 grid;
  const GemmParams p = gemm_params<BM, GATED ? BN / 2 : BN, ROUTED>(a, &grid);
  kernel<<<grid, WAVES * 64, bytes, stream>>>(p);
  return hipGetLastError();
}

// Rows whose length is no multiple of the stage, and float32 rows: through registers.
template <typename T, int BM, int GATED, bool ROUTED>
hipError_t run_registers(const DenseLinearArgs &a, hipStream_t stream) {
  if (a.k % 8 == 0 && a.ldx % 8 == 0) return run_gemm<T, BM, 64, 2, GATED, ROUTED, true>(a, stream);
  return run_gemm<T, BM, 64, 2, GATED, ROUTED, false>(a, stream);
}

template <int GATED>
hipError_t pick_routed(const DenseLinearArgs &a, hipStream_t stream) {
  const bool direct = !a.f32 && a.k % kStageK == 0 && a.ldx % 8 == 0;
  if (a.tile == 128) return direct ? run_direct<128, 128, 2, 4, 2, GATED, true>(a, stream) : hipErrorInvalidValue;
  if (direct) return run_direct<64, 128, 2, 4, 3, GATED, true>(a, stream);
  return a.f32 ? run_registers<float, 64, GATED, true>(a, stream) : run_registers<__bf16, 64, GATED, true>(a, stream);
}

// The largest tile that still gives the 256 CUs whole rounds of work.  Measured, TFLOP/s (m x n x k):
// 8192 x 4096 x 4096 937 / 827 with 256 x 256 / 128 x 128 tiles; 2048 x 8512 x 2048 500 / 680 / 643 with
// 256 x 256 / 128 x 128 / 64 x 128; 2048 x 2048 x 8192 723 / 842 / 681 with 128 x 128 / 64 x 128 / 64 x 64;
// 512 x 2048 x 4096 261 / 359 with 64 x 128 / 64 x 64; 64 x 4096 x 2048 80 / 89 with 64 x 64 / 32 x 64.
template <int GATED>
hipError_t pick_gemm(const DenseLinearArgs &a, hipStream_t stream) {
  if (a.f32) return run_registers<float, 32, GATED, false>(a, stream);
  const uint32_t columns = a.n * (GATED ? 2 : 1);
  auto tiles = [&](uint32_t rows, uint32_t width) {
    return (uint64_t)((a.m + rows - 1) / rows) * ((columns + width - 1) / width);
  };
  if (a.k % kStageK != 0 || a.ldx % 8 != 0) return run_registers<__bf16, 32, GATED, false>(a, stream);
  const uint64_t largest = tiles(256, 256), over = largest % 256;
  if (largest >= 1024 || (largest >= 256 && (over == 0 || over >= 192)))
    return run_direct<256, 256, 2, 8, 2, GATED, false>(a, stream);
  if (tiles(128, 128) > 320) return run_direct<128, 128, 2, 4, 2, GATED, false>(a, stream);
  if (tiles(64, 128) >= 320) return run_direct<64, 128, 2, 4, 3, GATED, false>(a, stream);
  if (tiles(64, 64) >= 160) return run_direct<64, 64, 2, 4, 4, GATED, false>(a, stream);
  return run_direct<32, 64, 2, 4, 6, GATED, false>(a, stream);
}

// ---- row-wise kernels ------------------------------------------------------------------------------

template <typename T>
__global__ __launch_bounds__(256) void dense_norm_kernel(DenseNormArgs a) {
  extern __shared__ float row[];
  __shared__ float scratch[4];
  const uint32_t r = blockIdx.x;
  const uint32_t source = a.rows_index ? a.rows_index[r] : r;
  const __bf16 *weight = reinterpret_cast<const __bf16 *>(a.weight);
  const uint32_t part = a.width / a.groups;
  for (uint32_t g = 0; g < a.groups; ++g) {
    float sum = 0.0f;
    for (uint32_t i = g * part + threadIdx.x; i < (g + 1) * part; i += 256) {
      float v;
      if (a.x_act) {
        v = to_f32(static_cast<const T *>(a.x_act)[(size_t)source * a.width + i]);
        if (a.gate) v *= silu_f32(to_f32(static_cast<const T *>(a.gate)[(size_t)source * a.ld_gate + i]));
      } else {
        v = a.x[(size_t)source * a.width + i];
      }
      row[i] = v;
      sum += v * v;
    }
    sum = block_sum<4>(sum, scratch);
    const float inverse = 1.0f / sqrtf(sum / (float)part + a.epsilon);
    for (uint32_t i = g * part + threadIdx.x; i < (g + 1) * part; i += 256)
      static_cast<T *>(a.out)[(size_t)r * a.width + i] = (T)(row[i] * inverse * (float)weight[i]);
  }
}

// The same for widths a thread covers in pieces of eight (part % 8 == 0, at most 8 pieces a thread):
// 16-byte accesses and the row in registers; four waves a row, one group at a time.
template <typename T>
__global__ __launch_bounds__(256) void dense_norm_vec_kernel(DenseNormArgs a) {
  __shared__ float scratch[4];
  const uint32_t r = blockIdx.x, group = blockIdx.y;
  const uint32_t source = a.rows_index ? a.rows_index[r] : r;
  const __bf16 *weight = reinterpret_cast<const __bf16 *>(a.weight);
  const uint32_t part = a.width / a.groups, first = group * part;
  f32x8 v[8];
  float sum = 0.0f;
#pragma unroll
  for (int q = 0; q < 8; ++q) {
    const uint32_t i = (q * 256 + threadIdx.x) * 8;
    if (i >= part) break;
    if (a.x_act) {
      v[q] = convert_frag<float>(
          *reinterpret_cast<const Frag<T> *>(static_cast<const T *>(a.x_act) + (size_t)source * a.width + first + i));
      if (a.gate) {
        const f32x8 g = convert_frag<float>(*reinterpret_cast<const Frag<T> *>(
            static_cast<const T *>(a.gate) + (size_t)source * a.ld_gate + first + i));
#pragma unroll
        for (int e = 0; e < 8; ++e) v[q][e] *= silu_f32(g[e]);
      }
    } else {
      v[q] = *reinterpret_cast<const f32x8 *>(a.x + (size_t)source * a.width + first + i);
    }
#pragma unroll
    for (int e = 0; e < 8; ++e) sum += v[q][e] * v[q][e];
  }
  sum = block_sum<4>(sum, scratch);
  const float inverse = 1.0f / sqrtf(sum / (float)part + a.epsilon);
#pragma unroll
  for (int q = 0; q < 8; ++q) {
    const uint32_t i = (q * 256 + threadIdx.x) * 8;
    if (i >= part) break;
    const bf16x8 w = *reinterpret_cast<const bf16x8 *>(weight + first + i);
    Frag<T> out;
#pragma unroll
    for (int e = 0; e < 8; ++e) out[e] = (T)(v[q][e] * inverse * (float)w[e]);
    *reinterpret_cast<Frag<T> *>(static_cast<T *>(a.out) + (size_t)r * a.width + first + i) = out;
  }
}

// A workgroup a row.  VEC: eight values a thread and piece in registers (width % 8 == 0, at most 8 pieces),
// else the row's parts are read again from cache.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void norm_add_kernel(NormAddArgs a) {
  __shared__ float scratch[4];
  const uint32_t r = blockIdx.x, source = a.rows_index ? a.rows_index[r] : r;
  const float *x = a.x + (size_t)source * a.width, *y = a.y ? a.y + (size_t)source * a.width : nullptr;
  const __bf16 *add = reinterpret_cast<const __bf16 *>(a.add_weight), *norm = reinterpret_cast<const __bf16 *>(a.norm_weight);
  float *out = a.stream_out ? a.stream_out + (size_t)r * a.width : nullptr;
  T *operand = a.operand ? static_cast<T *>(a.operand) + (size_t)r * a.width : nullptr;
  if (VEC) {
    f32x8 v[8], z[8];
    float sum = 0.0f;
#pragma unroll
    for (int q = 0; q < 8; ++q) {
      const uint32_t i = (q * 256 + threadIdx.x) * 8;
      if (i >= a.width) break;
      v[q] = *reinterpret_cast<const f32x8 *>(x + i);
      if (y) {
        z[q] = *reinterpret_cast<const f32x8 *>(y + i);
#pragma unroll
        for (int e = 0; e < 8; ++e) sum += z[q][e] * z[q][e];
      }
    }
    if (y) {
      sum = block_sum<4>(sum, scratch);
      const float factor = a.scale / sqrtf(sum / (float)a.width + a.epsilon);
#pragma unroll
      for (int q = 0; q < 8; ++q) {
        const uint32_t i = (q * 256 + threadIdx.x) * 8;
        if (i >= a.width) break;
        const bf16x8 w = *reinterpret_cast<const bf16x8 *>(add + i);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[q][e] = fmaf(z[q][e] * factor, a.offset + (float)w[e], v[q][e]);
      }
    }
    float inverse = 1.0f;
    if (norm) {
      sum = 0.0f;
#pragma unroll
      for (int q = 0; q < 8; ++q) {
        if ((q * 256 + threadIdx.x) * 8 >= a.width) break;
#pragma unroll
        for (int e = 0; e < 8; ++e) sum += v[q][e] * v[q][e];
      }
      inverse = 1.0f / sqrtf(block_sum<4>(sum, scratch) / (float)a.width + a.epsilon);
    }
#pragma unroll
    for (int q = 0; q < 8; ++q) {
      const uint32_t i = (q * 256 + threadIdx.x) * 8;
      if (i >= a.width) break;
      if (out) *reinterpret_cast<f32x8 *>(out + i) = v[q];
      if (!operand) continue;
      if (norm) {
        const bf16x8 w = *reinterpret_cast<const bf16x8 *>(norm + i);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[q][e] *= inverse * (a.offset + (float)w[e]);
      }
      *reinterpret_cast<Frag<T> *>(operand + i) = convert_frag<T>(v[q]);
    }
    return;
  }
  float factor = 0.0f;
  if (y) {
    float sum = 0.0f;
    for (uint32_t i = threadIdx.x; i < a.width; i += 256) sum += y[i] * y[i];
    factor = a.scale / sqrtf(block_sum<4>(sum, scratch) / (float)a.width + a.epsilon);
  }
  auto value = [&](uint32_t i) { return y ? fmaf(y[i] * factor, a.offset + (float)add[i], x[i]) : x[i]; };
  float inverse = 1.0f;
  if (norm) {
    float sum = 0.0f;
    for (uint32_t i = threadIdx.x; i < a.width; i += 256) sum += value(i) * value(i);
    inverse = 1.0f / sqrtf(block_sum<4>(sum, scratch) / (float)a.width + a.epsilon);
  }
  for (uint32_t i = threadIdx.x; i < a.width; i += 256) {
    const float v = value(i);
    if (out) out[i] = v;
    if (operand) operand[i] = (T)(norm ? v * inverse * (a.offset + (float)norm[i]) : v);
  }
}

__global__ __launch_bounds__(256) void soft_cap_kernel(float *values, uint64_t count, float cap) {
  const uint64_t i = (uint64_t)blockIdx.x * 256 + threadIdx.x;
  if (i < count) values[i] = soft_capped(values[i], cap);
}

__global__ __launch_bounds__(256) void dense_embedding_kernel(DenseEmbeddingArgs a) {
  const uint32_t t = blockIdx.x;
  const int64_t token = a.tokens[t];
  const bool known = token >= 0 && token < (int64_t)a.vocabulary;
  const __bf16 *source = reinterpret_cast<const __bf16 *>(a.embed) + (size_t)(known ? token : 0) * a.width;
  for (uint32_t i = threadIdx.x; i < a.width; i += 256)
    a.stream[(size_t)t * a.width + i] = known ? (float)source[i] * a.scale : 0.0f;
}

}  // namespace

hipError_t launch_dense_gemm(const DenseLinearArgs &a, hipStream_t stream) {
  const bool pair = a.epilogue == DenseEpilogue::kGated, clamped = a.activation == kGateClamped;
  if (a.tile_expert) {
    if (pair && clamped) return hipErrorInvalidValue;
    return pair ? pick_routed<kOneSided>(a, stream) : pick_routed<0>(a, stream);
  }
  if (!pair) return pick_gemm<0>(a, stream);
  return clamped ? pick_gemm<kClampedPair>(a, stream) : pick_gemm<kOneSided>(a, stream);
}

hipError_t launch_dense_norm(const DenseNormArgs &a, hipStream_t stream) {
  const uint32_t part = a.width / a.groups;
  const bool vec = part % 8 == 0 && part <= 8 * 256 * 8 && (!a.gate || a.ld_gate % 8 == 0);
  if (vec) {
    const dim3 grid(a.rows, a.groups);
    if (a.f32) dense_norm_vec_kernel<float><<<grid, 256, 0, stream>>>(a);
    else dense_norm_vec_kernel<__bf16><<<grid, 256, 0, stream>>>(a);
    return hipGetLastError();
  }
  const size_t bytes = (size_t)a.width * 4;
  if (bytes > 60 * 1024) return hipErrorInvalidValue;
  if (a.f32) dense_norm_kernel<float><<<a.rows, 256, bytes, stream>>>(a);
  else dense_norm_kernel<__bf16><<<a.rows, 256, bytes, stream>>>(a);
  return hipGetLastError();
}

hipError_t launch_soft_cap(float *values, uint64_t count, float cap, hipStream_t stream) {
  soft_cap_kernel<<<(uint32_t)((count + 255) / 256), 256, 0, stream>>>(values, count, cap);
  return hipGetLastError();
}

hipError_t launch_norm_add(const NormAddArgs &a, hipStream_t stream) {
  const bool vec = a.width % 8 == 0 && a.width <= 8 * 256 * 8;
  if (a.f32) {
    if (vec) norm_add_kernel<float, true><<<a.rows, 256, 0, stream>>>(a);
    else norm_add_kernel<float, false><<<a.rows, 256, 0, stream>>>(a);
  } else {
    if (vec) norm_add_kernel<__bf16, true><<<a.rows, 256, 0, stream>>>(a);
    else norm_add_kernel<__bf16, false><<<a.rows, 256, 0, stream>>>(a);
  }
  return hipGetLastError();
}

hipError_t launch_dense_embedding(const DenseEmbeddingArgs &a, hipStream_t stream) {
  dense_embedding_kernel<<<a.m, 256, 0, stream>>>(a);
  return hipGetLastError();
}

}  // namespace llmopt
