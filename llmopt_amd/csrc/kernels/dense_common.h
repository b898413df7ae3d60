// Shared device helpers of the kernels over bfloat16 weights (dense_gemm.hip, dense_gemv.hip,
// chunk_attention.hip, ssm.hip, delta.hip, moe.hip).  Every kernel is a template over the element type T of the
// activations: __bf16 (products on the bfloat16 matrix cores) or float (products on the float32
// matrix cores, v_mfma_f32_16x16x4_f32: no reduced precision anywhere).  Accumulation is float32 in both.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

namespace llmopt {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x8 __attribute__((ext_vector_type(8)));

template <typename T>
struct VecOf;
template <>
struct VecOf<__bf16> {
  typedef bf16x8 x8;
};
template <>
struct VecOf<float> {
  typedef f32x8 x8;
};

// One lane's share of a 16 x 32 matrix-core operand: eight consecutive contraction indices of one row.
template <typename T>
using Frag = typename VecOf<T>::x8;

__device__ __forceinline__ float to_f32(__bf16 v) { return (float)v; }
__device__ __forceinline__ float to_f32(float v) { return v; }

// D[16 x 16] += A[16 x 32] B[32 x 16].  Lane l holds row (A) / column (B) l % 16, contraction indices
// 8 (l / 16) .. + 7; D: column l % 16, rows 4 (l / 16) .. + 3.
__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma(f32x8 a, f32x8 b, f32x4 c) {
#pragma unroll
  for (int i = 0; i < 8; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
  return c;
}

template <typename T>
__device__ __forceinline__ Frag<T> zero_frag() {
  Frag<T> f;
#pragma unroll
  for (int i = 0; i < 8; ++i) f[i] = (T)0.0f;
  return f;
}

// A float32 operand as the matrix cores take it.  float: as it is.  __bf16: a high and a low part
// (16 bits of mantissa together), so that operands which must keep float32 accuracy (recurrent state,
// decay-weighted inputs) do not lose it to the operand format.
template <typename T>
struct WideFrag;
template <>
struct WideFrag<float> {
  f32x8 v;
  __device__ __forceinline__ void set(int i, float x) { v[i] = x; }
};
template <>
struct WideFrag<__bf16> {
  bf16x8 hi, lo;
  __device__ __forceinline__ void set(int i, float x) {
    hi[i] = (__bf16)x;
    lo[i] = (__bf16)(x - (float)hi[i]);
  }
};
__device__ __forceinline__ f32x4 mma_wide(const WideFrag<float> &a, f32x8 b, f32x4 c) { return mma(a.v, b, c); }
__device__ __forceinline__ f32x4 mma_wide(const WideFrag<__bf16> &a, bf16x8 b, f32x4 c) {
  return mma(a.lo, b, mma(a.hi, b, c));
}
__device__ __forceinline__ f32x4 mma_wide_b(f32x8 a, const WideFrag<float> &b, f32x4 c) { return mma(a, b.v, c); }
__device__ __forceinline__ f32x4 mma_wide_b(bf16x8 a, const WideFrag<__bf16> &b, f32x4 c) {
  return mma(a, b.lo, mma(a, b.hi, c));
}

// Both operands wide: everything but the product of the two low parts.
__device__ __forceinline__ f32x4 mma_wide_both(const WideFrag<float> &a, const WideFrag<float> &b, f32x4 c) {
  return mma(a.v, b.v, c);
}
__device__ __forceinline__ f32x4 mma_wide_both(const WideFrag<__bf16> &a, const WideFrag<__bf16> &b, f32x4 c) {
  return mma(a.hi, b.hi, mma(a.lo, b.hi, mma(a.hi, b.lo, c)));
}

// Eight consecutive elements from p, of which `count` (possibly <= 0 or > 8) exist; the rest are zero.
// vec: p is aligned to the whole piece and pieces are never partial (count >= 8 or count <= 0).
template <typename T>
__device__ __forceinline__ Frag<T> load_piece(const T *p, int count, bool vec) {
  if (count <= 0) return zero_frag<T>();
  if (vec) return *reinterpret_cast<const Frag<T> *>(p);
  Frag<T> f = zero_frag<T>();
#pragma unroll
  for (int i = 0; i < 8; ++i)
    if (i < count) f[i] = p[i];
  return f;
}

template <typename To, typename From>
__device__ __forceinline__ Frag<To> convert_frag(const From &from) {
  Frag<To> f;
#pragma unroll
  for (int i = 0; i < 8; ++i) f[i] = (To)(float)from[i];
  return f;
}
template <>
__device__ __forceinline__ bf16x8 convert_frag<__bf16, bf16x8>(const bf16x8 &from) {
  return from;
}

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + __expf(-z)); }
__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + __expf(-z)); }
// tanh through one exponential; |error| of a few 2^-24
__device__ __forceinline__ float tanh_f32(float z) {
  const float e = __expf(2.0f * fabsf(z));
  return copysignf(1.0f - 2.0f / (e + 1.0f), z);
}
__device__ __forceinline__ float softplus_f32(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

// log(1 + e^z) from the hardware's exponential and logarithm: log(u) e / (u - 1) with u = 1 + e rounded takes the
// rounding of u back out.
__device__ __forceinline__ float softplus_fast_f32(float z) {
  const float e = __expf(-fabsf(z)), u = 1.0f + e;
  return fmaxf(z, 0.0f) + (u == 1.0f ? e : __logf(u) * e * __builtin_amdgcn_rcpf(u - 1.0f));
}

// Activation of a gated feed-forward.
enum GateActivation : uint32_t { kGateSilu = 0, kGateGeluTanh = 1, kGateClamped = 2 };
__device__ __forceinline__ float gate_activation(float z, uint32_t kind) {
  if (kind == kGateGeluTanh) return 0.5f * z * (1.0f + tanh_f32(0.7978845608028654f * (z + 0.044715f * z * z * z)));
  return silu_f32(z);
}

// act(gate) up; clamped: both halves limited, a steeper sigmoid, and one more than the up half.
__device__ __forceinline__ float gated_value(float gate, float up, uint32_t kind, float limit) {
  if (kind == kGateClamped) {
    const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
    return g * sigmoid_f32(1.702f * g) * (u + 1.0f);
  }
  return gate_activation(gate, kind) * up;
}
__device__ __forceinline__ float soft_capped(float z, float cap) { return cap > 0.0f ? cap * tanh_f32(z / cap) : z; }

// Cosine and sine of position * frequency: the angle is reduced to one turn before it is rounded to float32.
__device__ __forceinline__ void turn(uint32_t position, double frequency, float &cosine, float &sine) {
  constexpr double kTurn = 6.283185307179586476925;
  const double angle = (double)position * frequency;
  sincosf((float)(angle - kTurn * rint(angle / kTurn)), &sine, &cosine);
}

// Sum over the 64 lanes of a wave, in every lane.
template <int CONTROL>
__device__ __forceinline__ float dpp_f32(float v) {
  return __builtin_bit_cast(float, __builtin_amdgcn_mov_dpp(__builtin_bit_cast(int, v), CONTROL, 0xf, 0xf, true));
}
__device__ __forceinline__ float wave_sum(float v) {
  // within rows of sixteen lanes: neighbours, pairs, halves, the row
  v += dpp_f32<0xb1>(v);   // quad_perm [1, 0, 3, 2]
  v += dpp_f32<0x4e>(v);   // quad_perm [2, 3, 0, 1]
  v += dpp_f32<0x141>(v);  // row_half_mirror
  v += dpp_f32<0x140>(v);  // row_mirror
  v += __shfl_xor(v, 16, 64);
  v += __shfl_xor(v, 32, 64);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int mask = 32; mask >= 1; mask >>= 1) v = fmaxf(v, __shfl_xor(v, mask, 64));
  return v;
}

// Sum over a workgroup of WAVES waves, in every thread; `scratch` holds WAVES floats and is free again
// after the caller's next barrier.
template <int WAVES>
__device__ __forceinline__ float block_sum(float v, float *scratch) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
  __syncthreads();
  float total = 0.0f;
#pragma unroll
  for (int w = 0; w < WAVES; ++w) total += scratch[w];
  return total;
}

}  // namespace llmopt
