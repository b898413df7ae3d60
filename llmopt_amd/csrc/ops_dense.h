// What the entry points over bfloat16 weights share (ops_dense.cpp, ops_parallel.cpp).
#pragma once

#include <cmath>
#include <cstdio>

#include "kernels/dense.h"
#include "runtime.h"

namespace llmopt {

inline const uint16_t *as_bf16(const BoundBuffer &b) { return reinterpret_cast<const uint16_t *>(b.device); }
inline float *as_f32(const BoundBuffer &b) { return reinterpret_cast<float *>(b.device); }
inline const uint32_t *as_u32(const BoundBuffer &b) { return reinterpret_cast<const uint32_t *>(b.device); }

inline int launched(hipError_t status, const char *name) {
  if (status != hipSuccess) return fail(LLMOPT_ERR_FAILURE, "%s launch failed: %s", name, hipGetErrorString(status));
  return LLMOPT_OK;
}

inline size_t round_up_256(size_t bytes) { return (bytes + 255) & ~(size_t)255; }

inline bool valid_epsilon(float epsilon) { return std::isfinite(epsilon) && epsilon >= 0.0f; }

inline int require_positive(const DispatchRecord &record, std::initializer_list<uint32_t> values) {
  for (uint32_t value : values)
    if (value == 0) return fail(LLMOPT_ERR_INVALID, "%s requires positive sizes", record.name.c_str());
  return LLMOPT_OK;
}

inline int require_sizes(const DispatchRecord &record, std::initializer_list<std::pair<int, uint64_t>> sizes) {
  for (const auto &size : sizes) {
    char name[32];
    snprintf(name, sizeof name, "operand %d", size.first);
    if (int status = require_buffer_size(record.buffers[size.first], size.second, name)) return status;
  }
  return LLMOPT_OK;
}

// Scratch of one entry, cut into aligned parts.
class Scratch {
 public:
  size_t want(size_t bytes) {
    const size_t at = total_;
    total_ += round_up_256(bytes);
    return at;
  }
  bool get(llmopt_hip_context *context) {
    base_ = static_cast<uint8_t *>(context_workspace(context, total_));
    return base_ != nullptr;
  }
  template <typename P>
  P *at(size_t offset) const {
    return reinterpret_cast<P *>(base_ + offset);
  }

 private:
  size_t total_ = 0;
  uint8_t *base_ = nullptr;
};

template <bool F32>
constexpr size_t kElement = F32 ? 4 : 2;

inline DenseLinearArgs linear(bool f32, const void *x, const uint16_t *w, uint32_t m, uint32_t n, uint32_t k) {
  DenseLinearArgs a = {};
  a.f32 = f32;
  a.x = x;
  a.w = w;
  a.m = m;
  a.n = n;
  a.k = k;
  a.ldx = k;
  return a;
}

}  // namespace llmopt
