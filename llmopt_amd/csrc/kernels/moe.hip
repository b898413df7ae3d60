// Routing of many tokens to their experts: selection, sorting by expert, and the weighted sum of the
// chosen experts' outputs.  (One token: dense_gemv.hip.)
#include <algorithm>

#include "dense.h"
#include "dense_common.h"
#include "kernels_internal.h"

namespace llmopt {
namespace {

// A wave a token: the rank of an expert is the number of logits ahead of it.
__global__ __launch_bounds__(256) void route_select_kernel(RoutePlan p) {
  extern __shared__ float lds[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const uint32_t t = blockIdx.x * 4 + wave;
  float *z = lds + wave * (p.experts + p.top), *chosen = z + p.experts;
  const bool live = t < p.m;
  if (live)
    for (uint32_t e = lane; e < p.experts; e += 64) z[e] = p.logits[(size_t)t * p.ld_logits + e];
  __syncthreads();
  if (live)
    for (uint32_t e = lane; e < p.experts; e += 64) {
      const float mine = z[e];
      uint32_t rank = 0;
      for (uint32_t other = 0; other < p.experts; ++other) rank += z[other] > mine || (z[other] == mine && other < e);
      if (rank < p.top) {
        chosen[rank] = mine;
        p.expert[(size_t)t * p.top + rank] = e;
      }
    }
  __syncthreads();
  if (!live) return;
  const float best = chosen[0];
  float total = 0.0f;
  for (uint32_t s = 0; s < p.top; ++s) total += __expf(chosen[s] - best);
  for (uint32_t s = lane; s < p.top; s += 64) p.weight[(size_t)t * p.top + s] = __expf(chosen[s] - best) / total;
}

// One workgroup: counts, starts, tiles, and every pair's row in the sorted order.
__global__ __launch_bounds__(1024) void route_sort_kernel(RoutePlan p) {
  extern __shared__ uint32_t words[];
  uint32_t *count = words, *start = words + p.experts;
  const uint32_t pairs = p.m * p.top;
  for (uint32_t e = threadIdx.x; e < p.experts; e += 1024) count[e] = 0;
  __syncthreads();
  for (uint32_t i = threadIdx.x; i < pairs; i += 1024) atomicAdd(&count[p.expert[i]], 1u);
  __syncthreads();
  if (threadIdx.x == 0) {
    uint32_t row = 0, tile = 0;
    for (uint32_t e = 0; e < p.experts; ++e) {
      start[e] = row;
      for (uint32_t done = 0; done < count[e]; done += kRoutedTileRows) {
        p.tile_expert[tile] = e;
        p.tile_first[tile] = row + done;
        p.tile_rows[tile] = min(kRoutedTileRows, count[e] - done);
        ++tile;
      }
      row += count[e];
    }
    for (; tile < p.max_tiles; ++tile) p.tile_rows[tile] = 0;
  }
  __syncthreads();
  for (uint32_t i = threadIdx.x; i < pairs; i += 1024) {
    const uint32_t row = atomicAdd(&start[p.expert[i]], 1u);
    p.position[i] = row;
    p.row_token[row] = i / p.top;
  }
}

template <typename T>
__global__ __launch_bounds__(256) void route_combine_kernel(RoutePlan p, const T *rows, float *stream, uint32_t width) {
  const uint32_t t = blockIdx.x;
  for (uint32_t c = threadIdx.x; c < width; c += 256) {
    float sum = 0.0f;
    for (uint32_t s = 0; s < p.top; ++s) {
      const size_t pair = (size_t)t * p.top + s;
      sum = fmaf(p.weight[pair], to_f32(rows[(size_t)p.position[pair] * width + c]), sum);
    }
    stream[(size_t)t * width + c] += sum;
  }
}

}  // namespace

uint32_t route_max_tiles(uint32_t m, uint32_t experts, uint32_t top) {
  const uint64_t pairs = (uint64_t)m * top;
  return (uint32_t)(pairs / kRoutedTileRows + std::min<uint64_t>(experts, pairs));
}

hipError_t launch_route(const RoutePlan &p, hipStream_t stream) {
  const size_t bytes = 4 * (p.experts + p.top) * 4;
  if (bytes > 60 * 1024) return hipErrorInvalidValue;
  route_select_kernel<<<(p.m + 3) / 4, 256, bytes, stream>>>(p);
  if (hipError_t status = hipGetLastError()) return status;
  route_sort_kernel<<<1, 1024, 2 * p.experts * 4, stream>>>(p);
  return hipGetLastError();
}

hipError_t launch_route_combine(const RouteCombineArgs &a, hipStream_t stream) {
  const RoutePlan &p = *a.plan;
  if (a.f32)
    route_combine_kernel<float><<<p.m, 256, 0, stream>>>(p, static_cast<const float *>(a.rows), a.stream, a.width);
  else
    route_combine_kernel<__bf16><<<p.m, 256, 0, stream>>>(p, static_cast<const __bf16 *>(a.rows), a.stream, a.width);
  return hipGetLastError();
}

}  // namespace llmopt
