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
  uint32_t *count = words, *start = count + p.experts, *tile_start = start + p.experts;
  const uint32_t pairs = p.m * p.top;
  for (uint32_t e = threadIdx.x; e < p.experts; e += 1024) count[e] = 0;
  for (uint32_t t = threadIdx.x; t < p.max_tiles; t += 1024) p.tile_rows[t] = 0;
  __syncthreads();
  constexpr int BLOCK = 8;  // pairs of a thread requested together
  for (uint32_t i0 = threadIdx.x; i0 < pairs; i0 += 1024 * BLOCK) {
    uint32_t e[BLOCK];
#pragma unroll
    for (int b = 0; b < BLOCK; ++b) e[b] = i0 + b * 1024 < pairs ? p.expert[i0 + b * 1024] : 0;
#pragma unroll
    for (int b = 0; b < BLOCK; ++b)
      if (i0 + b * 1024 < pairs) atomicAdd(&count[e[b]], 1u);
  }
  __syncthreads();
  if (threadIdx.x < 64) {  // one wave: running sums over the experts, 64 at a time
    uint32_t rows = 0, tiles = 0;
    for (uint32_t e0 = 0; e0 < p.experts; e0 += 64) {
      const uint32_t e = e0 + threadIdx.x;
      const uint32_t mine = e < p.experts ? count[e] : 0, mine_tiles = (mine + p.tile - 1) / p.tile;
      uint32_t sum = mine, tile_sum = mine_tiles;
#pragma unroll
      for (int step = 1; step < 64; step <<= 1) {
        const uint32_t a = __shfl_up(sum, step, 64), b = __shfl_up(tile_sum, step, 64);
        if ((int)threadIdx.x >= step) {
          sum += a;
          tile_sum += b;
        }
      }
      if (e < p.experts) {
        start[e] = rows + sum - mine;
        tile_start[e] = tiles + tile_sum - mine_tiles;
      }
      rows += __shfl(sum, 63, 64);
      tiles += __shfl(tile_sum, 63, 64);
    }
  }
  __syncthreads();
  for (uint32_t e = threadIdx.x; e < p.experts; e += 1024)
    for (uint32_t done = 0, tile = tile_start[e]; done < count[e]; done += p.tile, ++tile) {
      p.tile_expert[tile] = e;
      p.tile_first[tile] = start[e] + done;
      p.tile_rows[tile] = min(p.tile, count[e] - done);
    }
  __syncthreads();
  for (uint32_t i0 = threadIdx.x; i0 < pairs; i0 += 1024 * BLOCK) {
    uint32_t e[BLOCK];
#pragma unroll
    for (int b = 0; b < BLOCK; ++b) e[b] = i0 + b * 1024 < pairs ? p.expert[i0 + b * 1024] : 0;
#pragma unroll
    for (int b = 0; b < BLOCK; ++b) {
      const uint32_t i = i0 + b * 1024;
      if (i >= pairs) continue;
      const uint32_t row = atomicAdd(&start[e[b]], 1u);
      p.position[i] = row;
      p.row_token[row] = i / p.top;
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void route_combine_kernel(RoutePlan p, const T *rows, float *stream, uint32_t width) {
  const uint32_t t = blockIdx.x;
  const uint32_t *position = p.position + (size_t)t * p.top;
  const float *weight = p.weight + (size_t)t * p.top;
  if (width % 8 == 0) {
    const uint32_t c = (blockIdx.y * 256 + threadIdx.x) * 8;
    if (c >= width) return;
    f32x8 sum = *reinterpret_cast<f32x8 *>(stream + (size_t)t * width + c);
#pragma unroll 4
    for (uint32_t s = 0; s < p.top; ++s) {
      const Frag<T> row = *reinterpret_cast<const Frag<T> *>(rows + (size_t)position[s] * width + c);
#pragma unroll
      for (int e = 0; e < 8; ++e) sum[e] = fmaf(weight[s], to_f32(row[e]), sum[e]);
    }
    *reinterpret_cast<f32x8 *>(stream + (size_t)t * width + c) = sum;
    return;
  }
  for (uint32_t c = blockIdx.y * 2048 + threadIdx.x; c < min(width, (blockIdx.y + 1) * 2048); c += 256) {
    float sum = 0.0f;
    for (uint32_t s = 0; s < p.top; ++s) sum = fmaf(weight[s], to_f32(rows[(size_t)position[s] * width + c]), sum);
    stream[(size_t)t * width + c] += sum;
  }
}

}  // namespace

uint32_t route_tile_rows(uint32_t m, uint32_t experts, uint32_t top, uint32_t width, uint32_t ff, bool f32) {
  return !f32 && width % 64 == 0 && ff % 64 == 0 && (uint64_t)m * top >= 96 * (uint64_t)experts ? 128 : 64;
}

uint32_t route_max_tiles(uint32_t m, uint32_t experts, uint32_t top, uint32_t tile) {
  const uint64_t pairs = (uint64_t)m * top;
  return (uint32_t)(pairs / tile + std::min<uint64_t>(experts, pairs));
}

hipError_t launch_route(const RoutePlan &p, hipStream_t stream) {
  const size_t bytes = 4 * (p.experts + p.top) * 4;
  if (bytes > 60 * 1024) return hipErrorInvalidValue;
  route_select_kernel<<<(p.m + 3) / 4, 256, bytes, stream>>>(p);
  if (hipError_t status = hipGetLastError()) return status;
  route_sort_kernel<<<1, 1024, 3 * p.experts * 4, stream>>>(p);
  return hipGetLastError();
}

hipError_t launch_route_combine(const RouteCombineArgs &a, hipStream_t stream) {
  const RoutePlan &p = *a.plan;
  if (a.f32)
    route_combine_kernel<float><<<dim3(p.m, (a.width + 2047) / 2048), 256, 0, stream>>>(p, static_cast<const float *>(a.rows), a.stream, a.width);
  else
    route_combine_kernel<__bf16><<<dim3(p.m, (a.width + 2047) / 2048), 256, 0, stream>>>(p, static_cast<const __bf16 *>(a.rows), a.stream, a.width);
  return hipGetLastError();
}

}  // namespace llmopt
