// Writing a step's values into the (transposed) value pages [page, kv_head, dv, slot]; shared by the kernels that prepare heads.
#pragma once

#include "common.h"

namespace {

// What becomes of a token's values on their way from the projection into the pages:
//   bias    a value per column of the projection row (null: none), added first;
//   first   [tokens, nkv * dv] in the activation dtype, or null.  mix null: the values are left there as well, for later layers
//           of the step to mix with; mix given: v <- (1 - mix[0]) v + mix[0] first.
template <typename T>
struct ValuePath {
  const float* bias;
  T* first;
  const float* mix;
};

template <typename T>
__device__ __forceinline__ T value_on_its_way(const ValuePath<T>& path, T raw, int column, int64_t token, int vn, int e) {
  // column: of the projection row; e: of the values alone (0 .. vn - 1)
  if (!path.bias && !path.first) return raw;
  float v = to_float(raw) + (path.bias ? path.bias[column] : 0.f);
  if (path.mix) {
    const float lambda = path.mix[0];
    v = (1.f - lambda) * v + lambda * to_float(path.first[token * vn + e]);
  }
  const T out = from_float<T>(v);
  if (path.first && !path.mix) path.first[token * vn + e] = out;
  return out;
}

// One token's values into its slot by `threads` threads (this one is `tid`), four at a time: every load of the four is on its way
// before the first is used.
template <typename T>
__device__ __forceinline__ void store_values(const ValuePath<T>& path, const T* __restrict__ row, int v_offset, int64_t token, int nkv, int dv,
                                             T* __restrict__ v_pages, int64_t page, int64_t off, int page_size, int tid, int threads) {
  constexpr int AT_ONCE = 4;
  const int vn = nkv * dv;
  const float lambda = path.mix ? path.mix[0] : 0.f;
  for (int e0 = tid; e0 < vn; e0 += threads * AT_ONCE) {
    T raw[AT_ONCE], first[AT_ONCE];
    float bias[AT_ONCE];
#pragma unroll
    for (int n = 0; n < AT_ONCE; ++n) {
      const int e = min(e0 + n * threads, vn - 1);
      raw[n] = row[v_offset + e];
      bias[n] = path.bias ? path.bias[v_offset + e] : 0.f;
      first[n] = path.mix ? path.first[token * vn + e] : raw[n];
    }
#pragma unroll
    for (int n = 0; n < AT_ONCE; ++n) {
      const int e = e0 + n * threads;
      if (e >= vn) break;
      float v = to_float(raw[n]) + bias[n];
      if (path.mix) v = (1.f - lambda) * v + lambda * to_float(first[n]);
      const T out = from_float<T>(v);
      if (path.first && !path.mix) path.first[token * vn + e] = out;
      v_pages[((page * nkv + e / dv) * dv + e % dv) * page_size + off] = out;
    }
  }
}

// The values of 16 consecutive tokens of the step and one kv head into the value pages, for steps of many tokens: tokens that
// follow each other inside a page lie side by side there, so a thread gathers one dim of 16 / sizeof(T) such tokens
// (neighbouring lanes read neighbouring dims of one token) and writes one 16-byte store; where a run is broken (a page's edge,
// another request, a slot that is not stored) it stores one by one.
template <typename T>
__global__ __launch_bounds__(256) void values_in_runs_kernel(const T* __restrict__ qkv, int row_stride, int v_offset, int tokens, int nkv, int dv,
                                                             T* __restrict__ v_pages, const int* __restrict__ slots, int page_size,
                                                             ValuePath<T> path) {
  constexpr int RUN = 16 / sizeof(T);
  typedef T vec __attribute__((ext_vector_type(RUN)));
  __shared__ int slot_of[16];
  const int tid = threadIdx.x, token0 = blockIdx.x * 16, kvh = blockIdx.y;
  if (tid < 16) slot_of[tid] = token0 + tid < tokens ? slots[token0 + tid] : -1;
  __syncthreads();
  for (int e = tid; e < dv * (16 / RUN); e += 256) {
    const int dim = e % dv, first = (e / dv) * RUN;
    const int slot0 = slot_of[first];
    bool run = slot0 >= 0 && slot0 % RUN == 0 && slot0 % page_size + RUN <= page_size;
#pragma unroll
    for (int i = 1; i < RUN; ++i) run = run && slot_of[first + i] == slot0 + i;
    const int place = kvh * dv + dim, column = v_offset + place;
    const T* src = qkv + (int64_t)(token0 + first) * row_stride + column;
    if (run) {
      vec v;
#pragma unroll
      for (int i = 0; i < RUN; ++i) v[i] = value_on_its_way(path, src[(int64_t)i * row_stride], column, token0 + first + i, nkv * dv, place);
      const int64_t page = slot0 / page_size, off = slot0 % page_size;
      *(vec*)(v_pages + ((page * nkv + kvh) * dv + dim) * page_size + off) = v;
    } else {
#pragma unroll
      for (int i = 0; i < RUN; ++i) {
        const int slot = slot_of[first + i];
        if (slot < 0) continue;
        const int64_t page = slot / page_size, off = slot % page_size;
        v_pages[((page * nkv + kvh) * dv + dim) * page_size + off] =
            value_on_its_way(path, src[(int64_t)i * row_stride], column, token0 + first + i, nkv * dv, place);
      }
    }
  }
}

}  // namespace
