// A product's result as its consumer kernel reads it: fp32 split sums partial[split][row][col] that have not been added
// up yet (splits >= 1), or finished rows of the activation type.
#pragma once
#include "common.h"

namespace sglk {

// eight consecutive elements of an array of T, 16-byte aligned
template <typename T>
__device__ __forceinline__ void ld8(const void* p, int64_t i, float (&v)[8]) {
  if constexpr (sizeof(typename Raw<T>::type) == 4) {
    const float4v a = *reinterpret_cast<const float4v*>(reinterpret_cast<const float*>(p) + i);
    const float4v b = *reinterpret_cast<const float4v*>(reinterpret_cast<const float*>(p) + i + 4);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      v[j] = a[j];
      v[4 + j] = b[j];
    }
  } else {
    const short8 a = *reinterpret_cast<const short8*>(reinterpret_cast<const uint16_t*>(p) + i);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = Conv<T>::to_f32((uint16_t)a[j]);
  }
}

template <typename T>
__device__ __forceinline__ void st8(void* p, int64_t i, const float (&v)[8]) {
  if constexpr (sizeof(typename Raw<T>::type) == 4) {
    float* q = reinterpret_cast<float*>(p) + i;
    *reinterpret_cast<float4v*>(q) = float4v{v[0], v[1], v[2], v[3]};
    *reinterpret_cast<float4v*>(q + 4) = float4v{v[4], v[5], v[6], v[7]};
  } else {
    short8 o;
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = (short)Conv<T>::from_f32(v[j]);
    *reinterpret_cast<short8*>(reinterpret_cast<uint16_t*>(p) + i) = o;
  }
}

template <typename T>
__device__ __forceinline__ float round_to(float v) {
  return Conv<T>::to_f32(Conv<T>::from_f32(v));
}

struct RowSource {
  const void* p;
  int f32;              // 1: split sums, 0: rows of T
  int splits;
  int64_t part_stride;  // floats from one split to the next
  int64_t stride;       // elements from one row to the next
};

template <typename T>
__device__ __forceinline__ void source8(const RowSource& s, int64_t row, int col, float (&v)[8]) {
  if (s.f32)
    sum_partials(reinterpret_cast<const float*>(s.p), s.splits, s.part_stride, row * s.stride + col, v);
  else
    ld8<T>(s.p, row * s.stride + col, v);
}

// one element; the splits are added in the same order
template <typename T>
__device__ __forceinline__ float source1(const RowSource& s, int64_t row, int col) {
  if (!s.f32) return ld<T>(s.p, row * s.stride + col);
  float v = 0.f;
  for (int k = 0; k < s.splits; ++k) v += reinterpret_cast<const float*>(s.p)[k * s.part_stride + row * s.stride + col];
  return v;
}

__device__ __forceinline__ float gelu_tanh(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// the same through the hardware exponential and reciprocal, for results that are rounded to 16 bits
__device__ __forceinline__ float gelu_tanh_fast(float z) {
  const float t = 0.7978845608028654f * (z + 0.044715f * z * z * z);
  return z * (1.0f - __builtin_amdgcn_rcpf(1.0f + __expf(2.0f * t)));
}

__device__ __forceinline__ float sigmoidf(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf(float z) { return z > 20.f ? z : log1pf(expf(z)); }

__device__ __forceinline__ float silu_fast(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

// 0 none, 1 square of relu, 2 gelu (tanh form), 3 silu
__device__ __forceinline__ float activate(float z, int act) {
  if (act == 1) {
    const float r = fmaxf(z, 0.f);
    return r * r;
  }
  if (act == 3) return z / (1.0f + expf(-z));
  return act == 2 ? gelu_tanh(z) : z;
}

inline int check_source(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, int cols, int dtype,
                        const char* what) {
  if (!src) return SGLK_OK;
  SGLK_CHECK(aligned16(src) && src_stride % 8 == 0 && src_stride >= cols, "%s: source rows must be 16-byte aligned and hold %d columns",
             what, cols);
  SGLK_CHECK(!src_f32 || (splits >= 1 && part_stride % 4 == 0), "%s: bad split count", what);
  SGLK_CHECK(src_f32 || dtype != SGLK_F32, "%s: fp32 rows are split sums of one split", what);
  return SGLK_OK;
}

}  // namespace sglk
