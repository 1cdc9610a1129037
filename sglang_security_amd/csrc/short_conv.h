// Short causal convolutions over time, one filter per channel, batched over sequences with carried state: the last
// taps - 1 inputs of a sequence, of the activation type.
//
// Rows of a step belong to sequences; a sequence has its first row, its number of rows, the position of its first row
// (0: what lies in front counts as zero, so a state slot needs no clearing) and its state slot.  The first `singles` rows
// are sequences of one row.
#pragma once
#include "common.h"
#include "row_source.h"

namespace sglk {

struct RecurrentSeqs {
  const int32_t* row_seq;  // sequence of a row
  const int32_t* row0;     // first row of a sequence
  const int32_t* rows;     // number of its rows
  const int32_t* start;    // position of its first row
  const int32_t* slot;     // its state slot
};

struct ShortConv {
  RowSource src;          // columns [0, W): the inputs without their bias
  const float* bias;      // [W] (or nullptr)
  const float* conv;      // [taps][W], last tap: the row itself
  const float* conv_b;    // [W] (or nullptr)
  void* u;                // [rows, W]
  void* state;            // [slots][taps - 1][W]
  RecurrentSeqs seq;
  int M, W, taps, singles;
};

__device__ __forceinline__ void ld8_or_zero(const float* p, int c, float (&v)[8]) {
  if (p) {
    ld8<float>(p, c, v);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = 0.f;
  }
}

// convolution input of row m, as the activation type holds it
template <typename T>
__device__ __forceinline__ void conv_input8(const ShortConv& a, int m, int c, const float (&bias)[8], float (&x)[8]) {
  source8<T>(a.src, m, c, x);
#pragma unroll
  for (int j = 0; j < 8; ++j) x[j] = round_to<T>(x[j] + bias[j]);
}

// ACT of activate() on the result; the hardware exponential where the result is rounded to 16 bits
template <typename T, int ACT>
__device__ __forceinline__ float conv_act(float z) {
  if constexpr (ACT == 3 && sizeof(typename Raw<T>::type) == 2) return silu_fast(z);
  return activate(z, ACT);
}

// Channels c .. c + 7 of rows m0 .. m0 + R - 1 into u; for single rows also the shift of the state.
template <typename T, int R, int ACT>
__device__ __forceinline__ void short_conv_rows(const ShortConv& a, int m0, int c) {
  float bias[8], acc[8];
  ld8_or_zero(a.bias, c, bias);
  const int keep = a.taps - 1;
  if constexpr (R > 1) {
    // four taps, rows of one sequence with everything they need in this step: every input is formed once
    const int s = a.seq.row_seq[m0];
    if (keep == 3 && m0 + R <= a.M && a.seq.row_seq[m0 + R - 1] == s && m0 - a.seq.row0[s] >= 3) {
      float x[R + 3][8], w[4][8], cb[8];
#pragma unroll
      for (int r = 0; r < R + 3; ++r) conv_input8<T>(a, m0 - 3 + r, c, bias, x[r]);
#pragma unroll
      for (int t = 0; t < 4; ++t) ld8<float>(a.conv, (int64_t)t * a.W + c, w[t]);
      ld8_or_zero(a.conv_b, c, cb);
#pragma unroll
      for (int r = 0; r < R; ++r) {
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          acc[j] = cb[j];
#pragma unroll
          for (int t = 0; t < 4; ++t) acc[j] = fmaf(x[r + t][j], w[t][j], acc[j]);
          acc[j] = conv_act<T, ACT>(acc[j]);
        }
        st8<T>(a.u, (int64_t)(m0 + r) * a.W + c, acc);
      }
      return;
    }
  }
  if constexpr (R == 1) {
    // four taps, a sequence's only row: the whole state and every filter on their way at once
    if (keep == 3 && m0 < a.singles) {
      const int s = a.seq.row_seq[m0];
      const int64_t st0 = (int64_t)a.seq.slot[s] * 3 * a.W + c;
      float x[4][8], w[4][8];
      conv_input8<T>(a, m0, c, bias, x[3]);
#pragma unroll
      for (int t = 0; t < 4; ++t) ld8<float>(a.conv, (int64_t)t * a.W + c, w[t]);
      ld8_or_zero(a.conv_b, c, acc);
#pragma unroll
      for (int j = 0; j < 3; ++j) ld8<T>(a.state, st0 + (int64_t)j * a.W, x[j]);
      const bool fresh = a.seq.start[s] == 0;
#pragma unroll
      for (int j = 0; j < 3; ++j)
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] = fresh ? 0.f : x[j][e];
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] = fmaf(x[t][e], w[t][e], acc[e]);
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = conv_act<T, ACT>(acc[e]);
      st8<T>(a.u, (int64_t)m0 * a.W + c, acc);
#pragma unroll
      for (int j = 0; j < 3; ++j) st8<T>(a.state, st0 + (int64_t)j * a.W, x[j + 1]);
      return;
    }
  }
  for (int m = m0; m < min(m0 + R, a.M); ++m) {
    const int s = a.seq.row_seq[m];
    const int start = a.seq.start[s];
    const int k = m - a.seq.row0[s];  // row within its sequence's portion
    const int64_t st0 = (int64_t)a.seq.slot[s] * keep * a.W + c;
    float x[8], w[8];
    ld8_or_zero(a.conv_b, c, acc);
    for (int d = keep; d >= 0; --d) {  // d rows back
      if (k - d >= 0) {
        conv_input8<T>(a, m - d, c, bias, x);
      } else if (start > 0) {
        ld8<T>(a.state, st0 + (int64_t)(keep + k - d) * a.W, x);
      } else {
        continue;
      }
      ld8<float>(a.conv, (int64_t)(keep - d) * a.W + c, w);
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = fmaf(x[j], w[j], acc[j]);
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] = conv_act<T, ACT>(acc[j]);
    st8<T>(a.u, (int64_t)m * a.W + c, acc);
    if (m < a.singles && keep > 0) {
      // x holds the row's own input: shift the state by one
      float o[8];
      for (int j = 0; j + 1 < keep; ++j) {
        if (start > 0) {
          ld8<T>(a.state, st0 + (int64_t)(j + 1) * a.W, o);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) o[e] = 0.f;
        }
        st8<T>(a.state, st0 + (int64_t)j * a.W, o);
      }
      st8<T>(a.state, st0 + (int64_t)(keep - 1) * a.W, x);
    }
  }
}

// the last taps - 1 inputs of a sequence with n rows in this step, one channel per thread (ascending: what is read lies
// ahead of what is written)
template <typename T>
__device__ __forceinline__ void conv_state_update(const ShortConv& a, int s, int c) {
  const int n = a.seq.rows[s], start = a.seq.start[s], keep = a.taps - 1;
  const int64_t st0 = (int64_t)a.seq.slot[s] * keep * a.W + c;
  for (int j = 0; j < keep; ++j) {
    const int k = n - keep + j;
    float v = 0.f;
    if (k >= 0)
      v = source1<T>(a.src, a.seq.row0[s] + k, c) + (a.bias ? a.bias[c] : 0.f);
    else if (start > 0)
      v = ld<T>(a.state, st0 + (int64_t)(n + j) * a.W);
    st<T>(a.state, st0 + (int64_t)j * a.W, v);
  }
}

}  // namespace sglk
