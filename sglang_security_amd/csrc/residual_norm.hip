// Row kernels around the sublayers of a decoder whose residual stream is kept in fp32 and whose sublayers are normalised
// on both sides: x += norm(sublayer) * w_post, h = norm(x) * w_next in one launch, the embedding and the additions
// in front of a repeated group of layers included; activations of un-gated feed-forwards on the way out of a split
// product; capped fp32 logits; and the request table's new slots.
//
// A sublayer's output arrives either as the fp32 split sums of a product (added up here, in split order) or as finished
// rows of the activation type.  Every row buffer is padded to a multiple of eight elements with zeros in the padding.
#include <algorithm>

#include "common.h"
#include "row_source.h"

namespace sglk {

__device__ __forceinline__ float block_sum256(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();  // red may still be read from an earlier call
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  return red[0] + red[1] + red[2] + red[3];
}

struct ResidualNorm {
  float* x;               // [rows, pitch] residual stream
  const void* embed;      // embedding table [vocab, embed_stride] (or nullptr: x is read)
  const int32_t* ids;
  int64_t embed_stride;
  float embed_scale;
  RowSource src;          // sublayer output (src.p == nullptr: none)
  const float* w_post;    // weight of the norm over src (nullptr: src is added as it is)
  float* x0;              // embedding output: written together with `embed`, else added when add_x0
  int add_x0;
  const float* step;      // vector added to x (or nullptr)
  const float* w_next;    // weight of the norm that produces h (nullptr: no h)
  void* h;                // [out rows, h_stride]
  int64_t h_stride;
  const int32_t* rows;    // out row r works on row rows[r] (nullptr: r)
  int store_x;
  int width, pitch;       // true width, padded row length of x / x0 / h
  float eps;
};

template <typename T, int VPT>
__global__ void __launch_bounds__(256) residual_norm_kernel(ResidualNorm a) {
  __shared__ float red[4];
  const int out_row = blockIdx.x;
  const int row = a.rows ? a.rows[out_row] : out_row;
  const int nv = a.pitch / 8;
  float x[VPT][8], s[VPT][8];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int v = threadIdx.x + 256 * i;
#pragma unroll
    for (int j = 0; j < 8; ++j) x[i][j] = s[i][j] = 0.f;
    if (v >= nv) continue;
    if (a.embed) {
      const int64_t base = (int64_t)a.ids[row] * a.embed_stride + 8 * v;
      ld8<T>(a.embed, base, x[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] *= a.embed_scale;
      if (a.x0) st8<float>(a.x0, (int64_t)row * a.pitch + 8 * v, x[i]);
    } else {
      ld8<float>(a.x, (int64_t)row * a.pitch + 8 * v, x[i]);
    }
    if (a.src.p) {
      source8<T>(a.src, row, 8 * v, s[i]);
#pragma unroll
      for (int j = 0; j < 8; ++j) ss += s[i][j] * s[i][j];
    }
  }
  if (a.src.p) {
    float inv = 1.f;
    if (a.w_post) inv = 1.0f / sqrtf(block_sum256(ss, red) / (float)a.width + a.eps);
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int v = threadIdx.x + 256 * i;
      if (v >= nv) continue;
      float w[8];
      if (a.w_post) {
        ld8<float>(a.w_post, 8 * v, w);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] += s[i][j] * inv * w[j];
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) x[i][j] += s[i][j];
      }
    }
  }
  float xx = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int v = threadIdx.x + 256 * i;
    if (v >= nv) continue;
    float t[8];
    if (a.add_x0) {
      ld8<float>(a.x0, (int64_t)row * a.pitch + 8 * v, t);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += t[j];
    }
    if (a.step) {
      ld8<float>(a.step, 8 * v, t);
#pragma unroll
      for (int j = 0; j < 8; ++j) x[i][j] += t[j];
    }
    if (a.store_x) st8<float>(a.x, (int64_t)row * a.pitch + 8 * v, x[i]);
#pragma unroll
    for (int j = 0; j < 8; ++j) xx += x[i][j] * x[i][j];
  }
  if (a.w_next) {
    const float inv = 1.0f / sqrtf(block_sum256(xx, red) / (float)a.width + a.eps);
#pragma unroll
    for (int i = 0; i < VPT; ++i) {
      const int v = threadIdx.x + 256 * i;
      if (v >= nv) continue;
      float w[8];
      ld8<float>(a.w_next, 8 * v, w);
#pragma unroll
      for (int j = 0; j < 8; ++j) w[j] *= x[i][j] * inv;
      st8<T>(a.h, (int64_t)out_row * a.h_stride + 8 * v, w);
    }
  }
}

// out[m][n] = act(src[m][n] + bias[n]), eight outputs per thread
template <typename T>
__global__ void __launch_bounds__(256) source_act_kernel(RowSource src, const float* __restrict__ bias, void* __restrict__ out,
                                                         int M, int N, int64_t out_stride, int act) {
  const int nv = N / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * nv) return;
  const int m = (int)(idx / nv), n = (int)(idx - (int64_t)m * nv) * 8;
  float v[8];
  source8<T>(src, m, n, v);
  if (bias) {
    float b[8];
    ld8<float>(bias, n, b);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] += b[j];
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = activate(v[j], act);
  st8<T>(out, (int64_t)m * out_stride + n, v);
}

// out[m][n] = act(src[m][n]) * src[m][N + n]: gate columns, then as many others
template <typename T>
__global__ void __launch_bounds__(256) source_gated_act_kernel(RowSource src, void* __restrict__ out, int M, int N,
                                                               int64_t out_stride, int act) {
  const int nv = N / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * nv) return;
  const int m = (int)(idx / nv), n = (int)(idx - (int64_t)m * nv) * 8;
  float v[8], w[8];
  source8<T>(src, m, n, v);
  source8<T>(src, m, N + n, w);
#pragma unroll
  for (int j = 0; j < 8; ++j)
    v[j] = w[j] * (sizeof(typename Raw<T>::type) == 2 && act == 3 ? silu_fast(v[j]) : activate(v[j], act));
  st8<T>(out, (int64_t)m * out_stride + n, v);
}

// logits[m][n] = cap * tanh(src[m][n] / cap) in fp32 (cap <= 0: as they are)
template <typename T>
__global__ void __launch_bounds__(256) capped_logits_kernel(RowSource src, float* __restrict__ out, int M, int N, int V,
                                                            int64_t out_stride, float cap) {
  const int nv = N / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * nv) return;
  const int m = (int)(idx / nv), n = (int)(idx - (int64_t)m * nv) * 8;
  float v[8];
  source8<T>(src, m, n, v);
  if (cap > 0.f) {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = cap * tanhf(v[j] / cap);
  }
  if (n + 8 <= V && (out_stride & 3) == 0) {
    st8<float>(out, (int64_t)m * out_stride + n, v);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (n + j < V) out[(int64_t)m * out_stride + n + j] = v[j];
  }
}

// req_to_token[req[seq[t]]][pos[t]] = loc[t]
__global__ void __launch_bounds__(256) assign_slots_kernel(int32_t* __restrict__ r2t, int64_t stride,
                                                           const int32_t* __restrict__ row_seq, const int32_t* __restrict__ req,
                                                           const int32_t* __restrict__ pos, const int32_t* __restrict__ loc,
                                                           int T) {
  const int t = blockIdx.x * 256 + threadIdx.x;
  if (t < T) r2t[(int64_t)req[row_seq[t]] * stride + pos[t]] = loc[t];
}

}  // namespace sglk

using namespace sglk;

extern "C" {

int sglk_residual_norm(float* x, const void* embed, const int32_t* ids, int64_t embed_stride, float embed_scale,
                       const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride,
                       const float* w_post, float* x0, int add_x0, const float* step, const float* w_next, void* h,
                       int64_t h_stride, const int32_t* rows, int store_x, int M, int width, int pitch, float eps, int dtype,
                       void* stream) {
  SGLK_CHECK(M >= 0 && width > 0 && pitch >= width && pitch % 8 == 0, "residual_norm: bad shape (%d of %d)", width, pitch);
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(x && (embed || src || w_next), "residual_norm: null pointer");
  SGLK_CHECK(!embed || (ids && embed_stride % 8 == 0 && embed_stride >= pitch && aligned16(embed)),
             "residual_norm: embedding rows must be padded to the row length and 16-byte aligned");
  SGLK_CHECK(!add_x0 || (x0 && !embed), "residual_norm: nothing to add");
  SGLK_CHECK(!w_next || (h && h_stride >= pitch && h_stride % 8 == 0 && aligned16(h)), "residual_norm: bad output rows");
  SGLK_CHECK(!rows || !store_x, "residual_norm: picked rows are not stored back");
  SGLK_CHECK(aligned16(x) && (!x0 || aligned16(x0)), "residual_norm: rows must be 16-byte aligned");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, pitch, dtype, "residual_norm")) return rc;
  SGLK_CHECK(pitch <= 8 * 256 * 8, "residual_norm: rows of at most 16384 elements");
  ResidualNorm a{x, embed, ids, embed_stride, embed_scale, RowSource{src, src_f32, splits, part_stride, src_stride}, w_post, x0,
                 add_x0, step, w_next, h, h_stride, rows, store_x, width, pitch, eps};
  const int vecs = pitch / 8;
#define SGLK_RN(V) hipLaunchKernelGGL((residual_norm_kernel<T, V>), dim3(M), dim3(256), 0, (hipStream_t)stream, a)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (vecs <= 256) {
      SGLK_RN(1);
    } else if (vecs <= 512) {
      SGLK_RN(2);
    } else if (vecs <= 1024) {
      SGLK_RN(4);
    } else {
      SGLK_RN(8);
    }
  });
#undef SGLK_RN
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_source_act(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, const float* bias,
                    void* out, int M, int N, int64_t out_stride, int act, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && N > 0 && N % 8 == 0 && out_stride % 8 == 0 && out_stride >= N, "source_act: bad shape");
  SGLK_CHECK(act >= 0 && act <= 3, "source_act: act is 0 (none), 1 (square of relu), 2 (gelu, tanh form) or 3 (silu)");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && out && aligned16(out), "source_act: null or unaligned pointer");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, N, dtype, "source_act")) return rc;
  const int64_t vecs = (int64_t)M * (N / 8);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((source_act_kernel<T>), dim3((unsigned)((vecs + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, RowSource{src, src_f32, splits, part_stride, src_stride}, bias,
                                         out, M, N, out_stride, act));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_source_gated_act(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, void* out, int M,
                          int N, int64_t out_stride, int act, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && N > 0 && N % 8 == 0 && out_stride % 8 == 0 && out_stride >= N, "source_gated_act: bad shape");
  SGLK_CHECK(act >= 0 && act <= 3, "source_gated_act: act is 0 (none), 1 (square of relu), 2 (gelu, tanh form) or 3 (silu)");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && out && aligned16(out), "source_gated_act: null or unaligned pointer");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, 2 * N, dtype, "source_gated_act")) return rc;
  const int64_t vecs = (int64_t)M * (N / 8);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((source_gated_act_kernel<T>), dim3((unsigned)((vecs + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, RowSource{src, src_f32, splits, part_stride, src_stride}, out, M,
                                         N, out_stride, act));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_capped_logits(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, float* out, int M,
                       int N, int V, int64_t out_stride, float cap, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && V > 0 && N >= V && N % 8 == 0 && out_stride >= V, "capped_logits: bad shape");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && out && aligned16(out), "capped_logits: null or unaligned pointer");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, N, dtype, "capped_logits")) return rc;
  const int64_t vecs = (int64_t)M * (N / 8);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((capped_logits_kernel<T>), dim3((unsigned)((vecs + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, RowSource{src, src_f32, splits, part_stride, src_stride}, out, M,
                                         N, V, out_stride, cap));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_assign_slots(int32_t* req_to_token, int64_t row_stride, const int32_t* row_seq, const int32_t* req,
                      const int32_t* positions, const int32_t* loc, int T, void* stream) {
  SGLK_CHECK(T >= 0 && row_stride > 0, "assign_slots: bad shape");
  if (T == 0) return SGLK_OK;
  SGLK_CHECK(req_to_token && row_seq && req && positions && loc, "assign_slots: null pointer");
  hipLaunchKernelGGL(assign_slots_kernel, dim3((T + 255) / 256), dim3(256), 0, (hipStream_t)stream, req_to_token, row_stride,
                     row_seq, req, positions, loc, T);
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}
}
