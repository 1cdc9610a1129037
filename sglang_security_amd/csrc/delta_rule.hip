// The gated delta rule over heads with a matrix state, batched over sequences with carried state.  Per head, with unit
// vectors k and q (q also times dim^-1/2), a decay g and a step size beta per token:
//
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q;   out = out_scale * norm(o) * w * silu(gate)
//
// Rows of a step belong to sequences (short_conv.h); states are fp32, [dp][vp] per head and slot, zeros in the padding.
//
//   short_conv     convolution and activation of the q, k and v channels; the states of the convolution
//   delta_step     one sequence and head per block, row after row, the state in registers: single rows, and
//                  portions of any type and size
//
// The state is read once per row: o = g S^T q + (k . q) u needs the products of the old state only.  The unit norms stay
// factors on the products of the convolution's outputs, so they are never rounded to the activation type.
#include <algorithm>

#include "common.h"
#include "row_source.h"
#include "short_conv.h"

namespace sglk {

template <typename T, int R, int ACT>
__global__ void __launch_bounds__(256) short_conv_kernel(ShortConv a) {
  const int nv = a.W / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)((a.M + R - 1) / R) * nv) return;
  short_conv_rows<T, R, ACT>(a, (int)(idx / nv) * R, (int)(idx % nv) * 8);
}

template <typename T>
__global__ void __launch_bounds__(256) short_conv_state_kernel(ShortConv a, int seq0) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c < a.W) conv_state_update<T>(a, seq0 + blockIdx.y, c);
}

constexpr float kUnitEps = 1e-6f;

struct DeltaRule {
  const void* u;       // [rows, u_stride]: KH heads of dp query channels, KH of dp key channels, VH of vp value channels
  int64_t u_stride;
  RowSource src;       // columns: VH heads of vp gate channels, b_col .. step sizes, a_col .. decays before their activations
  int b_col, a_col;
  const float* rate;   // [VH] exp(A_log)
  const float* dt;     // [VH]
  const float* norm;   // [vp]
  float* state;        // [slots][VH][dp][vp]
  void* out;           // [rows, out_stride]: head h at h * vp
  int64_t out_stride;
  RecurrentSeqs seq;
  int KH, VH, dp, vp, vdim;
  float q_scale, out_scale, eps;
};

// log of the decay and the step size of a row's head
template <typename T>
__device__ __forceinline__ void delta_gates(const DeltaRule& a, int m, int h, float& log_g, float& beta) {
  beta = sigmoidf(source1<T>(a.src, m, a.b_col + h));
  log_g = -a.rate[h] * softplusf(source1<T>(a.src, m, a.a_col + h) + a.dt[h]);
}

// sums of three values over the block of 256 threads; red: 12 floats
__device__ __forceinline__ void block_sum3(float& x, float& y, float& z, float* red) {
  x = wave_sum(x);
  y = wave_sum(y);
  z = wave_sum(z);
  if ((threadIdx.x & 63) == 0) {
    const int w = threadIdx.x >> 6;
    red[w] = x;
    red[4 + w] = y;
    red[8 + w] = z;
  }
  __syncthreads();
  x = red[0] + red[1] + red[2] + red[3];
  y = red[4] + red[5] + red[6] + red[7];
  z = red[8] + red[9] + red[10] + red[11];
}

__host__ __device__ inline int delta_step_lds(int dp, int vp) { return (2 * dp + 2 * (256 / (vp / 4)) * vp + vp) * 4; }

// Block: one head of one sequence.  Thread (rg, cg) owns the columns 4 cg .. + 3 of the state's rows rg, rg + RG, ...; NR of
// them per thread in registers (NR = 0: any number, the state stays in memory).
template <typename T, int NR>
__global__ void __launch_bounds__(256) delta_step_kernel(DeltaRule a, int seq0) {
  extern __shared__ __attribute__((aligned(16))) float delta_lds[];
  __shared__ float red3[12], red1[4];
  const int h = blockIdx.x, s = seq0 + blockIdx.y;
  const int CG = a.vp / 4, RG = 256 / CG;
  const int cg = threadIdx.x % CG, rg = threadIdx.x / CG;
  const bool mine = rg < RG;
  float* kx = delta_lds;            // [dp] key channels, then [dp] query channels
  float* qx = kx + a.dp;
  float* part = qx + a.dp;          // [2][RG][vp]
  float* ub = part + 2 * RG * a.vp;  // [vp]
  const int n = a.seq.rows[s], row0 = a.seq.row0[s];
  const bool fresh = a.seq.start[s] == 0;
  float* sp = a.state + ((int64_t)a.seq.slot[s] * a.VH + h) * a.dp * a.vp + 4 * cg;
  const int kh = h / (a.VH / a.KH);
  const float4v zero = float4v{0.f, 0.f, 0.f, 0.f};
  float4v S[NR > 0 ? NR : 1];
  if constexpr (NR > 0) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int r = rg + RG * i;
      S[i] = mine && r < a.dp && !fresh ? *reinterpret_cast<const float4v*>(sp + (int64_t)r * a.vp) : zero;
    }
  } else if (fresh && mine) {
    for (int r = rg; r < a.dp; r += RG) *reinterpret_cast<float4v*>(sp + (int64_t)r * a.vp) = zero;
  }
  for (int k = 0; k < n; ++k) {
    const int m = row0 + k;
    const int64_t uq = (int64_t)m * a.u_stride + kh * a.dp, uk = uq + a.KH * a.dp;
    const int64_t uv = (int64_t)m * a.u_stride + 2 * a.KH * a.dp + h * a.vp;
    float sk = 0.f, sq = 0.f, dot = 0.f;
    for (int d = threadIdx.x; d < a.dp; d += 256) {
      const float kv = ld<T>(a.u, uk + d), qv = ld<T>(a.u, uq + d);
      kx[d] = kv;
      qx[d] = qv;
      sk += kv * kv;
      sq += qv * qv;
      dot += kv * qv;
    }
    float log_g, beta;
    delta_gates<T>(a, m, h, log_g, beta);
    const float g = expf(log_g);
    block_sum3(sk, sq, dot, red3);
    const float rk = 1.0f / sqrtf(sk + kUnitEps), rq = a.q_scale / sqrtf(sq + kUnitEps);
    if (mine) {
      float4v ak = zero, aq = zero;
      if constexpr (NR > 0) {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          const int r = min(rg + RG * i, a.dp - 1);  // rows past the state are zero
          ak += S[i] * kx[r];
          aq += S[i] * qx[r];
        }
      } else {
        for (int r = rg; r < a.dp; r += RG) {
          const float4v v = *reinterpret_cast<const float4v*>(sp + (int64_t)r * a.vp);
          ak += v * kx[r];
          aq += v * qx[r];
        }
      }
      *reinterpret_cast<float4v*>(part + rg * a.vp + 4 * cg) = ak;
      *reinterpret_cast<float4v*>(part + (RG + rg) * a.vp + 4 * cg) = aq;
    }
    __syncthreads();
    float so = 0.f;
    constexpr int OV = 4;  // vp <= 1024
    float o[OV];
#pragma unroll
    for (int i = 0; i < OV; ++i) {
      const int c = threadIdx.x + 256 * i;
      o[i] = 0.f;
      if (c >= a.vp) continue;
      float s1 = 0.f, s2 = 0.f;
      for (int r = 0; r < RG; ++r) {
        s1 += part[r * a.vp + c];
        s2 += part[(RG + r) * a.vp + c];
      }
      const float u = beta * (ld<T>(a.u, uv + c) - g * rk * s1);
      ub[c] = u * rk;
      o[i] = g * rq * s2 + u * (dot * rk * rq);
      so += o[i] * o[i];
    }
    so = wave_sum(so);
    if ((threadIdx.x & 63) == 0) red1[threadIdx.x >> 6] = so;
    __syncthreads();
    so = red1[0] + red1[1] + red1[2] + red1[3];
    if (mine) {
      const float4v u = *reinterpret_cast<const float4v*>(ub + 4 * cg);
      if constexpr (NR > 0) {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          const int r = rg + RG * i;
          if (r < a.dp) S[i] = S[i] * g + u * kx[r];
        }
      } else {
        for (int r = rg; r < a.dp; r += RG) {
          float4v* p = reinterpret_cast<float4v*>(sp + (int64_t)r * a.vp);
          *p = *p * g + u * kx[r];
        }
      }
    }
    const float inv = a.out_scale / sqrtf(so / (float)a.vdim + a.eps);
#pragma unroll
    for (int i = 0; i < OV; ++i) {
      const int c = threadIdx.x + 256 * i;
      if (c >= a.vp) continue;
      const float z = source1<T>(a.src, m, h * a.vp + c);
      const float gate = sizeof(typename Raw<T>::type) == 2 ? silu_fast(z) : activate(z, 3);
      st<T>(a.out, m * a.out_stride + h * a.vp + c, o[i] * inv * a.norm[c] * gate);
    }
    __syncthreads();  // the rows in LDS are read until here
  }
  if constexpr (NR > 0) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int r = rg + RG * i;
      if (mine && r < a.dp) *reinterpret_cast<float4v*>(sp + (int64_t)r * a.vp) = S[i];
    }
  }
}

}  // namespace sglk

using namespace sglk;

#define SGLK_DELTA_ARGS                                                                                                       \
  const void *u, int64_t u_stride, const void *src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, int b_col, \
      int a_col, const float *rate, const float *dt, const float *norm, float *state, void *out, int64_t out_stride,          \
      const int32_t *row_seq, const int32_t *row0, const int32_t *rows, const int32_t *start, const int32_t *slot, int M,      \
      int kv_heads, int heads, int dp, int vp, int dim, int vdim, float out_scale, float eps
#define SGLK_DELTA_MAKE                                                                                                   \
  const DeltaRule a { u, u_stride, RowSource{src, src_f32, splits, part_stride, src_stride}, b_col, a_col, rate, dt, norm, \
                      state, out, out_stride, RecurrentSeqs{row_seq, row0, rows, start, slot}, kv_heads, heads, dp, vp,    \
                      vdim, 1.0f / sqrtf((float)dim), out_scale, eps }

static int check_delta(const DeltaRule& a, int M, int dim, int seq0, int n_seqs, int dtype, const char* what) {
  SGLK_CHECK(M >= 0 && a.KH > 0 && a.VH > 0 && a.VH % a.KH == 0 && dim > 0 && a.vdim > 0 && a.dp >= dim && a.vp >= a.vdim &&
                 a.dp % 8 == 0 && a.vp % 8 == 0 && a.vp <= 1024 && a.dp <= 4096 && seq0 >= 0 && seq0 <= n_seqs && n_seqs - seq0 <= 65535,
             "%s: bad shape", what);
  SGLK_CHECK(a.u_stride >= 2 * a.KH * a.dp + a.VH * a.vp && a.u_stride % 8 == 0 && a.out_stride >= a.VH * a.vp && a.out_stride % 8 == 0 &&
                 a.b_col >= a.VH * a.vp && a.a_col >= a.b_col + a.VH,
             "%s: rows too short", what);
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(a.u && a.src.p && a.rate && a.dt && a.norm && a.state && a.out && a.seq.row_seq && a.seq.row0 && a.seq.rows &&
                 a.seq.start && a.seq.slot,
             "%s: null pointer", what);
  SGLK_CHECK(aligned16(a.u) && aligned16(a.state) && aligned16(a.out), "%s: unaligned pointer", what);
  return check_source(a.src.p, a.src.f32, a.src.splits, a.src.part_stride, a.src.stride, a.a_col + a.VH, dtype, what);
}

extern "C" {

int sglk_short_conv(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, const float* bias,
                    const float* conv, const float* conv_b, void* u, void* conv_state, const int32_t* row_seq,
                    const int32_t* row0, const int32_t* rows, const int32_t* start, const int32_t* slot, int M, int W, int taps,
                    int singles, int n_seqs, int act, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && W > 0 && W % 8 == 0 && taps >= 1 && singles >= 0 && singles <= M && singles <= n_seqs && n_seqs - singles <= 65535,
             "short_conv: bad shape");
  SGLK_CHECK(act == 0 || act == 3, "short_conv: act is 0 (none) or 3 (silu)");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && conv && u && row_seq && row0 && rows && start && slot && (conv_state || taps == 1), "short_conv: null pointer");
  SGLK_CHECK(aligned16(u) && aligned16(conv_state) && aligned16(conv), "short_conv: unaligned pointer");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, W, dtype, "short_conv")) return rc;
  const ShortConv a{RowSource{src, src_f32, splits, part_stride, src_stride}, bias, conv, conv_b, u, conv_state,
                    RecurrentSeqs{row_seq, row0, rows, start, slot}, M, W, taps, singles};
  const int per = M >= 256 ? 4 : 1;  // rows per thread
  const int64_t threads = (int64_t)((M + per - 1) / per) * (W / 8);
  const dim3 grid((unsigned)((threads + 255) / 256));
#define SGLK_SC(R, A) hipLaunchKernelGGL((short_conv_kernel<T, R, A>), grid, dim3(256), 0, (hipStream_t)stream, a)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (per == 4 && act == 3)
      SGLK_SC(4, 3);
    else if (per == 4)
      SGLK_SC(4, 0);
    else if (act == 3)
      SGLK_SC(1, 3);
    else
      SGLK_SC(1, 0);
    if (taps > 1 && n_seqs > singles)
      hipLaunchKernelGGL((short_conv_state_kernel<T>), dim3((W + 255) / 256, n_seqs - singles), dim3(256), 0, (hipStream_t)stream,
                         a, singles);
  });
#undef SGLK_SC
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_delta_step(SGLK_DELTA_ARGS, int seq0, int n_seqs, int dtype, void* stream) {
  SGLK_DELTA_MAKE;
  if (int rc = check_delta(a, M, dim, seq0, n_seqs, dtype, "delta_step")) return rc;
  if (M == 0 || n_seqs == seq0) return SGLK_OK;
  const int RG = 256 / (vp / 4), per = (dp + RG - 1) / RG;
  const int lds = delta_step_lds(dp, vp);
  const dim3 grid(heads, n_seqs - seq0);
#define SGLK_DS(NR) hipLaunchKernelGGL((delta_step_kernel<T, NR>), grid, dim3(256), lds, (hipStream_t)stream, a, seq0)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (per <= 4)
      SGLK_DS(4);
    else if (per <= 8)
      SGLK_DS(8);
    else if (per <= 16)
      SGLK_DS(16);
    else if (per <= 32)
      SGLK_DS(32);
    else
      SGLK_DS(0);
  });
#undef SGLK_DS
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}
}
