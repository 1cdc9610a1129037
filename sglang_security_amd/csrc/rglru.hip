// Gated linear recurrences behind a short causal convolution, batched over sequences with carried state.
//
//   S_t = a_t S_(t-1) + sqrt(1 - a_t^2) i_t u_t,   a_t = exp(-8 r_t softplus(lambda)),   out_t = S_t * y_t
//
// with u the convolution of the x branch, y = gelu(y branch), and r, i = sigmoid of block-diagonal products of u.
//
// Rows of a step belong to sequences; a sequence has its first row, its number of rows, the position of its first row
// (0: the state counts as zero, so a state slot needs no clearing) and its state slot.  The first `singles` rows are
// sequences of one row.
//
//   rglru_conv        bias + convolution of the x branch, bias + gelu of the y branch; for single rows also the shift of
//                     the convolution state
//   rglru_step        single rows: gates on the matrix cores, state update, output
//   rglru_gates       other rows, 64 of a sequence per block: gates on the matrix cores, the recurrence inside the 64 rows
//                     (from zero) and the product of its decays
//   rglru_carry       walks the 64-row tiles of every sequence: state in front of each tile, final states
//   rglru_apply       state in front of the tile * product of decays + local state, times y
//   rglru_rows_*      any type and block size: gates one output per thread, recurrence one channel per thread
//
// Channels are stored block by block, every block padded to a multiple of 32 with zero weights, so padded channels
// stay zero.  Gates, decays, states and their products are fp32; u, y and the convolution's inputs are of the activation
// type.
#include <algorithm>

#include "attention_tile.h"
#include "common.h"
#include "row_source.h"
#include "short_conv.h"

namespace sglk {

constexpr int kScanTile = 64;
constexpr int kGateMaxBlock = 1024;
constexpr int gate_lds(int bwp) { return kScanTile * (bwp * 2 + 16); }


// decay and input weight of a channel from its two gate pre-activations and softplus(lambda)
__device__ __forceinline__ void gate_terms(float zr, float zi, float sp, float u, float& a, float& b) {
  const float la = -8.0f * sigmoidf(zr) * sp;
  a = expf(la);
  b = sqrtf(fmaxf(-expm1f(2.0f * la), 0.f)) * sigmoidf(zi) * u;
}

// The tile kernels' form on the hardware exponential (base 2) and reciprocal.  zr, zi: products without their biases; nbr, nbi:
// biases * -log2(e); sp8: softplus(lambda) * -8 log2(e).  1 - a^2 by its series where it is small.
constexpr float kLog2e = 1.4426950408889634f;
__device__ __forceinline__ void gate_terms_fast(float zr, float zi, float nbr, float nbi, float sp8, float u, float& a, float& b) {
  const float sr = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(fmaf(zr, -kLog2e, nbr)));
  const float si = __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(fmaf(zi, -kLog2e, nbi)));
  const float la = sr * sp8;  // log2 of the decay
  a = __builtin_amdgcn_exp2f(la);
  const float x = la * (2.0f / kLog2e);
  const float near = -x * fmaf(x, fmaf(x, fmaf(x, 0.041666667f, 0.16666667f), 0.5f), 1.0f);
  b = __builtin_amdgcn_sqrtf(x > -0.03f ? near : fmaf(-a, a, 1.0f)) * si * u;
}

// the convolution of the x branch (columns [0, W) of its source) beside the y branch (columns [W, 2 W))
struct RglruConv : ShortConv {
  const float* by;        // [W]
  void* y;                // [rows, W]
};

// One thread: eight channels of R rows; blockIdx.y 0: the x branch, 1: the y branch.
template <typename T, int R>
__global__ void __launch_bounds__(256) rglru_conv_kernel(RglruConv a) {
  const int nv = a.W / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)((a.M + R - 1) / R) * nv) return;
  const int m0 = (int)(idx / nv) * R, c = (int)(idx % nv) * 8;
  if (blockIdx.y == 0) {
    short_conv_rows<T, R, 0>(a, m0, c);
    return;
  }
  float bias[8], acc[8];
  ld8<float>(a.by, c, bias);
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int m = m0 + r;
    if (m >= a.M) break;
    source8<T>(a.src, m, a.W + c, acc);
#pragma unroll
    for (int j = 0; j < 8; ++j)
      acc[j] = sizeof(typename Raw<T>::type) == 4 ? gelu_tanh(acc[j] + bias[j]) : gelu_tanh_fast(acc[j] + bias[j]);
    st8<T>(a.y, (int64_t)m * a.W + c, acc);
  }
}

struct RglruGates {
  const uint16_t* u;       // [rows, W]
  const uint16_t* wr;      // [blocks][bwp / 16][bwp / 32][64 lanes][8]
  const uint16_t* wi;
  const float* br;         // [W]
  const float* bi;
  const float* sp;         // softplus(lambda) [W]
  int M, W, bwp;
};

// 64 rows of u of one block of channels into LDS; rows from `valid` on are zero
__device__ __forceinline__ void park_u(char* lds, const uint16_t* u, int64_t W, int row0, int valid, int col0, int bwp) {
  const int pitch = bwp * 2 + 16;
  const int row = threadIdx.x >> 2, q = threadIdx.x & 3;
  const uint16_t* src = u + (int64_t)(row0 + min(row, valid - 1)) * W + col0;
  for (int c = q; c < bwp / 8; c += 4)
    *reinterpret_cast<int4v*>(lds + row * pitch + 16 * c) =
        row < valid ? *reinterpret_cast<const int4v*>(src + 8 * c) : int4v{0, 0, 0, 0};
}

// Single rows: a block owns 16 channels, wave w rows 16 w .. of the block's 64; S in place, out = S * y.
__global__ void __launch_bounds__(256) rglru_step_kernel(RglruGates a, const uint16_t* __restrict__ y, float* __restrict__ state,
                                                         const int32_t* __restrict__ start, const int32_t* __restrict__ slot,
                                                         uint16_t* __restrict__ out, int64_t out_stride) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int strip = blockIdx.x, b = blockIdx.y, m0 = blockIdx.z * 64;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int ksteps = a.bwp / 32, pitch = a.bwp * 2 + 16;
  const int64_t wo = (((int64_t)b * (a.bwp / 16) + strip) * ksteps) * 512 + 8 * lane;
  const int c = b * a.bwp + 16 * strip + i16;
  // eight k-steps of both weights, the state and the gate vectors are on their way before the rows are parked
  constexpr int PF = 8;
  short8 wr[PF], wi[PF];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int j = 0; j < PF; ++j)
      if (k0 + j < ksteps) {
        wr[j] = *reinterpret_cast<const short8*>(a.wr + wo + 512 * (k0 + j));
        wi[j] = *reinterpret_cast<const short8*>(a.wi + wo + 512 * (k0 + j));
      }
  };
  fetch(0);
  const float br = a.br[c] * -kLog2e, bi = a.bi[c] * -kLog2e, sp = a.sp[c] * (-8.0f * kLog2e);
  float old[4], yv[4];
  float* sl[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int m = min(m0 + 16 * wid + 4 * g + r, a.M - 1);
    sl[r] = state + (int64_t)slot[m] * a.W + c;
    old[r] = start[m] > 0 ? *sl[r] : 0.f;
    yv[r] = Conv<bf16_t>::to_f32(y[(int64_t)m * a.W + c]);
  }
  park_u(lds, a.u, a.W, m0, min(64, a.M - m0), b * a.bwp, a.bwp);
  __syncthreads();
  if (m0 + 16 * wid >= a.M) return;
  float4v ar = float4v{0.f, 0.f, 0.f, 0.f}, ai = ar;
  for (int k0 = 0; k0 < ksteps; k0 += PF) {
    if (k0 > 0) fetch(k0);
#pragma unroll
    for (int j = 0; j < PF; ++j)
      if (k0 + j < ksteps) {
        const short8 af = *reinterpret_cast<const short8*>(lds + (16 * wid + i16) * pitch + (4 * (k0 + j) + g) * 16);
        ar = Mfma16<bf16_t>::mma(af, wr[j], ar);
        ai = Mfma16<bf16_t>::mma(af, wi[j], ai);
      }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int m = m0 + 16 * wid + 4 * g + r;
    if (m >= a.M) continue;
    const float u = Conv<bf16_t>::to_f32(*reinterpret_cast<const uint16_t*>(lds + (m - m0) * pitch + (16 * strip + i16) * 2));
    float da, db;
    gate_terms_fast(ar[r], ai[r], br, bi, sp, u, da, db);
    const float S = fmaf(da, old[r], db);
    *sl[r] = S;
    out[(int64_t)m * out_stride + c] = Conv<bf16_t>::from_f32(S * yv[r]);
  }
}

// The recurrence over the 64 rows of a tile, one channel per lane group: lane (i16, g) holds rows 16 mt + 4 g + r of its
// channel, so it runs over r inside the lane, over g with two shuffles, over mt in sequence.  ucol: the channel's column of
// the u rows in LDS; h, p: the tile's first row of the outputs.
template <bool FULL>
__device__ __forceinline__ void tile_scan(const float4v (&ar)[4], const float4v (&ai)[4], float br, float bi, float sp,
                                          const char* ucol, int pitch, int valid, int W, int c, float* __restrict__ h,
                                          float* __restrict__ p) {
  const int lane = threadIdx.x & 63, i16 = lane & 15, g = lane >> 4;
  const uint32_t off = (uint32_t)(4 * g) * W + c;
  float P0 = 1.f, H0 = 0.f;  // decay product and state over the rows in front
#pragma unroll
  for (int mt = 0; mt < 4; ++mt) {
    float A[4], B[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int k = 16 * mt + 4 * g + r;
      const float u = Conv<bf16_t>::to_f32(*reinterpret_cast<const uint16_t*>(ucol + k * pitch));
      gate_terms_fast(ar[mt][r], ai[mt][r], br, bi, sp, u, A[r], B[r]);
      if (!FULL && k >= valid) {
        A[r] = 1.f;
        B[r] = 0.f;
      }
      if (r > 0) {
        B[r] = fmaf(A[r], B[r - 1], B[r]);
        A[r] *= A[r - 1];
      }
    }
    // inclusive scan of (A[3], B[3]) over g, then the exclusive one
    float sa = A[3], sb = B[3];
#pragma unroll
    for (int o = 16; o < 64; o <<= 1) {
      const float pa = __shfl_up(sa, o, 64), pb = __shfl_up(sb, o, 64);
      if (lane >= o) {
        sb = fmaf(sa, pb, sb);
        sa *= pa;
      }
    }
    float ea = __shfl_up(sa, 16, 64), eb = __shfl_up(sb, 16, 64);
    if (lane < 16) {
      ea = 1.f;
      eb = 0.f;
    }
    const float pin = ea * P0, hin = fmaf(ea, H0, eb);  // everything in front of this lane's four rows
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint32_t o = (uint32_t)(16 * mt + r) * W + off;
      if (FULL || 16 * mt + 4 * g + r < valid) {
        h[o] = fmaf(A[r], hin, B[r]);
        p[o] = A[r] * pin;
      }
    }
    const float ta = __shfl(sa, 48 + i16, 64), tb = __shfl(sb, 48 + i16, 64);
    H0 = fmaf(ta, H0, tb);
    P0 *= ta;
  }
}

// Tiles of 64 rows of one sequence: tile_row[t] first row, tile_rows[t] rows.  hloc / prod [rows, W].
__global__ void __launch_bounds__(256) rglru_gates_kernel(RglruGates a, const int32_t* __restrict__ tile_row,
                                                          const int32_t* __restrict__ tile_rows, float* __restrict__ hloc,
                                                          float* __restrict__ prod) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  // channel blocks run fastest: the blocks in flight then write whole rows, not one column strip of many rows
  const int row0 = tile_row[blockIdx.y], valid = tile_rows[blockIdx.y], b = blockIdx.x;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int ksteps = a.bwp / 32, strips = a.bwp / 16, pitch = a.bwp * 2 + 16;
  park_u(lds, a.u, a.W, row0, valid, b * a.bwp, a.bwp);
  __syncthreads();
  constexpr int PF = 8;
  for (int strip = wid + 4 * blockIdx.z; strip < strips; strip += 4 * gridDim.z) {
    const int64_t wo = (((int64_t)b * strips + strip) * ksteps) * 512 + 8 * lane;
    const int c = b * a.bwp + 16 * strip + i16;
    float4v ar[4], ai[4];
#pragma unroll
    for (int mt = 0; mt < 4; ++mt) ar[mt] = ai[mt] = float4v{0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < ksteps; k0 += PF) {
      short8 wr[PF], wi[PF];  // a strip's weights come from L2: eight k-steps in flight
#pragma unroll
      for (int j = 0; j < PF; ++j) {
        const int ks = min(k0 + j, ksteps - 1);
        wr[j] = *reinterpret_cast<const short8*>(a.wr + wo + 512 * ks);
        wi[j] = *reinterpret_cast<const short8*>(a.wi + wo + 512 * ks);
      }
#pragma unroll
      for (int j = 0; j < PF; ++j) {
        if (k0 + j >= ksteps) break;
#pragma unroll
        for (int mt = 0; mt < 4; ++mt) {
          const short8 af = *reinterpret_cast<const short8*>(lds + (16 * mt + i16) * pitch + (4 * (k0 + j) + g) * 16);
          ar[mt] = Mfma16<bf16_t>::mma(af, wr[j], ar[mt]);
          ai[mt] = Mfma16<bf16_t>::mma(af, wi[j], ai[mt]);
        }
      }
    }
    const float br = a.br[c] * -kLog2e, bi = a.bi[c] * -kLog2e, sp = a.sp[c] * (-8.0f * kLog2e);
    if (valid == kScanTile)
      tile_scan<true>(ar, ai, br, bi, sp, lds + (16 * strip + i16) * 2, pitch, valid, a.W, c, hloc + (int64_t)row0 * a.W,
                      prod + (int64_t)row0 * a.W);
    else
      tile_scan<false>(ar, ai, br, bi, sp, lds + (16 * strip + i16) * 2, pitch, valid, a.W, c, hloc + (int64_t)row0 * a.W,
                       prod + (int64_t)row0 * a.W);
  }
}

// one thread per (sequence, channel): the state in front of every tile, the final state, the convolution state
template <typename T>
__global__ void __launch_bounds__(256) rglru_carry_kernel(RglruConv cv, const float* __restrict__ hloc,
                                                          const float* __restrict__ prod, float* __restrict__ carry,
                                                          float* __restrict__ state, const int32_t* __restrict__ tile0, int seq0,
                                                          int used) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= used) return;
  const int s = seq0 + blockIdx.y;
  const int n = cv.seq.rows[s], row0 = cv.seq.row0[s];
  float* sl = state + (int64_t)cv.seq.slot[s] * cv.W + c;
  float S = cv.seq.start[s] > 0 ? *sl : 0.f;
  const int tiles = (n + kScanTile - 1) / kScanTile;
  const int64_t t0 = tile0[s];
  for (int t = 0; t < tiles; t += 8) {
    float h[8], p[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {  // eight tiles' totals in flight
      const int64_t o = (int64_t)(row0 + min((min(t + j, tiles - 1) + 1) * kScanTile, n) - 1) * cv.W + c;
      h[j] = hloc[o];
      p[j] = prod[o];
    }
#pragma unroll
    for (int j = 0; j < 8; ++j)
      if (t + j < tiles) {
        carry[(t0 + t + j) * cv.W + c] = S;
        S = fmaf(p[j], S, h[j]);
      }
  }
  *sl = S;
  conv_state_update<T>(cv, s, c);
}

template <typename T>
__global__ void __launch_bounds__(256) rglru_apply_kernel(const float* __restrict__ hloc, const float* __restrict__ prod,
                                                          const float* __restrict__ carry, const void* __restrict__ y,
                                                          void* __restrict__ out, int64_t out_stride, RecurrentSeqs seq,
                                                          const int32_t* __restrict__ tile0, int M0, int M, int W, int used) {
  const int nv = used / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)(M - M0) * nv) return;
  const int m = M0 + (int)(idx / nv), c = (int)(idx % nv) * 8;
  const int s = seq.row_seq[m];
  const int64_t tile = tile0[s] + (m - seq.row0[s]) / kScanTile;
  float h[8], p[8], k[8], v[8];
  ld8<float>(hloc, (int64_t)m * W + c, h);
  ld8<float>(prod, (int64_t)m * W + c, p);
  ld8<float>(carry, tile * W + c, k);
  ld8<T>(y, (int64_t)m * W + c, v);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] *= fmaf(p[j], k[j], h[j]);
  st8<T>(out, (int64_t)m * out_stride + c, v);
}

// any type and block size: a and b of every row and channel
template <typename T>
__global__ void __launch_bounds__(256) rglru_rows_gates_kernel(const void* __restrict__ u, const void* __restrict__ wr,
                                                               const void* __restrict__ wi, const float* __restrict__ br,
                                                               const float* __restrict__ bi, const float* __restrict__ sp,
                                                               float* __restrict__ da, float* __restrict__ db, int M, int W,
                                                               int bwp, int blocks) {
  const int used = blocks * bwp;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * used) return;
  const int m = (int)(idx / used), c = (int)(idx % used);
  const int64_t ui = (int64_t)m * W + c / bwp * bwp, wo = (int64_t)c * bwp;  // weights row-major [blocks][bwp][bwp]
  float zr = br[c], zi = bi[c];
  for (int k = 0; k < bwp; ++k) {
    const float uv = ld<T>(u, ui + k);
    zr = fmaf(uv, ld<T>(wr, wo + k), zr);
    zi = fmaf(uv, ld<T>(wi, wo + k), zi);
  }
  float a, b;
  gate_terms(zr, zi, sp[c], ld<T>(u, (int64_t)m * W + c), a, b);
  da[(int64_t)m * W + c] = a;
  db[(int64_t)m * W + c] = b;
}

template <typename T>
__global__ void __launch_bounds__(256) rglru_rows_scan_kernel(RglruConv cv, const float* __restrict__ da,
                                                              const float* __restrict__ db, float* __restrict__ state,
                                                              void* __restrict__ out, int64_t out_stride, int used) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= used) return;
  const int s = blockIdx.y;
  const int n = cv.seq.rows[s], row0 = cv.seq.row0[s];
  float* sl = state + (int64_t)cv.seq.slot[s] * cv.W + c;
  float S = cv.seq.start[s] > 0 ? *sl : 0.f;
  for (int k = 0; k < n; ++k) {
    const int64_t o = (int64_t)(row0 + k) * cv.W + c;
    S = fmaf(da[o], S, db[o]);
    st<T>(out, (int64_t)(row0 + k) * out_stride + c, S * ld<T>(cv.y, o));
  }
  *sl = S;
  conv_state_update<T>(cv, s, c);
}

}  // namespace sglk

using namespace sglk;

static int check_conv(const RglruConv& a, int src_f32, int splits, int64_t part_stride, int64_t src_stride, int n_seqs, int dtype,
                      const char* what) {
  SGLK_CHECK(a.M >= 0 && a.W > 0 && a.W % 8 == 0 && a.taps >= 1 && n_seqs >= 0 && a.singles >= 0 && a.singles <= a.M,
             "%s: bad shape", what);
  SGLK_CHECK(a.M == 0 || (a.src.p && a.bias && a.by && a.conv && a.conv_b && a.u && a.y && a.seq.row_seq && a.seq.row0 && a.seq.rows &&
                          a.seq.start && a.seq.slot && (a.state || a.taps == 1)),
             "%s: null pointer", what);
  SGLK_CHECK(aligned16(a.u) && aligned16(a.y) && aligned16(a.state), "%s: rows must be 16-byte aligned", what);
  return check_source(a.src.p, src_f32, splits, part_stride, src_stride, 2 * a.W, dtype, what);
}

#define SGLK_CONV_ARGS                                                                                                       \
  const void *src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, const float *bx, const float *by,      \
      const float *conv, const float *conv_b, void *u, void *y, void *conv_state, const int32_t *row_seq, const int32_t *row0, \
      const int32_t *rows, const int32_t *start, const int32_t *slot, int M, int W, int taps, int singles, int n_seqs
#define SGLK_CONV_MAKE                                                                                                \
  RglruConv a {                                                                                                       \
    ShortConv{RowSource{src, src_f32, splits, part_stride, src_stride}, bx, conv, conv_b, u, conv_state,              \
              RecurrentSeqs{row_seq, row0, rows, start, slot}, M, W, taps, singles},                                  \
        by, y                                                                                                         \
  }

extern "C" {

int sglk_rglru_conv(SGLK_CONV_ARGS, int dtype, void* stream) {
  SGLK_CONV_MAKE;
  if (int rc = check_conv(a, src_f32, splits, part_stride, src_stride, n_seqs, dtype, "rglru_conv")) return rc;
  if (M == 0) return SGLK_OK;
  const int per = M >= 256 ? 4 : 1;  // rows per thread
  const int64_t threads = (int64_t)((M + per - 1) / per) * (W / 8);
  const dim3 grid((unsigned)((threads + 255) / 256), 2);
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (per == 4)
      hipLaunchKernelGGL((rglru_conv_kernel<T, 4>), grid, dim3(256), 0, (hipStream_t)stream, a);
    else
      hipLaunchKernelGGL((rglru_conv_kernel<T, 1>), grid, dim3(256), 0, (hipStream_t)stream, a);
  });
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

static int check_gates(const void* u, const void* wr, const void* wi, const float* br, const float* bi, const float* sp, int W,
                       int bwp, int blocks, const char* what) {
  SGLK_CHECK(bwp > 0 && bwp % 32 == 0 && bwp <= kGateMaxBlock && blocks > 0 && blocks * bwp <= W && W % 8 == 0,
             "%s: %d blocks of %d channels in rows of %d", what, blocks, bwp, W);
  SGLK_CHECK(u && wr && wi && br && bi && sp, "%s: null pointer", what);
  SGLK_CHECK(aligned16(u) && aligned16(wr) && aligned16(wi), "%s: unaligned pointer", what);
  return SGLK_OK;
}

int sglk_rglru_step(const void* u, const void* wr, const void* wi, const float* br, const float* bi, const float* sp,
                    const void* y, float* state, const int32_t* start, const int32_t* slot, void* out, int64_t out_stride, int M,
                    int W, int bwp, int blocks, void* stream) {
  SGLK_CHECK(M >= 0 && out_stride >= (int64_t)bwp * blocks, "rglru_step: bad shape");
  if (M == 0) return SGLK_OK;
  if (int rc = check_gates(u, wr, wi, br, bi, sp, W, bwp, blocks, "rglru_step")) return rc;
  SGLK_CHECK(y && state && start && slot && out, "rglru_step: null pointer");
  RglruGates a{(const uint16_t*)u, (const uint16_t*)wr, (const uint16_t*)wi, br, bi, sp, M, W, bwp};
  if (int rc = ensure_lds<rglru_step_kernel>(gate_lds(kGateMaxBlock))) return rc;
  hipLaunchKernelGGL(rglru_step_kernel, dim3(bwp / 16, blocks, (M + 63) / 64), dim3(256), gate_lds(bwp), (hipStream_t)stream, a,
                     (const uint16_t*)y, state, start, slot, (uint16_t*)out, out_stride);
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_rglru_gates(const void* u, const void* wr, const void* wi, const float* br, const float* bi, const float* sp,
                     const int32_t* tile_row, const int32_t* tile_rows, int tiles, float* hloc, float* prod, int W, int bwp,
                     int blocks, void* stream) {
  SGLK_CHECK(tiles >= 0 && tiles <= 65535, "rglru_gates: at most 65535 tiles");
  if (tiles == 0) return SGLK_OK;
  if (int rc = check_gates(u, wr, wi, br, bi, sp, W, bwp, blocks, "rglru_gates")) return rc;
  SGLK_CHECK(tile_row && tile_rows && hloc && prod, "rglru_gates: null pointer");
  RglruGates a{(const uint16_t*)u, (const uint16_t*)wr, (const uint16_t*)wi, br, bi, sp, 0, W, bwp};
  if (int rc = ensure_lds<rglru_gates_kernel>(gate_lds(kGateMaxBlock))) return rc;
  // a few tiles only: the strips of a channel block spread over more blocks
  const int groups = (bwp / 16 + 3) / 4;
  const int z = std::max(1, std::min(groups, 1024 / std::max(tiles * blocks, 1)));
  hipLaunchKernelGGL(rglru_gates_kernel, dim3(blocks, tiles, z), dim3(256), gate_lds(bwp), (hipStream_t)stream, a, tile_row,
                     tile_rows, hloc, prod);
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_rglru_carry(SGLK_CONV_ARGS, const float* hloc, const float* prod, float* carry, float* state, const int32_t* tile0,
                     int seq0, int used, int dtype, void* stream) {
  SGLK_CONV_MAKE;
  if (int rc = check_conv(a, src_f32, splits, part_stride, src_stride, n_seqs, dtype, "rglru_carry")) return rc;
  SGLK_CHECK(seq0 >= 0 && seq0 <= n_seqs && n_seqs - seq0 <= 65535, "rglru_carry: bad sequence range");
  SGLK_CHECK(used > 0 && used <= W, "rglru_carry: bad channel count");
  if (M == 0 || n_seqs == seq0) return SGLK_OK;
  SGLK_CHECK(hloc && prod && carry && state && tile0, "rglru_carry: null pointer");
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((rglru_carry_kernel<T>), dim3((used + 255) / 256, n_seqs - seq0), dim3(256),
                                         0, (hipStream_t)stream, a, hloc, prod, carry, state, tile0, seq0, used));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_rglru_apply(const float* hloc, const float* prod, const float* carry, const void* y, void* out, int64_t out_stride,
                     const int32_t* row_seq, const int32_t* row0, const int32_t* tile0, int first_row, int M, int W, int used,
                     int dtype, void* stream) {
  SGLK_CHECK(first_row >= 0 && M >= first_row && W % 8 == 0 && used > 0 && used <= W && used % 8 == 0 && out_stride >= used &&
                 out_stride % 8 == 0,
             "rglru_apply: bad shape");
  if (M == first_row) return SGLK_OK;
  SGLK_CHECK(hloc && prod && carry && y && out && row_seq && row0 && tile0, "rglru_apply: null pointer");
  SGLK_CHECK(aligned16(y) && aligned16(out), "rglru_apply: rows must be 16-byte aligned");
  const int64_t vecs = (int64_t)(M - first_row) * (used / 8);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((rglru_apply_kernel<T>), dim3((unsigned)((vecs + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, hloc, prod, carry, y, out, out_stride,
                                         RecurrentSeqs{row_seq, row0, nullptr, nullptr, nullptr}, tile0, first_row, M, W, used));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_rglru_rows(SGLK_CONV_ARGS, const void* wr, const void* wi, const float* br, const float* bi, const float* sp, float* da,
                    float* db, float* state, void* out, int64_t out_stride, int bwp, int blocks, int dtype, void* stream) {
  SGLK_CONV_MAKE;
  if (int rc = check_conv(a, src_f32, splits, part_stride, src_stride, n_seqs, dtype, "rglru_rows")) return rc;
  SGLK_CHECK(bwp > 0 && blocks > 0 && (int64_t)bwp * blocks <= W && out_stride >= (int64_t)bwp * blocks && n_seqs <= 65535, "rglru_rows: bad shape");
  SGLK_CHECK(singles == 0, "rglru_rows: convolution states of all sequences are updated here");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(wr && wi && br && bi && sp && da && db && state && out, "rglru_rows: null pointer");
  const int used = bwp * blocks;
  const int64_t total = (int64_t)M * used;
  SGLK_DISPATCH_FLOAT(dtype, T, {
    hipLaunchKernelGGL((rglru_rows_gates_kernel<T>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0, (hipStream_t)stream, u,
                       wr, wi, br, bi, sp, da, db, M, W, bwp, blocks);
    hipLaunchKernelGGL((rglru_rows_scan_kernel<T>), dim3((used + 255) / 256, n_seqs), dim3(256), 0, (hipStream_t)stream, a, da,
                       db, state, out, out_stride, used);
  });
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}
}
