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
//   delta_prep     portions in tiles of 64 rows, one wave per tile and head: what the tile's rows do to each other
//   delta_chunk    walks the tiles of a sequence: the state in registers, every product on the matrix cores
//   delta_gate     norm and gate of the rows delta_chunk leaves
//
// delta_step reads the state once per row: o = g S^T q + (k . q) u needs the products of the old state only.  The unit
// norms stay factors on the products of the convolution's outputs, so they are never rounded to the activation type.
//
// A tile of rows 1 .. n in front of which the state is S0, with c_i the product of its first i decays:
//
//   u_i = beta_i (v_i - c_i S0^T k_i) - sum_{j < i} A_ij u_j,     A_ij = beta_i (k_i . k_j) c_i / c_j
//   o_i = c_i S0^T q_i + sum_{j <= i} P_ij u_j,                   P_ij = (q_i . k_j) c_i / c_j
//   S   = c_n S0 + sum_j (c_n / c_j) k_j u_j^T
//
// so U = T (beta V - beta c K S0) with T = (1 + A)^-1, which does not depend on the state.  The convolution's outputs enter
// the matrix cores as the 16-bit numbers they are; every other operand (T, P, states, u) as the sum of two bfloat16
// numbers, which leaves 2^-17 of it, and products are added in fp32.
#include <algorithm>

#include "attention_tile.h"
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
// them per thread in registers (NR = 0: any number, the state stays in memory).  EXACT: every thread owns NR rows.
template <typename T, int NR, bool EXACT>
__global__ void __launch_bounds__(256) delta_step_kernel(DeltaRule a, int seq0) {
  extern __shared__ __attribute__((aligned(16))) float delta_lds[];
  __shared__ float red3[12], red1[4];
  const int h = blockIdx.x, s = seq0 + blockIdx.y;
  const int CG = a.vp / 4, RG = 256 / CG;
  const int cg = threadIdx.x % CG, rg = threadIdx.x / CG;
  const bool mine = EXACT || rg < RG;
  float* kx = delta_lds;            // [dp] key channels, then [dp] query channels
  float* qx = kx + a.dp;
  float* part = qx + a.dp;          // [2][RG][vp]
  float* ub = part + 2 * RG * a.vp;  // [vp]
  const int n = a.seq.rows[s], row0 = a.seq.row0[s];
  const bool fresh = a.seq.start[s] == 0;
  float* sp = a.state + ((int64_t)a.seq.slot[s] * a.VH + h) * a.dp * a.vp + 4 * cg;
  const int kh = h / (a.VH / a.KH);
  const float4v zero = float4v{0.f, 0.f, 0.f, 0.f};
  float* base = sp + (int64_t)rg * a.vp;
  float4v S[NR > 0 ? NR : 1];
  if constexpr (NR > 0) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int r = rg + RG * i;
      S[i] = zero;  // states are read and written once: past the caches
      if (!fresh && mine && (EXACT || r < a.dp))
        S[i] = __builtin_nontemporal_load(reinterpret_cast<const float4v*>(base + (int64_t)(RG * i) * a.vp));
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
          const int r = EXACT ? rg + RG * i : min(rg + RG * i, a.dp - 1);  // rows past the state are zero
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
          if (EXACT || r < a.dp) S[i] = S[i] * g + u * kx[r];
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
      if (mine && (EXACT || r < a.dp))
        __builtin_nontemporal_store(S[i], reinterpret_cast<float4v*>(base + (int64_t)(RG * i) * a.vp));
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// tiles of 64 rows
// ---------------------------------------------------------------------------------------------------------------------
constexpr int kDeltaTile = 64;
constexpr int kDeltaFrag = 4 * 2 * 2 * 64 * 8;  // a 64 x 64 matrix as operands: [row block][k-step of 32][high, low][lane][8]

// what delta_prep leaves per (tile, head)
struct DeltaTiles {
  uint16_t* mats;   // [tiles][VH][T, P][kDeltaFrag]
  float* rows;      // [tiles][VH][64][4]: beta, beta c / |k|, c / |q|, (c_n / c) / |k|   (|q| with the query's scale)
  float* decay;     // [tiles][VH]: c_n
};

__device__ __forceinline__ void split_bf16(float x, uint16_t& hi, uint16_t& lo) {
  hi = Conv<bf16_t>::from_f32(x);
  lo = Conv<bf16_t>::from_f32(x - Conv<bf16_t>::to_f32(hi));
}

__device__ __forceinline__ void split4(const float4v& x, short4v& hi, short4v& lo) {
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    uint16_t a, b;
    split_bf16(x[r], a, b);
    hi[r] = (short)a;
    lo[r] = (short)b;
  }
}

__device__ __forceinline__ void wave_lds_sync() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

constexpr int kMatPitch = 68;  // floats
constexpr int kDeltaPrepLds = 4 * (64 * kMatPitch + 4 * 64) * 4;

// the lower triangle of a wave's 64 x 64 matrix in LDS -> operands: lane (i, g) of step s holds the columns
// 32 s + (j < 4 ? 4 g + j : 16 + 4 g + j - 4) of row i, the order transposed LDS reads deliver a tile's rows in
__device__ __forceinline__ void store_operands(const float* mat, uint16_t* __restrict__ out) {
  const int lane = threadIdx.x & 63, i16 = lane & 15, g = lane >> 4;
#pragma unroll
  for (int rb = 0; rb < 4; ++rb)
#pragma unroll
    for (int s = 0; s <= rb / 2; ++s) {
      const float* row = mat + (16 * rb + i16) * kMatPitch + 32 * s + 4 * g;
      short4v h0, l0, h1, l1;
      split4(*reinterpret_cast<const float4v*>(row), h0, l0);
      split4(*reinterpret_cast<const float4v*>(row + 16), h1, l1);
      uint16_t* o = out + ((rb * 2 + s) * 2 * 64 + lane) * 8;
      *reinterpret_cast<short8*>(o) = short8{h0[0], h0[1], h0[2], h0[3], h1[0], h1[1], h1[2], h1[3]};
      *reinterpret_cast<short8*>(o + 64 * 8) = short8{l0[0], l0[1], l0[2], l0[3], l1[0], l1[1], l1[2], l1[3]};
    }
}

// One wave per (tile, head).
__global__ void __launch_bounds__(256, 2) delta_prep_kernel(DeltaRule a, DeltaTiles t, const int32_t* __restrict__ tile_row,
                                                            const int32_t* __restrict__ tile_rows) {
  extern __shared__ __attribute__((aligned(16))) float prep_lds[];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x * 4 + wid, tile = blockIdx.y;
  if (h >= a.VH) return;  // wave-uniform; no block barrier below
  float* mat = prep_lds + wid * (64 * kMatPitch + 4 * 64);
  float* rk = mat + 64 * kMatPitch;
  float* rq = rk + 64;
  float* cum = rq + 64;   // log2 of the running decay
  float* bet = cum + 64;
  const int row0 = tile_row[tile], valid = tile_rows[tile];
  float log_g, beta;
  delta_gates<bf16_t>(a, row0 + min(lane, valid - 1), h, log_g, beta);
  float c = lane < valid ? log_g * 1.4426950408889634f : 0.f;
  if (lane >= valid) beta = 0.f;
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const float up = __shfl_up(c, o, 64);
    if (lane >= o) c += up;
  }
  cum[lane] = c;
  bet[lane] = beta;

  const int kh = h / (a.VH / a.KH);
  const uint16_t* u = reinterpret_cast<const uint16_t*>(a.u) + kh * a.dp + 8 * g;
  const uint16_t* qrow[4];
#pragma unroll
  for (int rb = 0; rb < 4; ++rb) qrow[rb] = u + (int64_t)(row0 + min(16 * rb + i16, valid - 1)) * a.u_stride;
  const int koff = a.KH * a.dp;
  float4v G[10], P[10];  // tiles (bi, bj), bj <= bi, at bi (bi + 1) / 2 + bj
#pragma unroll
  for (int i = 0; i < 10; ++i) G[i] = P[i] = float4v{0.f, 0.f, 0.f, 0.f};
  float sk[4] = {0.f, 0.f, 0.f, 0.f}, sq[4] = {0.f, 0.f, 0.f, 0.f};
  for (int ks = 0; ks < a.dp / 32; ++ks) {
    short8 kf[4], qf[4];
#pragma unroll
    for (int rb = 0; rb < 4; ++rb) {
      qf[rb] = *reinterpret_cast<const short8*>(qrow[rb] + 32 * ks);
      kf[rb] = *reinterpret_cast<const short8*>(qrow[rb] + koff + 32 * ks);
    }
#pragma unroll
    for (int rb = 0; rb < 4; ++rb) {
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float kv = Conv<bf16_t>::to_f32((uint16_t)kf[rb][j]), qv = Conv<bf16_t>::to_f32((uint16_t)qf[rb][j]);
        sk[rb] = fmaf(kv, kv, sk[rb]);
        sq[rb] = fmaf(qv, qv, sq[rb]);
      }
#pragma unroll
      for (int bj = 0; bj <= rb; ++bj) {
        G[rb * (rb + 1) / 2 + bj] = Mfma16<bf16_t>::mma(kf[rb], kf[bj], G[rb * (rb + 1) / 2 + bj]);
        P[rb * (rb + 1) / 2 + bj] = Mfma16<bf16_t>::mma(qf[rb], kf[bj], P[rb * (rb + 1) / 2 + bj]);
      }
    }
  }
#pragma unroll
  for (int rb = 0; rb < 4; ++rb) {
    float x = sk[rb], y = sq[rb];
    x += __shfl_xor(x, 16, 64);
    x += __shfl_xor(x, 32, 64);
    y += __shfl_xor(y, 16, 64);
    y += __shfl_xor(y, 32, 64);
    if (g == 0) {
      rk[16 * rb + i16] = 1.0f / sqrtf(x + kUnitEps);
      rq[16 * rb + i16] = a.q_scale / sqrtf(y + kUnitEps);
    }
  }
  wave_lds_sync();
  const int64_t th = (int64_t)tile * a.VH + h;
  const float total = cum[63], e = __builtin_amdgcn_exp2f(c);
  *reinterpret_cast<float4v*>(t.rows + (th * 64 + lane) * 4) =
      float4v{beta, beta * e * rk[lane], e * rq[lane], __builtin_amdgcn_exp2f(total - c) * rk[lane]};
  if (lane == 0) t.decay[th] = __builtin_amdgcn_exp2f(total);

  // both matrices pass through the wave's LDS: P, then A and its triangular inverse
  uint16_t* out = t.mats + th * 2 * kDeltaFrag;
#pragma unroll
  for (int which = 1; which >= 0; --which) {
#pragma unroll
    for (int bi = 0; bi < 4; ++bi)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int i = 16 * bi + 4 * g + r;
        const float ci = cum[i], left = which ? rq[i] : bet[i] * rk[i];
#pragma unroll
        for (int bj = 0; bj < 4; ++bj) {
          const int j = 16 * bj + i16;
          float v = 0.f;
          if (bj <= bi && (which ? j <= i : j < i))
            v = (which ? P : G)[bi * (bi + 1) / 2 + (bj <= bi ? bj : 0)][r] * left * rk[j] * __builtin_amdgcn_exp2f(ci - cum[j]);
          mat[i * kMatPitch + j] = v;
        }
      }
    wave_lds_sync();
    if (which == 0) {
      // lane j owns column j of T: t_i = [i == j] - sum_{l < i} A_il t_l
      float tc[64];
#pragma unroll
      for (int i = 0; i < 64; ++i) {
        float s[4] = {i == lane ? 1.f : 0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int l = 0; l < i; l += 4) {
          const float4v row = *reinterpret_cast<const float4v*>(mat + i * kMatPitch + l);  // columns from i on are zero
#pragma unroll
          for (int j = 0; j < 4; ++j)
            if (l + j < i) s[j] = fmaf(-row[j], tc[l + j], s[j]);
        }
        tc[i] = (s[0] + s[1]) + (s[2] + s[3]);
      }
      wave_lds_sync();
#pragma unroll
      for (int i = 0; i < 64; ++i) mat[i * kMatPitch + lane] = tc[i];
      wave_lds_sync();
    }
    store_operands(mat, out + which * kDeltaFrag);
    wave_lds_sync();
  }
}

constexpr int delta_x_pitch(int DP) { return DP * 2 + 16; }
constexpr int delta_r_pitch(int NT) { return NT * 32 + 16; }
constexpr int delta_st_bytes(int DP, int NT) {
  const int st = 2 * NT * 16 * delta_x_pitch(DP), u = 2 * 64 * delta_r_pitch(NT);
  return st > u ? st : u;
}
constexpr int delta_chunk_lds(int DP, int NT) {
  return delta_st_bytes(DP, NT) + 64 * delta_x_pitch(DP) + 2 * 64 * delta_r_pitch(NT);
}

// 16 columns of 32 rows (32 step ..) of a row-major 16-bit tile, as an operand: lane (i, g) gets column 16 block + i of the rows
// (j < 4 ? 4 g + j : 16 + 4 g + j - 4)
__device__ __forceinline__ short8 read_columns(const char* tile, int pitch, int step, int block) {
  const int lane = threadIdx.x & 63, hl = lane & 15, g = lane >> 4;
  const char* p = tile + (32 * step + 4 * g + (hl >> 2)) * pitch + 32 * block + 8 * (hl & 3);
  const short4v lo = lds_read_tr16(p), hi = lds_read_tr16(p + 16 * pitch);
  return short8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
}

// Block: one sequence, one head, 16 NT columns of its values.  Wave w owns the rows 16 w .. of every tile (as columns of
// the products) and the state's rows 16 w .., 16 (w + 4) .. in accumulators.  o: [rows, VH * vp] fp32 before norm and gate.
template <int DP, int NT>
__global__ void __launch_bounds__(256, delta_chunk_lds(DP, NT) <= 80 * 1024 ? 2 : 1)
    delta_chunk_kernel(DeltaRule a, DeltaTiles t, const int32_t* __restrict__ tile0, float* __restrict__ o, int seq0) {
  constexpr int KS = DP / 32, KB = (DP + 63) / 64, XP = delta_x_pitch(DP), RP = delta_r_pitch(NT);
  extern __shared__ __attribute__((aligned(16))) char dc_lds[];
  char* st_hi = dc_lds;                       // S^T [16 NT][DP], then u [64][16 NT]
  char* st_lo = st_hi + NT * 16 * XP;
  char* u_hi = dc_lds;
  char* u_lo = u_hi + 64 * RP;
  char* xk = dc_lds + delta_st_bytes(DP, NT);  // k [64][DP]
  char* r_hi = xk + 64 * XP;                  // the right-hand side [64][16 NT], then u c_n / c
  char* r_lo = r_hi + 64 * RP;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x, n0 = blockIdx.y * 16 * NT, s = seq0 + blockIdx.z;
  const int nt_used = min(NT, (a.vp - n0) / 16);
  const int row0 = a.seq.row0[s], n = a.seq.rows[s];
  const int tiles = (n + kDeltaTile - 1) / kDeltaTile;
  const int64_t first = tile0[s];
  const int kh = h / (a.VH / a.KH);
  float* state = a.state + ((int64_t)a.seq.slot[s] * a.VH + h) * a.dp * a.vp + n0 + i16;
  const bool fresh = a.seq.start[s] == 0;
  float4v S[KB][NT];
#pragma unroll
  for (int i = 0; i < KB; ++i)
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      S[i][nt] = float4v{0.f, 0.f, 0.f, 0.f};
      const int kb = wid + 4 * i;
      if (!fresh && 16 * kb < DP && nt < nt_used) {
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][nt][r] = state[(int64_t)(16 * kb + 4 * g + r) * a.vp + 16 * nt];
      }
    }
  const uint16_t* u = reinterpret_cast<const uint16_t*>(a.u);
  short8 kf[KS], qf[KS], tf[2][2], pf[2][2];
  short4v vf[NT];
  float4v sc;
  float dec;
  auto row_of = [&](int tile) { return (int64_t)(row0 + min(64 * tile + 16 * wid + i16, n - 1)); };
  auto fetch_x = [&](int tile) {
    const uint16_t* p = u + row_of(tile) * a.u_stride + kh * a.dp + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) {
      qf[ks] = *reinterpret_cast<const short8*>(p + 32 * ks);
      kf[ks] = *reinterpret_cast<const short8*>(p + a.KH * a.dp + 32 * ks);
    }
  };
  auto fetch_v = [&](int tile) {
    const uint16_t* p = u + row_of(tile) * a.u_stride + 2 * a.KH * a.dp + h * a.vp + n0 + 4 * g;
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) vf[nt] = nt < nt_used ? *reinterpret_cast<const short4v*>(p + 16 * nt) : short4v{0, 0, 0, 0};
  };
  auto fetch_mat = [&](short8(&f)[2][2], int tile, int which) {
    const uint16_t* p = t.mats + (((first + tile) * a.VH + h) * 2 + which) * kDeltaFrag + wid * 4 * 512 + 8 * lane;
#pragma unroll
    for (int st = 0; st < 2; ++st)
      if (st <= wid / 2) {
#pragma unroll
        for (int hl = 0; hl < 2; ++hl) f[st][hl] = *reinterpret_cast<const short8*>(p + (st * 2 + hl) * 512);
      }
  };
  auto fetch_rows = [&](int tile) {
    const int64_t th = (first + tile) * a.VH + h;
    sc = *reinterpret_cast<const float4v*>(t.rows + (th * 64 + 16 * wid + i16) * 4);
    dec = t.decay[th];
  };
  fetch_x(0);
  fetch_v(0);
  fetch_rows(0);
  fetch_mat(tf, 0, 0);
  fetch_mat(pf, 0, 1);
  for (int tile = 0; tile < tiles; ++tile) {
    const int next = min(tile + 1, tiles - 1);
    // the state in front of the tile, two 16-bit halves, transposed; the tile's keys
#pragma unroll
    for (int i = 0; i < KB; ++i) {
      const int kb = wid + 4 * i;
      if (16 * kb < DP) {
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          short4v hi, lo;
          split4(S[i][nt], hi, lo);
          *reinterpret_cast<short4v*>(st_hi + (16 * nt + i16) * XP + (16 * kb + 4 * g) * 2) = hi;
          *reinterpret_cast<short4v*>(st_lo + (16 * nt + i16) * XP + (16 * kb + 4 * g) * 2) = lo;
        }
      }
    }
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) *reinterpret_cast<short8*>(xk + (16 * wid + i16) * XP + (4 * ks + g) * 16) = kf[ks];
    __syncthreads();
    float4v oacc[NT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      float4v y = float4v{0.f, 0.f, 0.f, 0.f}, z = y;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const short8 hi = *reinterpret_cast<const short8*>(st_hi + (16 * nt + i16) * XP + (4 * ks + g) * 16);
        const short8 lo = *reinterpret_cast<const short8*>(st_lo + (16 * nt + i16) * XP + (4 * ks + g) * 16);
        y = Mfma16<bf16_t>::mma(hi, kf[ks], y);
        z = Mfma16<bf16_t>::mma(hi, qf[ks], z);
        y = Mfma16<bf16_t>::mma(lo, kf[ks], y);
        z = Mfma16<bf16_t>::mma(lo, qf[ks], z);
      }
      float4v r;
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = sc[0] * Conv<bf16_t>::to_f32((uint16_t)vf[nt][e]) - sc[1] * y[e];
      short4v hi, lo;
      split4(r, hi, lo);
      *reinterpret_cast<short4v*>(r_hi + (16 * wid + i16) * RP + (16 * nt + 4 * g) * 2) = hi;
      *reinterpret_cast<short4v*>(r_lo + (16 * wid + i16) * RP + (16 * nt + 4 * g) * 2) = lo;
      oacc[nt] = z * sc[2];
    }
    const float tail = sc[3], d = dec;
    fetch_x(next);  // the next tile's operands fly during the rest of this one
    fetch_v(next);
    fetch_rows(next);
    __syncthreads();
    float4v uacc[NT];
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) uacc[nt] = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < 2; ++st)
      if (st <= wid / 2) {  // wave-uniform: T is lower triangular
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const short8 hi = read_columns(r_hi, RP, st, nt), lo = read_columns(r_lo, RP, st, nt);
          uacc[nt] = Mfma16<bf16_t>::mma(hi, tf[st][0], uacc[nt]);
          uacc[nt] = Mfma16<bf16_t>::mma(lo, tf[st][0], uacc[nt]);
          uacc[nt] = Mfma16<bf16_t>::mma(hi, tf[st][1], uacc[nt]);
        }
      }
    fetch_mat(tf, next, 0);
    __syncthreads();  // the right-hand side and the state's copy have been read
#pragma unroll
    for (int nt = 0; nt < NT; ++nt) {
      const int at = (16 * wid + i16) * RP + (16 * nt + 4 * g) * 2;
      short4v hi, lo;
      split4(uacc[nt], hi, lo);
      *reinterpret_cast<short4v*>(u_hi + at) = hi;
      *reinterpret_cast<short4v*>(u_lo + at) = lo;
      split4(uacc[nt] * tail, hi, lo);
      *reinterpret_cast<short4v*>(r_hi + at) = hi;
      *reinterpret_cast<short4v*>(r_lo + at) = lo;
    }
    __syncthreads();
#pragma unroll
    for (int st = 0; st < 2; ++st)
      if (st <= wid / 2) {
#pragma unroll
        for (int nt = 0; nt < NT; ++nt) {
          const short8 hi = read_columns(u_hi, RP, st, nt), lo = read_columns(u_lo, RP, st, nt);
          oacc[nt] = Mfma16<bf16_t>::mma(hi, pf[st][0], oacc[nt]);
          oacc[nt] = Mfma16<bf16_t>::mma(lo, pf[st][0], oacc[nt]);
          oacc[nt] = Mfma16<bf16_t>::mma(hi, pf[st][1], oacc[nt]);
        }
      }
    fetch_mat(pf, next, 1);
    const int i = 64 * tile + 16 * wid + i16;
    if (i < n) {
      float* dst = o + (int64_t)(row0 + i) * (a.VH * a.vp) + h * a.vp + n0 + 4 * g;
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
        if (nt < nt_used) *reinterpret_cast<float4v*>(dst + 16 * nt) = oacc[nt];
    }
#pragma unroll
    for (int k = 0; k < KB; ++k)
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) S[k][nt] *= d;
#pragma unroll
    for (int st = 0; st < 2; ++st) {
      short8 kc[KB];
#pragma unroll
      for (int k = 0; k < KB; ++k) kc[k] = read_columns(xk, XP, st, min(wid + 4 * k, DP / 16 - 1));
#pragma unroll
      for (int nt = 0; nt < NT; ++nt) {
        const short8 hi = read_columns(r_hi, RP, st, nt), lo = read_columns(r_lo, RP, st, nt);
#pragma unroll
        for (int k = 0; k < KB; ++k) {
          S[k][nt] = Mfma16<bf16_t>::mma(kc[k], hi, S[k][nt]);
          S[k][nt] = Mfma16<bf16_t>::mma(kc[k], lo, S[k][nt]);
        }
      }
    }
    __syncthreads();  // keys and u have been read
  }
#pragma unroll
  for (int i = 0; i < KB; ++i) {
    const int kb = wid + 4 * i;
    if (16 * kb < DP) {
#pragma unroll
      for (int nt = 0; nt < NT; ++nt)
        if (nt < nt_used) {
#pragma unroll
          for (int r = 0; r < 4; ++r) state[(int64_t)(16 * kb + 4 * g + r) * a.vp + 16 * nt] = S[i][nt][r];
        }
    }
  }
}

// norm over a head's values, its weight and gate: TPH threads per (row, head), eight values each
template <typename T>
__global__ void __launch_bounds__(256) delta_gate_kernel(DeltaRule a, const float* __restrict__ o, int M0, int M, int TPH) {
  const int64_t idx = ((int64_t)blockIdx.x * 256 + threadIdx.x) / TPH;
  const int t = threadIdx.x & (TPH - 1), c = 8 * t;
  const bool live = idx < (int64_t)(M - M0) * a.VH && c < a.vp;
  const int64_t mh = live ? idx : 0;
  const int m = M0 + (int)(mh / a.VH), h = (int)(mh % a.VH);
  float v[8], w[8], z[8], ss = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = 0.f;
  if (live) {
    ld8<float>(o, (int64_t)m * (a.VH * a.vp) + h * a.vp + c, v);
    ld8<float>(a.norm, c, w);
    source8<T>(a.src, m, h * a.vp + c, z);
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) ss += v[j] * v[j];
  for (int off = 1; off < TPH; off <<= 1) ss += __shfl_xor(ss, off, 64);
  if (!live) return;
  const float inv = a.out_scale / sqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
  for (int j = 0; j < 8; ++j)
    v[j] *= inv * w[j] * (sizeof(typename Raw<T>::type) == 2 ? silu_fast(z[j]) : activate(z[j], 3));
  st8<T>(a.out, (int64_t)m * a.out_stride + h * a.vp + c, v);
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
  const bool exact = 256 % (vp / 4) == 0 && per * RG == dp;
#define SGLK_DS(NR, E) hipLaunchKernelGGL((delta_step_kernel<T, NR, E>), grid, dim3(256), lds, (hipStream_t)stream, a, seq0)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (exact && per == 4)
      SGLK_DS(4, true);
    else if (exact && per == 8)
      SGLK_DS(8, true);
    else if (exact && per == 16)
      SGLK_DS(16, true);
    else if (per <= 8)
      SGLK_DS(8, false);
    else if (per <= 32)
      SGLK_DS(32, false);
    else
      SGLK_DS(0, false);
  });
#undef SGLK_DS
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

// head sizes delta_chunk has tile kernels for
#define SGLK_DELTA_SIZES(X) X(32) X(64) X(96) X(128) X(192) X(256)

int sglk_delta_chunk_supported(int dp, int vp) {
  if (vp % 16 != 0 || vp <= 0 || vp > 512) return 0;
#define X(S) if (dp == S) return 1;
  SGLK_DELTA_SIZES(X)
#undef X
  return 0;
}

// bytes of delta_chunk's workspace for that many tiles
int64_t sglk_delta_chunk_workspace_bytes(int tiles, int heads) {
  return (int64_t)tiles * heads * (2 * kDeltaFrag * 2 + 64 * 16 + 4) + 16;
}

int sglk_delta_chunk(SGLK_DELTA_ARGS, const int32_t* tile_row, const int32_t* tile_rows, const int32_t* tile0, int tiles,
                     void* workspace, int64_t workspace_bytes, float* o, int first_row, int seq0, int n_seqs, void* stream) {
  SGLK_DELTA_MAKE;
  if (int rc = check_delta(a, M, dim, seq0, n_seqs, SGLK_BF16, "delta_chunk")) return rc;
  SGLK_CHECK(sglk_delta_chunk_supported(dp, vp), "delta_chunk: no tile kernel for heads of %d / %d", dp, vp);
  SGLK_CHECK(tiles >= 0 && tiles <= 65535 && first_row >= 0 && first_row <= M, "delta_chunk: bad shape");
  if (M == first_row || n_seqs == seq0 || tiles == 0) return SGLK_OK;
  SGLK_CHECK(tile_row && tile_rows && tile0 && workspace && o && aligned16(workspace) && aligned16(o),
             "delta_chunk: null or unaligned pointer");
  SGLK_CHECK(workspace_bytes >= sglk_delta_chunk_workspace_bytes(tiles, heads), "delta_chunk: workspace too small");
  DeltaTiles t;
  t.mats = (uint16_t*)workspace;
  t.rows = (float*)(t.mats + (int64_t)tiles * heads * 2 * kDeltaFrag);
  t.decay = t.rows + (int64_t)tiles * heads * 64 * 4;
  hipStream_t s = (hipStream_t)stream;
  if (int rc = ensure_lds<delta_prep_kernel>(kDeltaPrepLds)) return rc;
  hipLaunchKernelGGL(delta_prep_kernel, dim3((heads + 3) / 4, tiles), dim3(256), kDeltaPrepLds, s, a, t, tile_row, tile_rows);
  SGLK_LAUNCH_CHECK();
  // 64 columns of values per block, 32 where that leaves half of the chip idle
  const int wide = vp > 32 && (int64_t)heads * (n_seqs - seq0) * ((vp + 63) / 64) >= 192;
#define SGLK_DC(S, NT)                                                                                                   \
  {                                                                                                                      \
    if (int rc = ensure_lds<delta_chunk_kernel<S, NT>>(delta_chunk_lds(S, NT))) return rc;                               \
    hipLaunchKernelGGL((delta_chunk_kernel<S, NT>), dim3(heads, (vp + 16 * NT - 1) / (16 * NT), n_seqs - seq0), dim3(256), \
                       delta_chunk_lds(S, NT), s, a, t, tile0, o, seq0);                                                 \
  }
#define X(S)         \
  if (dp == S) {     \
    if (wide)        \
      SGLK_DC(S, 4)  \
    else             \
      SGLK_DC(S, 2)  \
  }
  SGLK_DELTA_SIZES(X)
#undef X
#undef SGLK_DC
  SGLK_LAUNCH_CHECK();
  int tph = 1;
  while (tph * 8 < vp) tph *= 2;
  const int64_t threads = (int64_t)(M - first_row) * heads * tph;
  hipLaunchKernelGGL((delta_gate_kernel<bf16_t>), dim3((unsigned)((threads + 255) / 256)), dim3(256), 0, s, a, o, first_row, M, tph);
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}
}
