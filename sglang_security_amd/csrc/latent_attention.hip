// Latent attention with sizes as parameters: a token caches one row [latent | rotated key part] (zero-padded: the latent to
// a multiple of 64, the rotated part to 64), every head's keys and values are linear in the latent.
//
//   latent_prep            the down projections' rows -> normalised query latent, normalised key/value latent + rotated
//                          key part into the pool
//   latent_rope_q          rotation of the heads' rotated query parts
//   head_gemm              one small product per head (keys folded into the query, values out of the mixed latents)
//   latent_decode          absorbed form over the pool: split over the window, tile loop of attention_mla.h
//   latent_prefill         keys and values of a run of tokens expanded once, attention over them under a sliding window
//   latent_attention_rows  absorbed form, one wave per (row, head): any size and type
//
// The visible range of a row at position p is (p - window, p]; pool slots are found through the request table.
#include <algorithm>

#include "attention_mla.h"
#include "common.h"
#include "row_source.h"

namespace sglk {

// ---------------------------------------------------------------------------------------------------------------------
// normalisation of both latents, rotation of the shared key part, pool write
// ---------------------------------------------------------------------------------------------------------------------
struct LatentPrep {
  RowSource src;           // columns [0, q_pitch) query latent, then r_pitch latent, then rot_dim rotated key part
  const float* wq;         // [q_pitch] norm weights, zero-padded
  const float* wkv;        // [r_pitch]
  void* cq;                // [rows, cq_stride]
  int64_t cq_stride;
  void* pool;              // [slots, pool_stride]
  int64_t pool_stride;
  const int32_t* loc;
  const float* cos_sin;    // [positions][rot_dims]: cos, then sin
  const int32_t* positions;
  int q_rank, q_pitch, kv_rank, r_pitch, rot_dim, rot_pitch, rot_dims;
  float eps;
};

// TPR threads per row (a wave, or the whole block), VPT pieces of eight elements per thread
template <typename T, int TPR, int VPT>
__global__ void __launch_bounds__(256) latent_prep_kernel(LatentPrep a, int M) {
  extern __shared__ float rotbuf[];  // [256 / TPR][rot_pitch]
  __shared__ float red[2][4];
  const int t = threadIdx.x % TPR, sub = threadIdx.x / TPR;
  const int m = blockIdx.x * (256 / TPR) + sub;
  const bool row_ok = m < M;
  const int row = row_ok ? m : M - 1;
  const int vq = a.q_pitch / 8, vk = vq + a.r_pitch / 8, nv = vk + a.rot_pitch / 8;
  float* rot = rotbuf + sub * a.rot_pitch;
  float x[VPT][8], sq = 0.f, sk = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int v = t + TPR * i;
#pragma unroll
    for (int j = 0; j < 8; ++j) x[i][j] = 0.f;
    if (v >= nv) continue;
    source8<T>(a.src, row, 8 * v, x[i]);
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) ss += x[i][j] * x[i][j];
    if (v < vq)
      sq += ss;
    else if (v < vk)
      sk += ss;
    else {
#pragma unroll
      for (int j = 0; j < 8; ++j) rot[8 * (v - vk) + j] = x[i][j];
    }
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if (TPR > 64 && (threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = sq;
    red[1][threadIdx.x >> 6] = sk;
  }
  __syncthreads();
  if (TPR > 64) {
    sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
    sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  }
  if (!row_ok) return;
  const float iq = 1.0f / sqrtf(sq / (float)a.q_rank + a.eps);
  const float ik = 1.0f / sqrtf(sk / (float)a.kv_rank + a.eps);
  const int64_t slot = (int64_t)a.loc[m] * a.pool_stride;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int v = t + TPR * i;
    if (v >= vk) continue;
    float w[8];
    if (v < vq) {
      ld8<float>(a.wq, 8 * v, w);
#pragma unroll
      for (int j = 0; j < 8; ++j) w[j] *= x[i][j] * iq;
      st8<T>(a.cq, (int64_t)m * a.cq_stride + 8 * v, w);
    } else {
      ld8<float>(a.wkv, 8 * (v - vq), w);
#pragma unroll
      for (int j = 0; j < 8; ++j) w[j] *= x[i][j] * ik;
      st8<T>(a.pool, slot + 8 * (v - vq), w);
    }
  }
  const float* cs = a.cos_sin + (int64_t)a.positions[m] * a.rot_dims;
  const int half = a.rot_dims / 2;
  for (int d = t; d < a.rot_pitch; d += TPR) {
    float v = d < a.rot_dim ? rot[d] : 0.f;
    if (d < a.rot_dims) {
      const int i = d < half ? d : d - half;
      float ra, rb;
      rope_pair(rot[i], rot[i + half], cs[i], cs[half + i], ra, rb);
      v = d < half ? ra : rb;
    }
    st<T>(a.pool, slot + a.r_pitch + d, v);
  }
}

// out[m][h][d] = rotation of src[m][h][d], d < rot_pitch (elements from rot_dims on are copied); may be in place
template <typename T>
__global__ void __launch_bounds__(256) latent_rope_q_kernel(const void* src, int64_t src_m, int64_t src_h, void* out, int64_t out_m,
                                                            int64_t out_h, const float* __restrict__ cos_sin,
                                                            const int32_t* __restrict__ positions, int M, int H, int rot_pitch,
                                                            int rot_dims) {
  const int half = rot_dims / 2, rest = rot_pitch - rot_dims, per = half + rest;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * H * per) return;
  const int i = (int)(idx % per);
  const int64_t mh = idx / per;
  const int h = (int)(mh % H), m = (int)(mh / H);
  const int64_t si = m * src_m + h * src_h, oi = m * out_m + h * out_h;
  if (i >= half) {
    const int d = rot_dims + i - half;
    st<T>(out, oi + d, ld<T>(src, si + d));
    return;
  }
  const float* cs = cos_sin + (int64_t)positions[m] * rot_dims;
  float ra, rb;
  rope_pair(ld<T>(src, si + i), ld<T>(src, si + i + half), cs[i], cs[half + i], ra, rb);
  st<T>(out, oi + i, ra);
  st<T>(out, oi + i + half, rb);
}

// whole rows turned (rot_dims == rot_pitch), eight pairs per thread, rows 16-byte aligned
template <typename T>
__global__ void __launch_bounds__(256) latent_rope_q8_kernel(const void* src, int64_t src_m, int64_t src_h, void* out, int64_t out_m,
                                                             int64_t out_h, const float* __restrict__ cos_sin,
                                                             const int32_t* __restrict__ positions, int M, int H, int rot) {
  const int half = rot / 2, per = half / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * H * per) return;
  const int i = (int)(idx % per) * 8;
  const int mh = (int)(idx / per), h = mh % H, m = mh / H;
  const int64_t si = m * src_m + h * src_h + i, oi = m * out_m + h * out_h + i;
  const float* cs = cos_sin + (int64_t)positions[m] * rot + i;
  float a[8], b[8], c[8], s[8];
  ld8<T>(src, si, a);
  ld8<T>(src, si + half, b);
  ld8<float>(cs, 0, c);
  ld8<float>(cs, half, s);
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    float ra, rb;
    rope_pair(a[j], b[j], c[j], s[j], ra, rb);
    a[j] = ra;
    b[j] = rb;
  }
  st8<T>(out, oi, a);
  st8<T>(out, oi + half, b);
}

// out[m][h][0 .. K) = the merged split partials part[m][h][S][K] (log-sum-exps lse [m][h][S]; -inf: nothing was left)
template <typename T>
__global__ void __launch_bounds__(256) latent_merge_kernel(const float* __restrict__ part, const float* __restrict__ lse, int S, int K,
                                                           void* __restrict__ out, int64_t rows) {
  const int nv = K / 8;
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= rows * nv) return;
  const int64_t row = idx / nv;
  const int c = (int)(idx - row * nv) * 8;
  const float* l = lse + row * S;
  float e_max = -INFINITY;
  for (int s = 0; s < S; ++s) e_max = fmaxf(e_max, l[s]);
  float acc[8], tot = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) acc[j] = 0.f;
  for (int s0 = 0; s0 < S; s0 += 4) {  // four splits' loads in flight
    float t[4][8], w[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      w[u] = s0 + u < S ? __expf(l[s0 + u] - e_max) : 0.f;
      if (w[u] > 0.f) {
        ld8<float>(part, (row * S + s0 + u) * K + c, t[u]);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) t[u][j] = 0.f;
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      tot += w[u];
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = fmaf(w[u], t[u][j], acc[j]);
    }
  }
  const float inv = 1.0f / tot;
#pragma unroll
  for (int j = 0; j < 8; ++j) acc[j] *= inv;
  st8<T>(out, row * K + c, acc);
}

// ---------------------------------------------------------------------------------------------------------------------
// out[m][h][n] = sum_k a[m][h][k] * w[h][n][k].  Weights in operand order [H][Np / 16][K / 32][64 lanes][8].  Wave w of a
// block owns rows 16 w .. of 64 and the block's NS strips of 16 columns; both operands go straight from memory into
// registers, eight k-steps ahead (a head's product is too small to pay for a trip through LDS and its barrier).
// ---------------------------------------------------------------------------------------------------------------------
template <int NS>
__global__ void __launch_bounds__(256) head_gemm_kernel(const uint16_t* __restrict__ a, int64_t a_m, int64_t a_h,
                                                        const uint16_t* __restrict__ w, uint16_t* __restrict__ out, int M, int N,
                                                        int Np, int K, int64_t out_m, int64_t out_h) {
  const int h = blockIdx.y;
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int i16 = lane & 15, g = lane >> 4;
  const int m0 = blockIdx.z * 64 + 16 * wid;
  if (m0 >= M) return;
  const int ksteps = K / 32, strip0 = blockIdx.x * NS;
  const uint16_t* as = a + (int64_t)min(m0 + i16, M - 1) * a_m + h * a_h + 8 * g;  // rows past M repeat the last one
  const uint16_t* ws[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s)
    ws[s] = w + (((int64_t)h * (Np / 16) + min(strip0 + s, Np / 16 - 1)) * ksteps) * 512 + 8 * lane;
  float4v acc[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) acc[s] = float4v{0.f, 0.f, 0.f, 0.f};
  constexpr int PF = 8;
  for (int k0 = 0; k0 < ksteps; k0 += PF) {
    short8 af[PF], bf[PF][NS];
#pragma unroll
    for (int j = 0; j < PF; ++j) {
      const int ks = min(k0 + j, ksteps - 1);
      af[j] = *reinterpret_cast<const short8*>(as + 32 * ks);
#pragma unroll
      for (int s = 0; s < NS; ++s) bf[j][s] = *reinterpret_cast<const short8*>(ws[s] + 512 * ks);
    }
#pragma unroll
    for (int j = 0; j < PF; ++j)
      if (k0 + j < ksteps) {
#pragma unroll
        for (int s = 0; s < NS; ++s) acc[s] = Mfma16<bf16_t>::mma(af[j], bf[j][s], acc[s]);
      }
  }
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    const int n = (strip0 + s) * 16 + i16;
    if (n >= N) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = m0 + 4 * g + r;
      if (m < M) out[m * out_m + h * out_h + n] = Conv<bf16_t>::from_f32(acc[s][r]);
    }
  }
}

// the same product for any type: weights row-major [H][Np][K], one output per thread
template <typename T>
__global__ void __launch_bounds__(256) head_gemm_rows_kernel(const void* __restrict__ a, int64_t a_m, int64_t a_h,
                                                             const void* __restrict__ w, void* __restrict__ out, int M, int H,
                                                             int N, int Np, int K, int64_t out_m, int64_t out_h) {
  const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (idx >= (int64_t)M * H * N) return;
  const int n = (int)(idx % N);
  const int64_t mh = idx / N;
  const int h = (int)(mh % H), m = (int)(mh / H);
  const int64_t ai = m * a_m + h * a_h, wi = ((int64_t)h * Np + n) * K;
  float s = 0.f;
  for (int k = 0; k < K; ++k) s = fmaf(ld<T>(a, ai + k), ld<T>(w, wi + k), s);
  st<T>(out, m * out_m + h * out_h + n, s);
}

// ---------------------------------------------------------------------------------------------------------------------
// absorbed form over the pool
// ---------------------------------------------------------------------------------------------------------------------
struct LatentRows {
  const void* q;       // [M, H, D]
  int64_t q_m, q_h;
  const void* pool;
  int64_t pool_stride;
  const int32_t* r2t;
  int64_t r2t_stride;
  const int32_t* req;        // request of row m
  const int32_t* positions;  // position of row m
  int H, window, splits;     // window <= 0: everything up to the position
  float scale;
};

template <int HT, int D, int DV>
__global__ void __launch_bounds__(256, HT == 1 ? 3 : 2) latent_decode_kernel(LatentRows a, float* __restrict__ part,
                                                                            float* __restrict__ lse) {
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int hl = threadIdx.x & 15;
  const int b = blockIdx.x, split = blockIdx.z;
  const int end = a.positions[b] + 1;
  const int lo = a.window > 0 ? max(0, end - a.window) : 0;
  const int len = end - lo;
  const int per = ((len + a.splits - 1) / a.splits + kTile - 1) / kTile * kTile;
  const int s0 = per * split, s1 = min(s0 + per, len);
  bool ok[HT];
  int head[HT];
  const uint16_t* qrow[HT];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    head[t] = (blockIdx.y * HT + t) * 16 + hl;
    ok[t] = head[t] < a.H;
    qrow[t] = ok[t] ? reinterpret_cast<const uint16_t*>(a.q) + b * a.q_m + head[t] * a.q_h : nullptr;
  }
  if (s1 <= s0) {  // block-uniform: an empty split says so
#pragma unroll
    for (int t = 0; t < HT; ++t)
      if (threadIdx.x < 16 && ok[t]) lse[((int64_t)b * a.H + head[t]) * a.splits + split] = -INFINITY;
    return;
  }
  MlaRun<bf16_t, HT, false, D, DV> r;
  r.run(lds, qrow, reinterpret_cast<const uint16_t*>(a.pool), a.pool_stride, a.r2t + a.req[b] * a.r2t_stride + lo, s0, s1,
        a.scale, 0.f);
#pragma unroll
  for (int t = 0; t < HT; ++t) r.store(t, ok[t], ((int64_t)b * a.H + head[t]) * a.splits + split, part, lse);
}

// one wave per (row, head): any size, any type; out[m][h][0 .. DV)
template <typename T, int PER>
__global__ void __launch_bounds__(64) latent_attention_rows_kernel(LatentRows a, void* __restrict__ out, int64_t out_m,
                                                                   int64_t out_h, int D, int DV) {
  extern __shared__ float qs[];
  const int m = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  for (int d = lane; d < D; d += 64) qs[d] = ld<T>(a.q, m * a.q_m + h * a.q_h + d);
  __syncthreads();
  const int end = a.positions[m] + 1;
  const int lo = a.window > 0 ? max(0, end - a.window) : 0;
  const int32_t* idx = a.r2t + a.req[m] * a.r2t_stride;
  float mx = -INFINITY, l = 0.f, acc[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) acc[i] = 0.f;
  for (int t0 = lo; t0 < end; t0 += 64) {
    const int tok = t0 + lane;
    const int64_t row = tok < end ? (int64_t)idx[tok] * a.pool_stride : 0;
    float s = -INFINITY;
    if (tok < end) {
      s = 0.f;
      for (int d = 0; d < D; ++d) s = fmaf(qs[d], ld<T>(a.pool, row + d), s);
      s *= a.scale;
    }
    const float m_new = fmaxf(mx, wave_max(s));
    const float alpha = expf(mx - m_new);
    const float p = tok < end ? expf(s - m_new) : 0.f;
    l = l * alpha + wave_sum(p);
    mx = m_new;
#pragma unroll
    for (int i = 0; i < PER; ++i) acc[i] *= alpha;
    const int cnt = min(64, end - t0);
    for (int j = 0; j < cnt; ++j) {
      const float pj = __shfl(p, j, 64);
      const int64_t rj = __shfl((long long)row, j, 64);
#pragma unroll
      for (int i = 0; i < PER; ++i) {
        const int d = lane + 64 * i;
        if (d < DV) acc[i] = fmaf(pj, ld<T>(a.pool, rj + d), acc[i]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int d = lane + 64 * i;
    if (d < DV) st<T>(out, m * out_m + h * out_h + d, acc[i] / l);
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// Expanded form: one block per (head, 64 * NC query rows of a sequence).  Keys [KD | 64]: KD expanded elements of the head,
// 64 of the shared rotated part; values VD.  Four waves share every 32-token tile through two LDS stages and multiply it
// against NC tiles of 16 query rows each: S^T = K . Q^T, O^T += V^T . P^T, as in attention_tile.h.
// ---------------------------------------------------------------------------------------------------------------------
struct LatentPrefill {
  const uint16_t* q;    // [rows, H, KD + 64], rotated
  int64_t q_m;
  const uint16_t* k;    // [tokens, k_n]: head h at h * KD
  int64_t k_n;
  const uint16_t* v;    // [tokens, v_n]: head h at h * VD
  int64_t v_n;
  const uint16_t* kr;   // [tokens, kr_n] rotated key parts
  int64_t kr_n;
  uint16_t* o;          // [rows, o_m]: head h at h * o_h, the first `vdim` of VD elements are stored
  int64_t o_m, o_h;
  const int32_t* row0;  // per sequence: first row, number of rows, first token, tokens in front of the first row
  const int32_t* rows;
  const int32_t* tok0;
  const int32_t* ahead;
  int H, vdim, window;
  float scale;
};

template <int KD, int VD, int NC>
__global__ void __launch_bounds__(256, 2) latent_prefill_kernel(LatentPrefill a) {
  constexpr int D = KD + 64;
  constexpr int KP = D * 2 + 16, VP = VD * 2 + 16;
  constexpr int kStage = kTile * (KP + VP);
  constexpr int KS = D / 32, NV = VD / 16, PK = KD / 64, PV = VD / 64;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int h = blockIdx.x, b = blockIdx.z;
  const int n = a.rows[b];
  const int i0 = blockIdx.y * 64 * NC;
  if (i0 >= n) return;  // block-uniform
  const int row0 = a.row0[b], ahead = a.ahead[b];
  const int64_t tok0 = a.tok0[b];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int hl = lane & 15, g = lane >> 4;
  const int window = a.window > 0 ? a.window : (1 << 30);
  const float qk_scale = a.scale * 1.4426950408889634f;

  short8 qf[NC][KS];
  int qpos[NC];
  bool ok[NC];
  int wmin = 1 << 30, wmax = -1;
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    const int first = i0 + (c * 4 + wid) * 16;  // interleaved: every wave gets early and late rows
    const int i = first + hl;
    ok[c] = i < n;
    qpos[c] = ahead + min(i, n - 1);
    if (first < n) {
      wmin = min(wmin, ahead + first);
      wmax = max(wmax, ahead + min(first + 15, n - 1));
    }
    const uint16_t* qr = a.q + (int64_t)(row0 + min(i, n - 1)) * a.q_m + h * D;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qf[c][ks] = *reinterpret_cast<const short8*>(qr + 32 * ks + 8 * g);
  }
  float m[NC], lsum[NC];
  float4v oacc[NC][NV];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    m[c] = -INFINITY;
    lsum[c] = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) oacc[c][i] = float4v{0.f, 0.f, 0.f, 0.f};
  }

  const int t_end = ahead + min(i0 + 64 * NC, n);
  const int t_begin = max(0, ahead + i0 - window + 1) & ~(kTile - 1);
  const int frow = threadIdx.x >> 3, fsub = threadIdx.x & 7;
  int4v kreg[PK + 1], vreg[PV];
  auto fetch = [&](int t0) {
    const int64_t tok = tok0 + min(t0 + frow, t_end - 1);  // rows past the end re-read a valid row; masked
    const uint16_t* kp = a.k + tok * a.k_n + h * KD + fsub * 8;
    const uint16_t* vp = a.v + tok * a.v_n + h * VD + fsub * 8;
#pragma unroll
    for (int j = 0; j < PK; ++j) kreg[j] = *reinterpret_cast<const int4v*>(kp + 64 * j);
    kreg[PK] = *reinterpret_cast<const int4v*>(a.kr + tok * a.kr_n + fsub * 8);
#pragma unroll
    for (int j = 0; j < PV; ++j) vreg[j] = *reinterpret_cast<const int4v*>(vp + 64 * j);
  };
  fetch(t_begin);
  int stage = 0;
  for (int t0 = t_begin; t0 < t_end; t0 += kTile) {
    char* kl = lds + stage * kStage;
    char* vl = kl + kTile * KP;
#pragma unroll
    for (int j = 0; j <= PK; ++j) *reinterpret_cast<int4v*>(kl + frow * KP + (fsub + 8 * j) * 16) = kreg[j];
#pragma unroll
    for (int j = 0; j < PV; ++j) *reinterpret_cast<int4v*>(vl + frow * VP + (fsub + 8 * j) * 16) = vreg[j];
    __syncthreads();
    if (t0 + kTile < t_end) fetch(t0 + kTile);
    stage ^= 1;
    if (t0 > wmax || t0 + kTile - 1 <= wmin - window) continue;  // wave-uniform: nothing of this tile is visible here
    float4v sacc[NC][2];
#pragma unroll
    for (int c = 0; c < NC; ++c) sacc[c][0] = sacc[c][1] = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int hh = 0; hh < 2; ++hh)
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const short8 kf = *reinterpret_cast<const short8*>(kl + (16 * hh + hl) * KP + (4 * ks + g) * 16);
#pragma unroll
        for (int c = 0; c < NC; ++c) sacc[c][hh] = Mfma16<bf16_t>::mma(kf, qf[c][ks], sacc[c][hh]);
      }
    // tiles every row of the wave sees whole need no mask
    const bool inner = t0 + kTile - 1 <= wmin && t0 > wmax - window;
    short8 pf[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      float sv[8], tmax = -INFINITY;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float s = sacc[c][j >> 2][j & 3] * qk_scale;
        if (!inner) {
          const int tok = t0 + 16 * (j >> 2) + 4 * g + (j & 3);
          s = (tok <= qpos[c] && qpos[c] - tok < window) ? s : -INFINITY;
        }
        sv[j] = s;
        tmax = fmaxf(tmax, s);
      }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float m_new = fmaxf(m[c], tmax);
      const float m_use = m_new == -INFINITY ? 0.f : m_new;  // nothing visible yet: everything stays zero
      const float alpha = exp2f(m[c] - m_use);
      m[c] = m_new;
      float psum = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float p = exp2f(sv[j] - m_use);
        psum += p;
        pf[c][j] = (short)Conv<bf16_t>::from_f32(p);
      }
      lsum[c] = lsum[c] * alpha + psum;
#pragma unroll
      for (int i = 0; i < NV; ++i) oacc[c][i] *= alpha;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int byte_in_row = 32 * i + 8 * (hl & 3);
      const short4v lo = lds_read_tr16(vl + (4 * g + (hl >> 2)) * VP + byte_in_row);
      const short4v hi = lds_read_tr16(vl + (16 + 4 * g + (hl >> 2)) * VP + byte_in_row);
      const short8 vf = short8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
#pragma unroll
      for (int c = 0; c < NC; ++c) oacc[c][i] = Mfma16<bf16_t>::mma(vf, pf[c], oacc[c][i]);
    }
  }
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    float tot = lsum[c];
    tot += __shfl_xor(tot, 16, 64);
    tot += __shfl_xor(tot, 32, 64);
    if (!ok[c]) continue;
    const float inv = 1.0f / tot;
    uint16_t* dst = a.o + (int64_t)(row0 + qpos[c] - ahead) * a.o_m + h * a.o_h;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int d = 16 * i + 4 * g;
      short4v pk;
#pragma unroll
      for (int r = 0; r < 4; ++r) pk[r] = (short)Conv<bf16_t>::from_f32(oacc[c][i][r] * inv);
      if (d + 4 <= a.vdim && (a.vdim & 3) == 0) {
        *reinterpret_cast<short4v*>(dst + d) = pk;
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (d + r < a.vdim) dst[d + r] = (uint16_t)pk[r];
      }
    }
  }
}

}  // namespace sglk

using namespace sglk;

extern "C" {

int sglk_latent_prep(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, const float* wq,
                     const float* wkv, void* cq, int64_t cq_stride, void* pool, int64_t pool_stride, const int32_t* loc,
                     const float* cos_sin, const int32_t* positions, int M, int q_rank, int q_pitch, int kv_rank, int r_pitch,
                     int rot_dim, int rot_pitch, int rot_dims, float eps, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && q_rank > 0 && kv_rank > 0 && rot_dim > 0, "latent_prep: bad shape");
  SGLK_CHECK(q_pitch >= q_rank && q_pitch % 8 == 0 && r_pitch >= kv_rank && r_pitch % 8 == 0 && rot_pitch >= rot_dim &&
                 rot_pitch % 8 == 0,
             "latent_prep: the parts of a row must be padded to multiples of 8");
  SGLK_CHECK(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= rot_dim, "latent_prep: rotation of %d of %d elements", rot_dims, rot_dim);
  SGLK_CHECK(pool_stride >= r_pitch + rot_pitch && pool_stride % 8 == 0 && cq_stride >= q_pitch && cq_stride % 8 == 0,
             "latent_prep: rows too short");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && wq && wkv && cq && pool && loc && cos_sin && positions, "latent_prep: null pointer");
  SGLK_CHECK(aligned16(cq) && aligned16(pool), "latent_prep: rows must be 16-byte aligned");
  const int cols = q_pitch + r_pitch + rot_pitch;
  SGLK_CHECK(cols <= 16384 && rot_pitch <= 1024, "latent_prep: rows of at most 16384 elements, 1024 of them rotated");
  SGLK_CHECK(aligned16(wq) && aligned16(wkv), "latent_prep: norm weights must be 16-byte aligned");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, cols, dtype, "latent_prep")) return rc;
  LatentPrep a{RowSource{src, src_f32, splits, part_stride, src_stride}, wq, wkv, cq, cq_stride, pool, pool_stride, loc, cos_sin,
               positions, q_rank, q_pitch, kv_rank, r_pitch, rot_dim, rot_pitch, rot_dims, eps};
  // many rows: a wave each; a decode batch: a block each
  const bool waves = M > 512 && cols <= 64 * 8 * 8;
  const int vpt = (cols / 8 + (waves ? 63 : 255)) / (waves ? 64 : 256);
#define SGLK_PREP(TPR, V)                                                                                                     \
  hipLaunchKernelGGL((latent_prep_kernel<T, TPR, V>), dim3((M + 256 / TPR - 1) / (256 / TPR)), dim3(256),                     \
                     (256 / TPR) * rot_pitch * 4, (hipStream_t)stream, a, M)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (waves && vpt <= 5)
      SGLK_PREP(64, 5);
    else if (waves)
      SGLK_PREP(64, 8);
    else if (vpt <= 2)
      SGLK_PREP(256, 2);
    else
      SGLK_PREP(256, 8);
  });
#undef SGLK_PREP
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_latent_rope_q(const void* src, int64_t src_m, int64_t src_h, void* out, int64_t out_m, int64_t out_h,
                       const float* cos_sin, const int32_t* positions, int M, int H, int rot_pitch, int rot_dims, int dtype,
                       void* stream) {
  SGLK_CHECK(M >= 0 && H > 0 && rot_dims >= 0 && rot_dims % 2 == 0 && rot_pitch >= rot_dims && rot_pitch > 0,
             "latent_rope_q: bad shape");
  SGLK_CHECK(src_h >= rot_pitch && out_h >= rot_pitch, "latent_rope_q: head stride too small");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && out && cos_sin && positions, "latent_rope_q: null pointer");
  const bool wide = rot_dims == rot_pitch && rot_dims % 16 == 0 && aligned16(src) && aligned16(out) && aligned16(cos_sin) &&
                    src_m % 8 == 0 && src_h % 8 == 0 && out_m % 8 == 0 && out_h % 8 == 0 && (int64_t)M * H < (1 << 30);
  if (wide) {
    const int64_t threads = (int64_t)M * H * (rot_dims / 16);
    SGLK_DISPATCH_FLOAT(dtype, T,
                        hipLaunchKernelGGL((latent_rope_q8_kernel<T>), dim3((unsigned)((threads + 255) / 256)), dim3(256), 0,
                                           (hipStream_t)stream, src, src_m, src_h, out, out_m, out_h, cos_sin, positions, M, H,
                                           rot_dims));
    SGLK_LAUNCH_CHECK();
    return SGLK_OK;
  }
  const int64_t total = (int64_t)M * H * (rot_pitch - rot_dims / 2);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((latent_rope_q_kernel<T>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, src, src_m, src_h, out, out_m, out_h, cos_sin, positions, M, H,
                                         rot_pitch, rot_dims));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_head_gemm(const void* a, int64_t a_m, int64_t a_h, const void* w, void* out, int M, int H, int N, int Np, int K,
                   int64_t out_m, int64_t out_h, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && H > 0 && N > 0 && Np >= N && Np % 16 == 0 && K > 0 && K % 32 == 0, "head_gemm: bad shape");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(a && w && out, "head_gemm: null pointer");
  SGLK_CHECK(out_h >= N && a_h >= K, "head_gemm: head stride too small");
  if (dtype != SGLK_BF16) {
    const int64_t total = (int64_t)M * H * N;
    SGLK_DISPATCH_FLOAT(dtype, T,
                        hipLaunchKernelGGL((head_gemm_rows_kernel<T>), dim3((unsigned)((total + 255) / 256)), dim3(256), 0,
                                           (hipStream_t)stream, a, a_m, a_h, w, out, M, H, N, Np, K, out_m, out_h));
    SGLK_LAUNCH_CHECK();
    return SGLK_OK;
  }
  SGLK_CHECK(aligned16(a) && aligned16(w) && a_m % 8 == 0 && a_h % 8 == 0, "head_gemm: rows must be 16-byte aligned");
  const int ns = (int64_t)H * (Np / 32) >= 256 ? 2 : 1;  // two strips per wave where that still covers the chip
  const dim3 grid((Np / 16 + ns - 1) / ns, H, (M + 63) / 64);
#define SGLK_HG(NS)                                                                                                       \
  hipLaunchKernelGGL((head_gemm_kernel<NS>), grid, dim3(256), 0, (hipStream_t)stream, (const uint16_t*)a, a_m, a_h,       \
                     (const uint16_t*)w, (uint16_t*)out, M, N, Np, K, out_m, out_h)
  if (ns == 2)
    SGLK_HG(2);
  else
    SGLK_HG(1);
#undef SGLK_HG
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_latent_merge(const float* part, const float* lse, int splits, void* out, int64_t rows, int K, int dtype, void* stream) {
  SGLK_CHECK(rows >= 0 && splits >= 1 && K > 0 && K % 8 == 0, "latent_merge: bad shape");
  if (rows == 0) return SGLK_OK;
  SGLK_CHECK(part && lse && out && aligned16(part) && aligned16(out), "latent_merge: null or unaligned pointer");
  const int64_t vecs = rows * (K / 8);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((latent_merge_kernel<T>), dim3((unsigned)((vecs + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, part, lse, splits, K, out, rows));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

// 1: sglk_latent_decode has a tile kernel for latents padded to r_pitch and a rotated part padded to rot_pitch
int sglk_latent_decode_supported(int r_pitch, int rot_pitch) {
  return rot_pitch == 64 && r_pitch % 64 == 0 && r_pitch >= 64 && r_pitch <= 512;
}

static int check_rows(const LatentRows& a, int M, const char* what) {
  SGLK_CHECK(M >= 0 && a.H > 0 && a.splits >= 1 && a.r2t_stride > 0, "%s: bad shape", what);
  SGLK_CHECK(M == 0 || (a.q && a.pool && a.r2t && a.req && a.positions), "%s: null pointer", what);
  return SGLK_OK;
}

int sglk_latent_decode(const void* q, int64_t q_m, int64_t q_h, const void* pool, int64_t pool_stride, const int32_t* r2t,
                       int64_t r2t_stride, const int32_t* req, const int32_t* positions, float* part, float* lse, int M, int H,
                       int r_pitch, int rot_pitch, int window, int splits, float scale, void* stream) {
  SGLK_CHECK(sglk_latent_decode_supported(r_pitch, rot_pitch), "latent_decode: no tile kernel for rows of %d + %d", r_pitch, rot_pitch);
  LatentRows a{q, q_m, q_h, pool, pool_stride, r2t, r2t_stride, req, positions, H, window, splits, scale};
  if (int rc = check_rows(a, M, "latent_decode")) return rc;
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(part && lse && aligned16(part), "latent_decode: null or unaligned pointer");
  SGLK_CHECK(aligned16(q) && aligned16(pool) && q_m % 8 == 0 && q_h % 8 == 0 && pool_stride % 8 == 0 &&
                 q_h >= r_pitch + rot_pitch && pool_stride >= r_pitch + rot_pitch,
             "latent_decode: rows must be 16-byte aligned and hold %d elements", r_pitch + rot_pitch);
  const int ht = H >= 32 ? 2 : 1;
  const dim3 grid(M, (H + 16 * ht - 1) / (16 * ht), splits);
#define SGLK_LD(HT, DV)                                                                                              \
  hipLaunchKernelGGL((latent_decode_kernel<HT, DV + 64, DV>), grid, dim3(256), mla_tile_bytes(DV + 64) + HT * kMlaScoreBytes, \
                     (hipStream_t)stream, a, part, lse)
#define SGLK_LD2(DV)   \
  case DV:             \
    if (ht == 2)       \
      SGLK_LD(2, DV);  \
    else               \
      SGLK_LD(1, DV);  \
    break
  switch (r_pitch) {
    SGLK_LD2(64);
    SGLK_LD2(128);
    SGLK_LD2(192);
    SGLK_LD2(256);
    SGLK_LD2(320);
    SGLK_LD2(384);
    SGLK_LD2(448);
    SGLK_LD2(512);
  }
#undef SGLK_LD2
#undef SGLK_LD
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_latent_attention_rows(const void* q, int64_t q_m, int64_t q_h, const void* pool, int64_t pool_stride,
                               const int32_t* r2t, int64_t r2t_stride, const int32_t* req, const int32_t* positions, void* out,
                               int64_t out_m, int64_t out_h, int M, int H, int D, int DV, int window, float scale, int dtype,
                               void* stream) {
  LatentRows a{q, q_m, q_h, pool, pool_stride, r2t, r2t_stride, req, positions, H, window, 1, scale};
  if (int rc = check_rows(a, M, "latent_attention_rows")) return rc;
  SGLK_CHECK(D > 0 && DV > 0 && DV <= D && D <= 8192 && DV <= 64 * 64, "latent_attention_rows: rows of %d / %d elements", D, DV);
  SGLK_CHECK(q_h >= D && pool_stride >= D && out_h >= DV, "latent_attention_rows: rows too short");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(out, "latent_attention_rows: null pointer");
#define SGLK_LR(PER)                                                                                                     \
  hipLaunchKernelGGL((latent_attention_rows_kernel<T, PER>), dim3(M, H), dim3(64), D * 4, (hipStream_t)stream, a, out, out_m, \
                     out_h, D, DV)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (DV <= 128)
      SGLK_LR(2);
    else if (DV <= 256)
      SGLK_LR(4);
    else if (DV <= 512)
      SGLK_LR(8);
    else if (DV <= 1024)
      SGLK_LR(16);
    else
      SGLK_LR(64);
  });
#undef SGLK_LR
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

// 1: sglk_latent_prefill has a tile kernel for keys of k_pitch + 64 and values of v_pitch elements per head
int sglk_latent_prefill_supported(int k_pitch, int v_pitch) {
  return (k_pitch == 64 || k_pitch == 128 || k_pitch == 192 || k_pitch == 256) && (v_pitch == 64 || v_pitch == 128 || v_pitch == 256);
}

int sglk_latent_prefill(const void* q, int64_t q_m, const void* k, int64_t k_n, const void* v, int64_t v_n, const void* kr,
                        int64_t kr_n, void* o, int64_t o_m, int64_t o_h, const int32_t* row0, const int32_t* rows,
                        const int32_t* tok0, const int32_t* ahead, int n_seqs, int max_rows, int H, int k_pitch, int v_pitch,
                        int vdim, int window, float scale, void* stream) {
  SGLK_CHECK(sglk_latent_prefill_supported(k_pitch, v_pitch), "latent_prefill: no tile kernel for heads of %d / %d", k_pitch, v_pitch);
  SGLK_CHECK(n_seqs >= 0 && max_rows >= 0 && H > 0 && vdim > 0 && vdim <= v_pitch, "latent_prefill: bad shape");
  if (n_seqs == 0 || max_rows == 0) return SGLK_OK;
  SGLK_CHECK(q && k && v && kr && o && row0 && rows && tok0 && ahead, "latent_prefill: null pointer");
  SGLK_CHECK(aligned16(q) && aligned16(k) && aligned16(v) && aligned16(kr) && q_m % 8 == 0 && k_n % 8 == 0 && v_n % 8 == 0 &&
                 kr_n % 8 == 0 && q_m >= (int64_t)H * (k_pitch + 64) && k_n >= (int64_t)H * k_pitch && v_n >= (int64_t)H * v_pitch,
             "latent_prefill: rows must be 16-byte aligned and hold every head");
  SGLK_CHECK(o_h >= vdim && (vdim % 4 != 0 || (o_h % 4 == 0 && o_m % 4 == 0 && (reinterpret_cast<uintptr_t>(o) & 7) == 0)),
             "latent_prefill: output rows must be 8-byte aligned");
  SGLK_CHECK(n_seqs <= 65535, "latent_prefill: at most 65535 sequences");
  LatentPrefill a{(const uint16_t*)q, q_m, (const uint16_t*)k, k_n, (const uint16_t*)v, v_n, (const uint16_t*)kr, kr_n,
                  (uint16_t*)o, o_m, o_h, row0, rows, tok0, ahead, H, vdim, window, scale};
  // heads run fastest: with a multiple of eight heads the query blocks of one head share an XCD's L2
#define SGLK_LP(KD, VD)                                                                                                  \
  if (k_pitch == KD && v_pitch == VD) {                                                                                  \
    constexpr int lds = 2 * kTile * ((KD + 64) * 2 + 16 + VD * 2 + 16);                                                  \
    if (int rc = ensure_lds<latent_prefill_kernel<KD, VD, 1>>(lds)) return rc;                                           \
    hipLaunchKernelGGL((latent_prefill_kernel<KD, VD, 1>), dim3(H, (max_rows + 63) / 64, n_seqs), dim3(256), lds,        \
                       (hipStream_t)stream, a);                                                                          \
  }
  SGLK_LP(64, 64)
  SGLK_LP(64, 128)
  SGLK_LP(64, 256)
  SGLK_LP(128, 64)
  SGLK_LP(128, 128)
  SGLK_LP(128, 256)
  SGLK_LP(192, 64)
  SGLK_LP(192, 128)
  SGLK_LP(192, 256)
  SGLK_LP(256, 64)
  SGLK_LP(256, 128)
  SGLK_LP(256, 256)
#undef SGLK_LP
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}
}
