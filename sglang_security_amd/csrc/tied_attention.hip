// Causal grouped-query attention whose values are its keys before their norm, with a learned bias by distance and a sink.
//
// A token caches one row per key/value head, v = the projected key, and one number per token: the key norm's reciprocal
// root mean square r.  The normalised key is r * w * v with a weight w per element, and w is folded into the query, so
//
//   score(i, j) = (q_i . v_j) r_j + bias[head][min(i - j, last)],   q_i = norm(query) * w * scale * temperature(i)
//
// and one row in LDS serves both products.  Scores, biases and sinks are in the base-2 domain (log2(e) is folded into
// the query's weight, the bias table and the sinks).
//
//   tied_prep      the projections' rows -> queries; rows and reciprocal root mean squares into the pool
//   tied_decode    single rows over the pool, split over the context, every wave with tiles of its own; with one split
//                  the rows are finished
//   tied_merge     split partials and the sink -> output rows
//   tied_prefill   runs of rows over the pool, 64 or 128 rows of a head per block
//   tied_rows      one wave per (row, head): any size and type
//
// A row at position p sees the positions [0, p]; pool slots are found through the request table.  The bias depends on the
// distance up to the table's last column only, so tiles further back than that take one number per head.
#include <algorithm>

#include "attention_tile.h"
#include "common.h"
#include "row_source.h"

namespace sglk {

// ---------------------------------------------------------------------------------------------------------------------
// norms over whole projections, pool write
// ---------------------------------------------------------------------------------------------------------------------
struct TiedPrep {
  RowSource src;           // columns [0, q_cols) queries, [q_cols, q_cols + k_cols) keys
  const float* bias;       // [q_cols + k_cols], zero in the padding
  const float* wq;         // [q_cols] weight of the query norm with everything that is folded into it
  const float* factor;     // [positions] temperature
  void* q;                 // [rows, q_cols]
  void* pool;              // [slots, pool_stride]
  int64_t pool_stride;
  float* rms;              // [slots]
  const int32_t* loc;
  const int32_t* positions;
  int q_cols, k_cols;      // padded
  int q_size, k_size;      // true sizes the norms run over
  float eps;
};

// one block of BT threads per row, VPT pieces of eight elements per thread
template <typename T, int BT, int VPT>
__global__ void __launch_bounds__(BT) tied_prep_kernel(TiedPrep a) {
  constexpr int NW = BT / 64;
  __shared__ float red[2][NW];
  const int m = blockIdx.x, vq = a.q_cols / 8, nv = vq + a.k_cols / 8;
  const float factor = a.factor[a.positions[m]];
  const int64_t slot = a.loc[m];
  float x[VPT][8], w[VPT][8], sq = 0.f, sk = 0.f;
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int v = threadIdx.x + BT * i;
    if (v >= nv) continue;
    float b[8];
    source8<T>(a.src, m, 8 * v, x[i]);
    ld8<float>(a.bias, 8 * v, b);
    if (v < vq) ld8<float>(a.wq, 8 * v, w[i]);
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      x[i][j] += b[j];
      ss += x[i][j] * x[i][j];
    }
    if (v < vq)
      sq += ss;
    else
      sk += ss;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = sq;
    red[1][threadIdx.x >> 6] = sk;
  }
  __syncthreads();
  sq = sk = 0.f;
#pragma unroll
  for (int i = 0; i < NW; ++i) {
    sq += red[0][i];
    sk += red[1][i];
  }
  const float iq = factor / sqrtf(sq / (float)a.q_size + a.eps);
  if (threadIdx.x == 0) a.rms[slot] = 1.0f / sqrtf(sk / (float)a.k_size + a.eps);
#pragma unroll
  for (int i = 0; i < VPT; ++i) {
    const int v = threadIdx.x + BT * i;
    if (v >= nv) continue;
    if (v < vq) {
#pragma unroll
      for (int j = 0; j < 8; ++j) w[i][j] *= x[i][j] * iq;
      st8<T>(a.q, (int64_t)m * a.q_cols + 8 * v, w[i]);
    } else {
      st8<T>(a.pool, slot * a.pool_stride + 8 * (v - vq), x[i]);
    }
  }
}

// ---------------------------------------------------------------------------------------------------------------------
// attention over the pool
// ---------------------------------------------------------------------------------------------------------------------
struct TiedAttn {
  const void* q;           // [rows, H, D]
  const void* pool;        // [slots, pool_stride]: key/value head g at g * D
  int64_t pool_stride;
  const float* rms;        // [slots]
  const int32_t* r2t;
  int64_t r2t_stride;
  const float* bias;       // [H][nb]
  const float* sink;       // [H]
  int H, share, nb;        // share: query heads per key/value head
};

__host__ __device__ constexpr int tied_pitch(int D) { return D * 2 + 16; }

struct TiedSplit {
  const int32_t* req;        // request of row m
  const int32_t* positions;  // position of row m
  float* part;               // [M][H][splits][D]
  float* lse;                // [M][H][splits], base 2 (-inf: nothing in this split)
  int splits;
  uint16_t* out;             // one split only: finished rows [M, out_stride], head h at h * D, instead of a partial
  int64_t out_stride;
  float out_scale;
};

__host__ __device__ constexpr int tied_decode_lds(int D) { return 4 * (kTile * tied_pitch(D) + kTile * 4); }

// Block: one row, HT tiles of 16 query heads of one key/value head, one split.  Wave w takes the split's tiles w, w + 4, ...:
// a tile's rows arrive in the layout of the K operand and pass through the wave's own LDS tile for the transposed
// reads of the V operand.  The waves' results are merged at the end.
template <int D, int HT>
__global__ void __launch_bounds__(256, D <= 128 && HT == 1 ? 3 : 1) tied_decode_kernel(TiedAttn a, TiedSplit s) {
  constexpr int KS = D / 32, NV = D / 16, P = tied_pitch(D), OP = D + 4;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  __shared__ float stat[2][HT][4][16];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int hl = lane & 15, g = lane >> 4;
  const int b = blockIdx.x, split = blockIdx.z;
  const int groups = (a.share + 16 * HT - 1) / (16 * HT);
  const int kv = blockIdx.y / groups, sub0 = (blockIdx.y % groups) * 16 * HT;
  const int pos = s.positions[b], end = pos + 1;
  const int tiles = (end + kTile - 1) / kTile, per = (tiles + s.splits - 1) / s.splits;
  const int t0 = per * split, t1 = min(t0 + per, tiles);
  int head[HT];
  bool ok[HT];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int sub = sub0 + 16 * t + hl;
    ok[t] = sub < a.share;
    head[t] = kv * a.share + min(sub, a.share - 1);
  }
  if (t0 >= t1) {  // block-uniform
    if (threadIdx.x < 16) {
#pragma unroll
      for (int t = 0; t < HT; ++t)
        if (ok[t]) s.lse[((int64_t)b * a.H + head[t]) * s.splits + split] = -INFINITY;
    }
    return;
  }
  char* tile = lds + wid * (kTile * P);
  float* rbuf = reinterpret_cast<float*>(lds + 4 * kTile * P) + wid * kTile;
  const int32_t* idx = a.r2t + s.req[b] * a.r2t_stride;
  const uint16_t* pool = reinterpret_cast<const uint16_t*>(a.pool) + kv * D + 8 * g;
  short8 kreg[2][KS];
  float rreg[2];
  int slot[2];
  auto slots_of = [&](int t) {
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) slot[hh] = idx[min(kTile * t + 16 * hh + hl, pos)];  // past the end: a valid row, masked
  };
  auto fetch = [&]() {
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
      const uint16_t* row = pool + (int64_t)slot[hh] * a.pool_stride;
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) kreg[hh][ks] = *reinterpret_cast<const short8*>(row + 32 * ks);
      rreg[hh] = a.rms[slot[hh]];
    }
  };
  if (t0 + wid < t1) {
    slots_of(t0 + wid);
    fetch();
    slots_of(min(t0 + wid + 4, t1 - 1));
  }
  short8 qf[HT][KS];
  float far[HT], m[HT], lsum[HT];
  const float* bt[HT];
  float4v oacc[HT][NV];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const uint16_t* qr = reinterpret_cast<const uint16_t*>(a.q) + ((int64_t)b * a.H + head[t]) * D + 8 * g;
#pragma unroll
    for (int ks = 0; ks < KS; ++ks) qf[t][ks] = *reinterpret_cast<const short8*>(qr + 32 * ks);
    bt[t] = a.bias + (int64_t)head[t] * a.nb;
    far[t] = bt[t][a.nb - 1];
    m[t] = -INFINITY;
    lsum[t] = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) oacc[t][i] = float4v{0.f, 0.f, 0.f, 0.f};
  }
  for (int t = t0 + wid; t < t1; t += 4) {  // wave-uniform
    float4v sacc[HT][2];
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
#pragma unroll
      for (int u = 0; u < HT; ++u) sacc[u][hh] = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        *reinterpret_cast<short8*>(tile + (16 * hh + hl) * P + (4 * ks + g) * 16) = kreg[hh][ks];
#pragma unroll
        for (int u = 0; u < HT; ++u) sacc[u][hh] = Mfma16<bf16_t>::mma(kreg[hh][ks], qf[u][ks], sacc[u][hh]);
      }
      if (g == 0) rbuf[16 * hh + hl] = rreg[hh];
    }
    if (t + 4 < t1) {  // the next tile's rows fly during the rest of this one
      fetch();
      slots_of(min(t + 8, t1 - 1));
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    float4v rr[2];
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) rr[hh] = *reinterpret_cast<const float4v*>(rbuf + 16 * hh + 4 * g);
    const int tok0 = kTile * t;
    const bool all_far = pos - (tok0 + kTile - 1) >= a.nb - 1;
    short8 pf[HT];
#pragma unroll
    for (int u = 0; u < HT; ++u) {
      float sv[8], tmax = -INFINITY;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float v = sacc[u][j >> 2][j & 3] * rr[j >> 2][j & 3];
        if (all_far) {
          v += far[u];
        } else {
          const int dist = pos - (tok0 + 16 * (j >> 2) + 4 * g + (j & 3));
          v = dist >= 0 ? v + bt[u][min(max(dist, 0), a.nb - 1)] : -INFINITY;
        }
        sv[j] = v;
        tmax = fmaxf(tmax, v);
      }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float m_new = fmaxf(m[u], tmax);  // finite: the tile's first token is visible
      const float alpha = __builtin_amdgcn_exp2f(m[u] - m_new);
      m[u] = m_new;
      float psum = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float p = __builtin_amdgcn_exp2f(sv[j] - m_new);
        psum += p;
        pf[u][j] = (short)Conv<bf16_t>::from_f32(p);
      }
      lsum[u] = lsum[u] * alpha + psum;
#pragma unroll
      for (int i = 0; i < NV; ++i) oacc[u][i] *= alpha;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int at = 32 * i + 8 * (hl & 3);
      const short4v lo = lds_read_tr16(tile + (4 * g + (hl >> 2)) * P + at);
      const short4v hi = lds_read_tr16(tile + (16 + 4 * g + (hl >> 2)) * P + at);
      const short8 vf = short8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
#pragma unroll
      for (int u = 0; u < HT; ++u) oacc[u][i] = Mfma16<bf16_t>::mma(vf, pf[u], oacc[u][i]);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  float* obuf = reinterpret_cast<float*>(lds);  // [4 waves][16 columns][OP]
#pragma unroll
  for (int u = 0; u < HT; ++u) {
    float l = lsum[u];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    __syncthreads();  // the tiles, or the previous column tile's results, have been read
    if (g == 0) {
      stat[0][u][wid][hl] = m[u];
      stat[1][u][wid][hl] = l;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) *reinterpret_cast<float4v*>(obuf + (wid * 16 + hl) * OP + 16 * i + 4 * g) = oacc[u][i];
    __syncthreads();
    const int c = threadIdx.x >> 4, e = threadIdx.x & 15;
    const int sub = sub0 + 16 * u + c;
    if (sub >= a.share) continue;
    float top = stat[0][u][0][c], w[4], tot = 0.f;
#pragma unroll
    for (int i = 1; i < 4; ++i) top = fmaxf(top, stat[0][u][i][c]);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      w[i] = __builtin_amdgcn_exp2f(stat[0][u][i][c] - top);
      tot += w[i] * stat[1][u][i][c];
    }
    const int64_t o = ((int64_t)b * a.H + kv * a.share + sub) * s.splits + split;
    float inv = 1.0f / tot;
    if (s.out) {  // the sink joins under the larger of the two maxima
      const float sink = a.sink[kv * a.share + sub], both = fmaxf(top, sink), own = exp2f(top - both);
      inv = s.out_scale * own / (tot * own + exp2f(sink - both));
    }
    for (int d = 4 * e; d < D; d += 64) {
      float4v v = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 4; ++i) v += *reinterpret_cast<const float4v*>(obuf + (i * 16 + c) * OP + d) * w[i];
      v *= inv;
      if (s.out) {
        short4v pk;
#pragma unroll
        for (int i = 0; i < 4; ++i) pk[i] = (short)Conv<bf16_t>::from_f32(v[i]);
        *reinterpret_cast<short4v*>(s.out + b * s.out_stride + (kv * a.share + sub) * D + d) = pk;
      } else {
        *reinterpret_cast<float4v*>(s.part + o * D + d) = v;
      }
    }
    if (e == 0 && !s.out) s.lse[o] = top + log2f(tot);
  }
}

// out[m][h * D + d] = out_scale * (merged split partials, the sink counted in the sum)
template <typename T>
__global__ void __launch_bounds__(256) tied_merge_kernel(const float* __restrict__ part, const float* __restrict__ lse,
                                                         const float* __restrict__ sink, int S, int H, int D, float out_scale,
                                                         void* __restrict__ out, int64_t out_stride, int64_t rows) {
  const int nv = D / 8;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * nv) return;
  const int64_t row = i / nv, m = row / H;
  const int c = (int)(i - row * nv) * 8, h = (int)(row - m * H);
  const float* l = lse + row * S;
  float top = sink[h];
  for (int s = 0; s < S; ++s) top = fmaxf(top, l[s]);
  float acc[8], tot = exp2f(sink[h] - top);
#pragma unroll
  for (int j = 0; j < 8; ++j) acc[j] = 0.f;
  for (int s0 = 0; s0 < S; s0 += 4) {  // four splits' loads in flight
    float t[4][8], w[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      w[u] = s0 + u < S ? exp2f(l[s0 + u] - top) : 0.f;
      if (w[u] > 0.f) {
        ld8<float>(part, (row * S + s0 + u) * D + c, t[u]);
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
  const float inv = out_scale / tot;
#pragma unroll
  for (int j = 0; j < 8; ++j) acc[j] *= inv;
  st8<T>(out, m * out_stride + (int64_t)h * D + c, acc);
}

struct TiedRuns {
  const int32_t* row0;   // per sequence: first row, number of rows, position of the first row, request
  const int32_t* rows;
  const int32_t* start;
  const int32_t* req;
  uint16_t* out;         // [rows, out_stride]: head h at h * D
  int64_t out_stride;
  float out_scale;
};

constexpr int kTiedBiasLds = 2048;  // columns of a head's bias table that are kept in LDS
__host__ __device__ constexpr int tied_prefill_lds(int D) { return 2 * (kTile * tied_pitch(D) + kTile * 4); }

// One block per (head, 64 * NC rows of a sequence): four waves share every 32-token tile through two LDS stages.
template <int D, int NC, bool BL>
__global__ void __launch_bounds__(256, 2) tied_prefill_kernel(TiedAttn a, TiedRuns r) {
  constexpr int KS = D / 32, NV = D / 16, P = tied_pitch(D), PIECES = (D + 63) / 64;
  constexpr int kStage = kTile * P + kTile * 4;
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int h = blockIdx.x, b = blockIdx.z;
  const int n = r.rows[b];
  const int i0 = ((int)gridDim.y - 1 - (int)blockIdx.y) * 64 * NC;  // the rows that see most start first
  if (i0 >= n) return;  // block-uniform
  const int row0 = r.row0[b], ahead = r.start[b];
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
  const int hl = lane & 15, g = lane >> 4;
  const int last = a.nb - 1;
  const float* gb = a.bias + (int64_t)h * a.nb;
  float* lb = reinterpret_cast<float*>(lds + 2 * kStage);
  if constexpr (BL)
    for (int i = threadIdx.x; i < a.nb; i += 256) lb[i] = gb[i];
  const float far = gb[last];

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
    const uint16_t* qr = reinterpret_cast<const uint16_t*>(a.q) + ((int64_t)(row0 + min(i, n - 1)) * a.H + h) * D;
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
  const int frow = threadIdx.x >> 3, fsub = threadIdx.x & 7;
  const int32_t* idx = a.r2t + r.req[b] * a.r2t_stride;
  const uint16_t* pool = reinterpret_cast<const uint16_t*>(a.pool) + (h / a.share) * D + fsub * 8;
  int4v kreg[PIECES];
  float rreg = 0.f;
  auto slot_of = [&](int t0) { return idx[min(t0 + frow, t_end - 1)]; };  // rows past the end: a valid row, masked
  auto fetch = [&](int slot) {
    const uint16_t* row = pool + (int64_t)slot * a.pool_stride;
#pragma unroll
    for (int j = 0; j < PIECES; ++j)
      if (D % 64 == 0 || fsub * 8 + 64 * j < D) kreg[j] = *reinterpret_cast<const int4v*>(row + 64 * j);
    if (fsub == 0) rreg = a.rms[slot];
  };
  fetch(slot_of(0));
  int slot_next = slot_of(kTile);
  int stage = 0;
  for (int t0 = 0; t0 < t_end; t0 += kTile) {
    char* kl = lds + stage * kStage;
    float* rl = reinterpret_cast<float*>(kl + kTile * P);
#pragma unroll
    for (int j = 0; j < PIECES; ++j)
      if (D % 64 == 0 || fsub * 8 + 64 * j < D) *reinterpret_cast<int4v*>(kl + frow * P + (fsub + 8 * j) * 16) = kreg[j];
    if (fsub == 0) rl[frow] = rreg;
    __syncthreads();
    if (t0 + kTile < t_end) {
      fetch(slot_next);
      slot_next = slot_of(t0 + 2 * kTile);
    }
    stage ^= 1;
    if (t0 > wmax) continue;  // wave-uniform: nothing of this tile is visible here
    float4v sacc[NC][2];
#pragma unroll
    for (int c = 0; c < NC; ++c) sacc[c][0] = sacc[c][1] = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int hh = 0; hh < 2; ++hh)
#pragma unroll
      for (int ks = 0; ks < KS; ++ks) {
        const short8 kf = *reinterpret_cast<const short8*>(kl + (16 * hh + hl) * P + (4 * ks + g) * 16);
#pragma unroll
        for (int c = 0; c < NC; ++c) sacc[c][hh] = Mfma16<bf16_t>::mma(kf, qf[c][ks], sacc[c][hh]);
      }
    float4v rr[2];
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) rr[hh] = *reinterpret_cast<const float4v*>(rl + 16 * hh + 4 * g);
    const bool all_far = wmin - (t0 + kTile - 1) >= last;  // then every row of the wave sees the tile whole, too
    short8 pf[NC];
#pragma unroll
    for (int c = 0; c < NC; ++c) {
      float sv[8], tmax = -INFINITY;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        float v = sacc[c][j >> 2][j & 3] * rr[j >> 2][j & 3];
        if (all_far) {
          v += far;
        } else {
          const int dist = qpos[c] - (t0 + 16 * (j >> 2) + 4 * g + (j & 3));
          const int at = min(max(dist, 0), last);
          const float bv = BL ? lb[at] : gb[at];
          v = dist >= 0 ? v + bv : -INFINITY;
        }
        sv[j] = v;
        tmax = fmaxf(tmax, v);
      }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float m_new = fmaxf(m[c], tmax);
      const float m_use = m_new == -INFINITY ? 0.f : m_new;  // nothing visible yet: everything stays zero
      const float alpha = __builtin_amdgcn_exp2f(m[c] - m_use);
      m[c] = m_new;
      float psum = 0.f;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const float p = __builtin_amdgcn_exp2f(sv[j] - m_use);
        psum += p;
        pf[c][j] = (short)Conv<bf16_t>::from_f32(p);
      }
      lsum[c] = lsum[c] * alpha + psum;
#pragma unroll
      for (int i = 0; i < NV; ++i) oacc[c][i] *= alpha;
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const int at = 32 * i + 8 * (hl & 3);
      const short4v lo = lds_read_tr16(kl + (4 * g + (hl >> 2)) * P + at);
      const short4v hi = lds_read_tr16(kl + (16 + 4 * g + (hl >> 2)) * P + at);
      const short8 vf = short8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
#pragma unroll
      for (int c = 0; c < NC; ++c) oacc[c][i] = Mfma16<bf16_t>::mma(vf, pf[c], oacc[c][i]);
    }
  }
  const float sink = a.sink[h];
#pragma unroll
  for (int c = 0; c < NC; ++c) {
    float tot = lsum[c];
    tot += __shfl_xor(tot, 16, 64);
    tot += __shfl_xor(tot, 32, 64);
    if (!ok[c]) continue;
    // the sink joins under the larger of the two maxima
    const float top = fmaxf(m[c], sink), own = exp2f(m[c] - top);
    const float inv = r.out_scale * own / (tot * own + exp2f(sink - top));
    uint16_t* dst = r.out + (int64_t)(row0 + qpos[c] - ahead) * r.out_stride + h * D;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      short4v pk;
#pragma unroll
      for (int e = 0; e < 4; ++e) pk[e] = (short)Conv<bf16_t>::from_f32(oacc[c][i][e] * inv);
      *reinterpret_cast<short4v*>(dst + 16 * i + 4 * g) = pk;
    }
  }
}

// one wave per (row, head): any size, any type
template <typename T, int PER>
__global__ void __launch_bounds__(64) tied_rows_kernel(TiedAttn a, const int32_t* __restrict__ req,
                                                       const int32_t* __restrict__ positions, float out_scale,
                                                       void* __restrict__ out, int64_t out_stride, int D) {
  extern __shared__ float qs[];
  const int m = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  for (int d = lane; d < D; d += 64) qs[d] = ld<T>(a.q, ((int64_t)m * a.H + h) * D + d);
  __syncthreads();
  const int pos = positions[m], end = pos + 1;
  const int32_t* idx = a.r2t + req[m] * a.r2t_stride;
  const int64_t kv = (int64_t)(h / a.share) * D;
  const float* bt = a.bias + (int64_t)h * a.nb;
  float mx = a.sink[h], l = 1.f, acc[PER];  // the sink is the first term of the sum
#pragma unroll
  for (int i = 0; i < PER; ++i) acc[i] = 0.f;
  for (int t0 = 0; t0 < end; t0 += 64) {
    const int tok = t0 + lane;
    int64_t row = 0;
    float s = -INFINITY;
    if (tok < end) {
      const int slot = idx[tok];
      row = slot * a.pool_stride + kv;
      s = 0.f;
      for (int d = 0; d < D; ++d) s = fmaf(qs[d], ld<T>(a.pool, row + d), s);
      s = s * a.rms[slot] + bt[min(pos - tok, a.nb - 1)];
    }
    const float m_new = fmaxf(mx, wave_max(s));
    const float alpha = exp2f(mx - m_new);
    const float p = tok < end ? exp2f(s - m_new) : 0.f;
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
        if (d < D) acc[i] = fmaf(pj, ld<T>(a.pool, rj + d), acc[i]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int d = lane + 64 * i;
    if (d < D) st<T>(out, m * out_stride + (int64_t)h * D + d, out_scale * acc[i] / l);
  }
}

}  // namespace sglk

using namespace sglk;

static int check_tied(const TiedAttn& a, int M, int D, const char* what) {
  SGLK_CHECK(M >= 0 && a.H > 0 && a.share > 0 && a.H % a.share == 0 && a.nb > 0 && D > 0 && D % 8 == 0 && a.r2t_stride > 0 &&
                 a.pool_stride >= (int64_t)(a.H / a.share) * D,
             "%s: bad shape", what);
  SGLK_CHECK(M == 0 || (a.q && a.pool && a.rms && a.r2t && a.bias && a.sink), "%s: null pointer", what);
  return SGLK_OK;
}

#define SGLK_TIED_ARGS                                                                                                    \
  const void *q, const void *pool, int64_t pool_stride, const float *rms, const int32_t *req_to_token, int64_t r2t_stride, \
      const float *bias, int nb, const float *sink, int H, int kv_heads, int D
#define SGLK_TIED_MAKE(what)                                                                                    \
  SGLK_CHECK(kv_heads > 0 && H > 0 && H % kv_heads == 0, what ": %d query heads over %d", H, kv_heads);           \
  const TiedAttn a{q, pool, pool_stride, rms, req_to_token, r2t_stride, bias, sink, H, H / kv_heads, nb}

// head sizes with tile kernels: the small ones also with two tiles of heads (or of rows) per wave
#define SGLK_TIED_SMALL(X) X(32) X(64) X(96) X(128)
#define SGLK_TIED_LARGE(X) X(192) X(256)

extern "C" {

int sglk_tied_prep(const void* src, int src_f32, int splits, int64_t part_stride, int64_t src_stride, const float* bias,
                   const float* wq, const float* factor, void* q, void* pool, int64_t pool_stride, float* rms, const int32_t* loc,
                   const int32_t* positions, int M, int q_cols, int k_cols, int q_size, int k_size, float eps, int dtype,
                   void* stream) {
  SGLK_CHECK(M >= 0 && q_size > 0 && k_size > 0 && q_cols >= q_size && k_cols >= k_size && q_cols % 8 == 0 && k_cols % 8 == 0 &&
                 pool_stride >= k_cols && pool_stride % 8 == 0,
             "tied_prep: bad shape");
  SGLK_CHECK(q_cols + k_cols <= 8 * 256 * 8, "tied_prep: rows of at most 16384 elements");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(src && bias && wq && factor && q && pool && rms && loc && positions, "tied_prep: null pointer");
  SGLK_CHECK(aligned16(q) && aligned16(pool) && aligned16(bias) && aligned16(wq), "tied_prep: unaligned pointer");
  if (int rc = check_source(src, src_f32, splits, part_stride, src_stride, q_cols + k_cols, dtype, "tied_prep")) return rc;
  const TiedPrep a{RowSource{src, src_f32, splits, part_stride, src_stride}, bias, wq, factor, q, pool, pool_stride, rms, loc,
                   positions, q_cols, k_cols, q_size, k_size, eps};
  const int vecs = (q_cols + k_cols) / 8;
  const bool wide = M <= 512 && vecs > 256;  // a decode batch: few rows, every piece on a thread of its own
#define SGLK_TP(BT, V) hipLaunchKernelGGL((tied_prep_kernel<T, BT, V>), dim3(M), dim3(BT), 0, (hipStream_t)stream, a)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (vecs <= 256)
      SGLK_TP(256, 1);
    else if (wide && vecs <= 768)
      SGLK_TP(768, 1);
    else if (wide)
      SGLK_TP(768, 3);
    else if (vecs <= 768)
      SGLK_TP(256, 3);
    else
      SGLK_TP(256, 8);
  });
#undef SGLK_TP
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

// 1: heads padded to D have tile kernels
int sglk_tied_supported(int D) {
#define X(S) if (D == S) return 1;
  SGLK_TIED_SMALL(X) SGLK_TIED_LARGE(X)
#undef X
  return 0;
}

int sglk_tied_decode(SGLK_TIED_ARGS, const int32_t* req, const int32_t* positions, float* part, float* lse, int M, int splits,
                     float out_scale, void* out, int64_t out_stride, void* stream) {
  SGLK_TIED_MAKE("tied_decode");
  if (int rc = check_tied(a, M, D, "tied_decode")) return rc;
  SGLK_CHECK(sglk_tied_supported(D), "tied_decode: no tile kernel for heads of %d", D);
  SGLK_CHECK(splits >= 1 && splits <= 65535, "tied_decode: bad split count");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(req && positions && (out || (part && lse)) && aligned16(part) && aligned16(q) && aligned16(pool) &&
                 pool_stride % 8 == 0 && aligned16(out),
             "tied_decode: null or unaligned pointer");
  SGLK_CHECK(!out || (splits == 1 && out_stride >= (int64_t)H * D && out_stride % 8 == 0),
             "tied_decode: finished rows come of one split");
  const TiedSplit s{req, positions, part, lse, splits, (uint16_t*)out, out_stride, out_scale};
  const int ht = a.share > 16 && D <= 128 ? 2 : 1;
  const dim3 grid(M, kv_heads * ((a.share + 16 * ht - 1) / (16 * ht)), splits);
  SGLK_CHECK(grid.y <= 65535, "tied_decode: too many heads");
#define SGLK_TD(S, HT)                                                                                                \
  {                                                                                                                   \
    if (int rc = ensure_lds<tied_decode_kernel<S, HT>>(tied_decode_lds(S))) return rc;                                \
    hipLaunchKernelGGL((tied_decode_kernel<S, HT>), grid, dim3(256), tied_decode_lds(S), (hipStream_t)stream, a, s);   \
  }
#define X(S)       \
  if (D == S) {    \
    if (ht == 2) { \
      SGLK_TD(S, 2) \
    } else {       \
      SGLK_TD(S, 1) \
    }              \
  }
#define Y(S) \
  if (D == S) SGLK_TD(S, 1)
  SGLK_TIED_SMALL(X)
  SGLK_TIED_LARGE(Y)
#undef X
#undef Y
#undef SGLK_TD
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_tied_merge(const float* part, const float* lse, const float* sink, int splits, float out_scale, void* out,
                    int64_t out_stride, int M, int H, int D, int dtype, void* stream) {
  SGLK_CHECK(M >= 0 && H > 0 && splits >= 1 && D > 0 && D % 8 == 0 && out_stride >= (int64_t)H * D && out_stride % 8 == 0,
             "tied_merge: bad shape");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(part && lse && sink && out && aligned16(part) && aligned16(out), "tied_merge: null or unaligned pointer");
  const int64_t vecs = (int64_t)M * H * (D / 8);
  SGLK_DISPATCH_FLOAT(dtype, T,
                      hipLaunchKernelGGL((tied_merge_kernel<T>), dim3((unsigned)((vecs + 255) / 256)), dim3(256), 0,
                                         (hipStream_t)stream, part, lse, sink, splits, H, D, out_scale, out, out_stride,
                                         (int64_t)M * H));
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_tied_prefill(SGLK_TIED_ARGS, const int32_t* row0, const int32_t* rows, const int32_t* start, const int32_t* req,
                      int n_seqs, int max_rows, float out_scale, void* out, int64_t out_stride, void* stream) {
  SGLK_TIED_MAKE("tied_prefill");
  if (int rc = check_tied(a, n_seqs, D, "tied_prefill")) return rc;
  SGLK_CHECK(sglk_tied_supported(D), "tied_prefill: no tile kernel for heads of %d", D);
  SGLK_CHECK(n_seqs <= 65535 && max_rows >= 0 && out_stride >= (int64_t)H * D && out_stride % 4 == 0, "tied_prefill: bad shape");
  if (n_seqs == 0 || max_rows == 0) return SGLK_OK;
  SGLK_CHECK(row0 && rows && start && req && out && aligned16(q) && aligned16(pool) && aligned16(out) && pool_stride % 8 == 0,
             "tied_prefill: null or unaligned pointer");
  const TiedRuns r{row0, rows, start, req, (uint16_t*)out, out_stride, out_scale};
  const bool bl = nb <= kTiedBiasLds;
  // heads run fastest: query blocks of one head share an XCD's L2 where the heads are a multiple of eight
#define SGLK_TF2(S, NC, BL)                                                                                            \
  {                                                                                                                    \
    constexpr int most = tied_prefill_lds(S) + (BL ? kTiedBiasLds * 4 : 0);                                            \
    if (int rc = ensure_lds<tied_prefill_kernel<S, NC, BL>>(most)) return rc;                                          \
    const dim3 grid(H, (max_rows + 64 * NC - 1) / (64 * NC), n_seqs);                                                  \
    SGLK_CHECK(grid.y <= 65535, "tied_prefill: too many rows");                                                        \
    hipLaunchKernelGGL((tied_prefill_kernel<S, NC, BL>), grid, dim3(256), tied_prefill_lds(S) + (BL ? nb * 4 : 0),      \
                       (hipStream_t)stream, a, r);                                                                     \
  }
#define SGLK_TF(S, NC)      \
  if (bl)                   \
    SGLK_TF2(S, NC, true)   \
  else                      \
    SGLK_TF2(S, NC, false)
  const bool wide = max_rows > 64 && (int64_t)H * n_seqs * ((max_rows + 127) / 128) >= 256;
#define X(S)       \
  if (D == S) {    \
    if (wide) {    \
      SGLK_TF(S, 2) \
    } else {       \
      SGLK_TF(S, 1) \
    }              \
  }
#define Y(S)       \
  if (D == S) {    \
    SGLK_TF(S, 1)  \
  }
  SGLK_TIED_SMALL(X)
  SGLK_TIED_LARGE(Y)
#undef X
#undef Y
#undef SGLK_TF
#undef SGLK_TF2
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}

int sglk_tied_rows(SGLK_TIED_ARGS, const int32_t* req, const int32_t* positions, float out_scale, void* out, int64_t out_stride,
                   int M, int dtype, void* stream) {
  SGLK_TIED_MAKE("tied_rows");
  if (int rc = check_tied(a, M, D, "tied_rows")) return rc;
  SGLK_CHECK(D <= 4096 && out_stride >= (int64_t)H * D && H <= 65535, "tied_rows: bad shape");
  if (M == 0) return SGLK_OK;
  SGLK_CHECK(req && positions && out, "tied_rows: null pointer");
#define SGLK_TR(PER)                                                                                                         \
  hipLaunchKernelGGL((tied_rows_kernel<T, PER>), dim3(M, H), dim3(64), D * 4, (hipStream_t)stream, a, req, positions, out_scale, \
                     out, out_stride, D)
  SGLK_DISPATCH_FLOAT(dtype, T, {
    if (D <= 128)
      SGLK_TR(2);
    else if (D <= 512)
      SGLK_TR(8);
    else
      SGLK_TR(64);
  });
#undef SGLK_TR
  SGLK_LAUNCH_CHECK();
  return SGLK_OK;
}
}
