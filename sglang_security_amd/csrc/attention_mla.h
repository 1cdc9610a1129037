// The tile loop of absorbed latent attention (every query head reads the same latent rows, which serve as keys and,
// in their first elements, as values), shared by the kernels over 576 / 512 rows and over other sizes.
#pragma once
#include "attention_tile.h"

namespace sglk {

static constexpr int kMlaD = 576, kMlaDv = 512;
// rows at a padded pitch: an odd number of 16-byte slots, so the 16 rows of a K operand read fall on different slots
__host__ __device__ constexpr int mla_pitch(int D) { return D * 2 + 16; }
__host__ __device__ constexpr int mla_tile_bytes(int D) { return kTile * mla_pitch(D); }
static constexpr int kMlaTileBytes = mla_tile_bytes(kMlaD);  // 37376
static constexpr int kMlaScoreBytes = 4 * 2 * 64 * 16;       // four waves' partial score tiles, per tile of 16 heads

// HT: tiles of 16 query heads per block (2 where the group has 32 heads or more: a latent tile in LDS and every
// operand read out of it then serve twice the heads).
// CAP: the logit cap (tanh) compiled in; a run-time test per score splits the tile loop into blocks the scheduler
// cannot interleave.
// The tile loop of the absorbed-MLA kernels: a block of four waves multiplies HT tiles of 16 query columns (lane hl of
// tile t holds the column whose query row is qrow[t]; nullptr: a column that does not exist) against tokens
// [s0, s1) (non-empty) of the slot list idx, whose latent rows are at kbase + slot * k_stride_n.  On return m / lsum /
// oacc hold the running maximum (log2 domain), this lane's share of the sum and this wave's DV / 4 output elements
// per tile.
// D, DV: elements of a latent row (multiples of 64) and how many of its first ones are the value; wave w owns output
// elements [w * DV / 4, (w + 1) * DV / 4).
template <typename T, int HT, bool CAP, int D = kMlaD, int DV = kMlaDv>
struct MlaRun {
  static_assert(D % 64 == 0 && DV % 64 == 0 && DV <= D, "whole 16-byte pieces per thread, whole output tiles per wave");
  static constexpr int kPitch = mla_pitch(D);
  static constexpr int kSteps = D / 32;            // k-steps of the scores, dealt round-robin to the four waves
  static constexpr int kRounds = (kSteps + 3) / 4;
  static constexpr int kPieces = D / 64;           // 16-byte pieces of a row per fetching thread
  static constexpr int kOut = DV / 64;             // output tiles of 16 elements per wave
  float m[HT], lsum[HT];
  float4v oacc[HT][kOut];

  __device__ __forceinline__ void run(char* lds, const uint16_t* const (&qrow)[HT], const uint16_t* kbase,
                                      int64_t k_stride_n, const int32_t* idx, int s0, int s1, float sm_scale,
                                      float logit_cap) {
    char* tile = lds;
    float4v* sbuf = reinterpret_cast<float4v*>(lds + mla_tile_bytes(D));  // [HT][4 waves][2 halves][64 lanes]
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int hl = lane & 15, g = lane >> 4;
    // Q^T operand of this wave's k-steps wid, wid + 4, ...: lane (hl, g) holds q[column][32*ks + 8*g .. +8)
    short8 qf[HT][kRounds];
#pragma unroll
    for (int t = 0; t < HT; ++t) {
#pragma unroll
      for (int i = 0; i < kRounds; ++i) {
        const int ks = wid + 4 * i;
        if (qrow[t] && ks < kSteps)
          qf[t][i] = *reinterpret_cast<const short8*>(qrow[t] + 32 * ks + 8 * g);
        else
          qf[t][i] = short8{0, 0, 0, 0, 0, 0, 0, 0};
      }
    }
    const float LOG2E = 1.4426950408889634f;
    const float qk_scale = CAP ? sm_scale : sm_scale * LOG2E;
#pragma unroll
    for (int t = 0; t < HT; ++t) {
      m[t] = -INFINITY, lsum[t] = 0.f;
#pragma unroll
      for (int n = 0; n < kOut; ++n) oacc[t][n] = float4v{0.f, 0.f, 0.f, 0.f};
    }

    // tile fetch: eight threads per row, thread (row, sub) takes 16-byte pieces sub, sub + 8, ...
    const int frow = threadIdx.x >> 3, fsub = threadIdx.x & 7;
    // FD tiles are in flight (registers) while one is multiplied (two measured no faster than one, with or without
    // the slots read ahead: the step is not bound by the way to the rows and back)
    constexpr int FD = 1;
    int4v kreg[FD][kPieces];
    // a row's slot is read one tile before its bytes are requested (slot and bytes are two dependent trips to memory)
    auto slot_of = [&](int t0) {
      int tok = t0 + frow;
      tok = tok < s1 ? tok : s0;  // rows past the end re-read a valid slot; their scores are masked
      return idx[tok];
    };
    auto fetch = [&](int4v(&kr)[kPieces], int slot) {
      const uint16_t* row = kbase + (int64_t)slot * k_stride_n + fsub * 8;
#pragma unroll
      for (int j = 0; j < kPieces; ++j) kr[j] = *reinterpret_cast<const int4v*>(row + 64 * j);
    };
    int slot_next = 0;
    auto park = [&](const int4v(&kr)[kPieces]) {
#pragma unroll
      for (int j = 0; j < kPieces; ++j) *reinterpret_cast<int4v*>(tile + frow * kPitch + (fsub + 8 * j) * 16) = kr[j];
    };

    auto step = [&](int4v(&kr)[kPieces], int t0) {
      __syncthreads();  // every wave is done with the previous tile
      park(kr);
      __syncthreads();
      if (t0 + FD * kTile < s1) {  // later tiles' rows fly while this one is multiplied
        fetch(kr, slot_next);
        slot_next = slot_of(t0 + (FD + 1) * kTile);
      }
      // ---- this wave's share of S^T = K . Q^T: a K operand read serves every column tile
#pragma unroll
      for (int hh = 0; hh < 2; ++hh) {
        float4v sacc[HT];
#pragma unroll
        for (int t = 0; t < HT; ++t) sacc[t] = float4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < kRounds; ++i) {
          // k-steps past the row (the last round of some waves) multiply the row's last step by the zeros their
          // q registers hold there: no branch in the tile loop
          const int ks = min(wid + 4 * i, kSteps - 1);
          const short8 kf = *reinterpret_cast<const short8*>(tile + (16 * hh + hl) * kPitch + (4 * ks + g) * 16);
#pragma unroll
          for (int t = 0; t < HT; ++t) sacc[t] = Mfma16<T>::mma(kf, qf[t][i], sacc[t]);
        }
#pragma unroll
        for (int t = 0; t < HT; ++t) sbuf[((t * 4 + wid) * 2 + hh) * 64 + lane] = sacc[t];
      }
      __syncthreads();
      // ---- full scores (same sum order in every wave), scale / cap / mask, online softmax (exp2 domain)
      short8 pf[HT];  // P^T operand: k-slot j <-> token (j < 4 ? 4g + j : 16 + 4g + j - 4), as the S^T registers stand
#pragma unroll
      for (int t = 0; t < HT; ++t) {
        float sv[8];
        float tmax = -INFINITY;
#pragma unroll
        for (int hh = 0; hh < 2; ++hh) {
          float4v tot = sbuf[((t * 4) * 2 + hh) * 64 + lane];
#pragma unroll
          for (int w = 1; w < 4; ++w) tot += sbuf[((t * 4 + w) * 2 + hh) * 64 + lane];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            float sc = tot[r] * qk_scale;
            if constexpr (CAP) sc = logit_cap * tanhf(sc / logit_cap) * LOG2E;
            const int tok = t0 + 16 * hh + 4 * g + r;
            sc = tok < s1 ? sc : -INFINITY;
            sv[hh * 4 + r] = sc;
            tmax = fmaxf(tmax, sc);
          }
        }
        tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
        tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
        const float m_new = fmaxf(m[t], tmax);  // finite: token t0 of this tile is always valid
        const float alpha = exp2f(m[t] - m_new);
        m[t] = m_new;
        float psum = 0.f;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float p = exp2f(sv[j] - m_new);
          psum += p;
          pf[t][j] = (short)Conv<T>::from_f32(p);
        }
        lsum[t] = lsum[t] * alpha + psum;
#pragma unroll
        for (int n = 0; n < kOut; ++n) oacc[t][n] *= alpha;
      }
      // ---- O^T += V^T . P^T over this wave's DV / 4 output elements, V read transposed out of the K rows
#pragma unroll
      for (int n = 0; n < kOut; ++n) {
        const int byte_in_row = (DV / 2) * wid + 32 * n + 8 * (hl & 3);
        const short4v lo = lds_read_tr16(tile + (4 * g + (hl >> 2)) * kPitch + byte_in_row);
        const short4v hi = lds_read_tr16(tile + (16 + 4 * g + (hl >> 2)) * kPitch + byte_in_row);
        const short8 vf = short8{lo[0], lo[1], lo[2], lo[3], hi[0], hi[1], hi[2], hi[3]};
#pragma unroll
        for (int t = 0; t < HT; ++t) oacc[t][n] = Mfma16<T>::mma(vf, pf[t], oacc[t][n]);
      }
    };

#pragma unroll
    for (int f = 0; f < FD; ++f)
      if (s0 + f * kTile < s1) fetch(kreg[f], slot_of(s0 + f * kTile));
    slot_next = slot_of(s0 + FD * kTile);
    for (int t0 = s0; t0 < s1; t0 += FD * kTile) {
#pragma unroll
      for (int f = 0; f < FD; ++f)
        if (t0 + f * kTile < s1) step(kreg[f], t0 + f * kTile);  // block-uniform
    }
  }

  // tile t's partial (normalised O[DV] + log-sum-exp) into row `ob` of [rows][DV] / [rows]
  __device__ __forceinline__ void store(int t, bool ok, int64_t ob, float* __restrict__ logits, float* __restrict__ lse) const {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int g = lane >> 4;
    float ls = lsum[t];
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (ok) {
      const float inv = 1.0f / ls;
      float* dst = logits + ob * DV + (DV / 4) * wid;
#pragma unroll
      for (int n = 0; n < kOut; ++n) *reinterpret_cast<float4v*>(dst + 16 * n + 4 * g) = oacc[t][n] * inv;
      if (wid == 0 && g == 0) lse[ob] = (m[t] + log2f(ls)) * 0.6931471805599453f;
    }
  }
};

}  // namespace sglk
