// stack_ssd_mfma.h — the scalar-decay state-space recurrence S_t = g_t S_(t-1) + B_t (dt_t x_t)^T, y_t = S_t^T C_t + D x_t over long portions, 64 tokens at a time on
// the fp32 matrix cores (v_mfma_f32_32x32x2_f32: nothing is rounded below fp32).
// With cs_i = log g_1 + .. + log g_i inside a block of 64 tokens, the recurrence unrolls to three products per block:
//   y_i = sum_{j <= i} (C_i . B_j) exp(cs_i - cs_j) dt_j x_j  +  exp(cs_i) S_in^T C_i  +  D x_i,      S_out = exp(cs_64) S_in + sum_j B_j (exp(cs_64 - cs_j) dt_j x_j)^T
//   ssd_gram_kernel     C_i . B_j of every block and group (all heads of a group share it)
//   ssd_block_kernel    one workgroup per (entry, head, 32 value channels) walks the entry's blocks with the state in matrix-core accumulators
// The sums cs are kept in double: a difference of two sums must be as exact as a sum of few logarithms.  Blocks are counted from the entry's first token, and a block
// past the entry's end is padded by tokens with dt = 0 and log g = 0, which change nothing.
#pragma once
#include "prefill.h"
#include "stack_meta.h"

namespace tgx {

constexpr int SSD_BLOCK = 64;
struct SsdArgs {
  const float* row; long long ld;      // per token [x (heads E) | B (groups N) | C (groups N) | dt (heads) | decay (heads) | log decay (heads)]
  int heads, groups, N, E;             // N and heads E multiples of 4
  float* gram;                         // [blocks][groups][64][64]
  const float* skip;                   // [heads]
  float* S;                            // [slots][heads][N][E]
  float* out; long long ldo;           // [T][heads E]
};
// the first block of an entry in `gram`: entries never share a block
__device__ __forceinline__ int ssd_first_block(int start, int e) { return start / SSD_BLOCK + e; }

// G[i][j] = C_i . B_j, one 32 x 32 tile per wave (the tile above the diagonal is never read).  A lane holds one row of either operand: four consecutive channels per
// load, channel 8 q + 4 (lane / 32) + u as the two contraction slots of step 4 q + u.  Grid: (blocks of the longest entry, groups, entries).
template <int Q = SSD_BLOCK>
__global__ __launch_bounds__(256) void ssd_gram_kernel(StepMeta m, SsdArgs a) {
  const int b = blockIdx.x, g = blockIdx.y, e = blockIdx.z, cnt = m.ent_count[e], start = m.ent_start[e];
  static_assert(Q == 64, "four tiles of 32 x 32");
  if (b * Q >= cnt) return;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, half = lane >> 5, l31 = lane & 31, it = wv >> 1, jt = wv & 1;
  if (jt > it) return;
  const int i = b * Q + 32 * it + l31, j = b * Q + 32 * jt + l31;
  const float* cr = a.row + (size_t)(start + min(i, cnt - 1)) * a.ld + (size_t)a.heads * a.E + (size_t)(a.groups + g) * a.N;
  const float* br = a.row + (size_t)(start + min(j, cnt - 1)) * a.ld + (size_t)a.heads * a.E + (size_t)g * a.N;
  f32x16 acc;
#pragma unroll
  for (int r = 0; r < 16; r++) acc[r] = 0.f;
  for (int q = 0; q < (a.N + 7) / 8; q++) {
    const int n = 8 * q + 4 * half;
    const f32x4 z = {0.f, 0.f, 0.f, 0.f};
    const f32x4 cv = n < a.N ? *reinterpret_cast<const f32x4*>(cr + n) : z, bv = n < a.N ? *reinterpret_cast<const f32x4*>(br + n) : z;
#pragma unroll
    for (int u = 0; u < 4; u++) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(cv[u], bv[u], acc, 0, 0, 0);
  }
  float* G = a.gram + ((size_t)(ssd_first_block(start, e) + b) * a.groups + g) * (Q * Q);
#pragma unroll
  for (int r = 0; r < 16; r++) G[(32 * it + (r & 3) + 8 * (r >> 2) + 4 * half) * Q + 32 * jt + l31] = acc[r];
}

// NW: 32-row tiles of the state per wave (4 NW 32 >= N).  Wave w owns the state rows n of its tiles and 32 columns, in the accumulator layout: register r of a lane is
// row (r & 3) + 8 (r >> 2) + 4 (lane / 32), column lane % 32.  Register r of the two half-waves is at the same time a B operand whose two contraction slots are those
// two rows, so S^T C needs no transposition: its A operand takes C's channels in that order.  A wave contributes its rows' share of S^T C and the share of sixteen
// keys j of the block's own product; the four waves' shares are added up in LDS.  Grid: (entries, heads, E / 32).
template <int NW>
__global__ __launch_bounds__(256, 1) void ssd_block_kernel(StepMeta m, SsdArgs a) {
  constexpr int Q = SSD_BLOCK;
  constexpr double LOG2E = 1.4426950408889634;
  __shared__ float s_x[2][Q][32];
  __shared__ double s_cs[2][Q];        // base-2 logarithms, summed from the block's start
  __shared__ float s_dt[2][Q];
  __shared__ float s_part[4][Q][33];
  const int e = blockIdx.x, h = blockIdx.y, e0 = blockIdx.z * 32, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, half = lane >> 5, l31 = lane & 31;
  const int start = m.ent_start[e], cnt = m.ent_count[e], slot = m.ent_row[e], grp = h / (a.heads / a.groups);
  const bool fresh = m.tok_pos[start] == 0;
  const float* base = a.row + (size_t)start * a.ld;
  const size_t oB = (size_t)a.heads * a.E + (size_t)grp * a.N, oC = oB + (size_t)a.groups * a.N, oD = (size_t)a.heads * a.E + 2 * (size_t)a.groups * a.N + h, oL = oD + 2 * (size_t)a.heads;
  const float* gram = a.gram + ((size_t)ssd_first_block(start, e) * a.groups + grp) * (Q * Q);
  float* Sg = a.S + ((size_t)slot * a.heads + h) * (size_t)a.N * a.E;
  const bool colok = e0 + l31 < a.E;
  f32x16 S[NW];
#pragma unroll
  for (int w = 0; w < NW; w++)
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int n = 32 * (wv * NW + w) + (r & 3) + 8 * (r >> 2) + 4 * half;
      S[w][r] = (!fresh && n < a.N && colok) ? Sg[(size_t)n * a.E + e0 + l31] : 0.f;
    }
  // operands of one block, fetched a block ahead: B[n][j] with j = kk + 32 half (the state's product), C[i][n] four channels at a time, the Gram rows of this wave's
  // sixteen keys j = 16 wv + 8 half + 0 .. 7, the value columns, step sizes and log decays
  struct Ops { float B[NW][32]; f32x4 C[NW][2][4]; f32x4 G[2][2]; float x[8]; float dt, la; };
  Ops cur, nxt;
  auto fetch = [&](Ops& o, int b) {
    const int t0 = b * Q, left = cnt - t0;
#pragma unroll
    for (int w = 0; w < NW; w++) {
      const int n = 32 * (wv * NW + w) + l31;
#pragma unroll
      for (int kk = 0; kk < 32; kk++) { const int j = kk + 32 * half; o.B[w][kk] = (j < left && n < a.N) ? base[(size_t)(t0 + j) * a.ld + oB + n] : 0.f; }
#pragma unroll
      for (int it = 0; it < 2; it++)
#pragma unroll
        for (int q = 0; q < 4; q++) {
          const int i = 32 * it + l31, nc = 32 * (wv * NW + w) + 8 * q + 4 * half;
          o.C[w][it][q] = (i < left && nc < a.N) ? *reinterpret_cast<const f32x4*>(base + (size_t)(t0 + i) * a.ld + oC + nc) : f32x4{0.f, 0.f, 0.f, 0.f};
        }
    }
    const float* G = gram + (size_t)b * a.groups * (Q * Q);
#pragma unroll
    for (int it = 0; it < 2; it++)
#pragma unroll
      for (int q = 0; q < 2; q++) {
        const int j = 16 * wv + 8 * half + 4 * q;
        o.G[it][q] = j <= 32 * it + 31 ? *reinterpret_cast<const f32x4*>(G + (32 * it + l31) * Q + j) : f32x4{0.f, 0.f, 0.f, 0.f};
      }
#pragma unroll
    for (int u = 0; u < 8; u++) { const int t = (tid >> 5) + 8 * u; o.x[u] = (t < left && colok) ? base[(size_t)(t0 + t) * a.ld + (size_t)h * a.E + e0 + l31] : 0.f; }
    if (wv == 0) { o.dt = lane < left ? base[(size_t)(t0 + lane) * a.ld + oD] : 0.f; o.la = lane < left ? base[(size_t)(t0 + lane) * a.ld + oL] : 0.f; }
  };
  auto stage = [&](const Ops& o, int buf) {
#pragma unroll
    for (int u = 0; u < 8; u++) s_x[buf][(tid >> 5) + 8 * u][l31] = o.x[u];
    if (wv == 0) {
      double v = (double)o.la * LOG2E;
#pragma unroll
      for (int d = 1; d < 64; d <<= 1) { const double p = __shfl_up(v, d, 64); if (lane >= d) v += p; }
      s_cs[buf][lane] = v; s_dt[buf][lane] = o.dt;
    }
  };
  const float Dh = a.skip[h];
  const int nblk = (cnt + Q - 1) / Q;
  fetch(cur, 0);
  stage(cur, 0);
  for (int b = 0; b < nblk; b++) {
    const int buf = b & 1, t0 = b * Q;
    __syncthreads();      // the block's columns and sums stand; the shares of the block before have been read
    if (b + 1 < nblk) fetch(nxt, b + 1);
    f32x16 acc[2];
#pragma unroll
    for (int it = 0; it < 2; it++)
#pragma unroll
      for (int r = 0; r < 16; r++) acc[it][r] = 0.f;
    double csi[2];
#pragma unroll
    for (int it = 0; it < 2; it++) csi[it] = s_cs[buf][32 * it + l31];
    // exp(cs_i) S_in^T C_i over this wave's state rows
#pragma unroll
    for (int it = 0; it < 2; it++) {
      const float ei = __builtin_amdgcn_exp2f((float)csi[it]);
#pragma unroll
      for (int w = 0; w < NW; w++)
        if (32 * (wv * NW + w) < a.N)      // (wave-uniform)
#pragma unroll
          for (int r = 0; r < 16; r++) acc[it] = __builtin_amdgcn_mfma_f32_32x32x2f32(cur.C[w][it][r >> 2][r & 3] * ei, S[w][r], acc[it], 0, 0, 0);
    }
    // the block's own tokens: this wave's sixteen keys
#pragma unroll
    for (int k = 0; k < 8; k++) {
      const int j = 16 * wv + 8 * half + k;
      const double csj = s_cs[buf][j];
      const float xj = s_x[buf][j][l31] * s_dt[buf][j];
#pragma unroll
      for (int it = 0; it < 2; it++) {
        if (16 * wv > 32 * it + 31) continue;      // (wave-uniform: all of the wave's keys lie behind these rows)
        const float mij = j <= 32 * it + l31 ? cur.G[it][k >> 2][k & 3] * __builtin_amdgcn_exp2f((float)(csi[it] - csj)) : 0.f;
        acc[it] = __builtin_amdgcn_mfma_f32_32x32x2f32(mij, xj, acc[it], 0, 0, 0);
      }
    }
#pragma unroll
    for (int it = 0; it < 2; it++)
#pragma unroll
      for (int r = 0; r < 16; r++) s_part[wv][32 * it + (r & 3) + 8 * (r >> 2) + 4 * half][l31] = acc[it][r];
    // S_out
    const double cse = s_cs[buf][Q - 1];
    const float ge = __builtin_amdgcn_exp2f((float)cse);
#pragma unroll
    for (int w = 0; w < NW; w++)
#pragma unroll
      for (int r = 0; r < 16; r++) S[w][r] *= ge;
#pragma unroll
    for (int kk = 0; kk < 32; kk++) {
      const int j = kk + 32 * half;
      const float xs = s_x[buf][j][l31] * s_dt[buf][j] * __builtin_amdgcn_exp2f((float)(cse - s_cs[buf][j]));
#pragma unroll
      for (int w = 0; w < NW; w++)
        if (32 * (wv * NW + w) < a.N) S[w] = __builtin_amdgcn_mfma_f32_32x32x2f32(cur.B[w][kk], xs, S[w], 0, 0, 0);
    }
    if (b + 1 < nblk) stage(nxt, buf ^ 1);
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int t = (tid >> 5) + 8 * u;
      if (t0 + t < cnt && colok)
        a.out[(size_t)(start + t0 + t) * a.ldo + (size_t)h * a.E + e0 + l31] =
            fmaf(Dh, s_x[buf][t][l31], s_part[0][t][l31] + s_part[1][t][l31] + s_part[2][t][l31] + s_part[3][t][l31]);
    }
    cur = nxt;
  }
#pragma unroll
  for (int w = 0; w < NW; w++)
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int n = 32 * (wv * NW + w) + (r & 3) + 8 * (r >> 2) + 4 * half;
      if (n < a.N && colok) Sg[(size_t)n * a.E + e0 + l31] = S[w][r];
    }
}

}  // namespace tgx
