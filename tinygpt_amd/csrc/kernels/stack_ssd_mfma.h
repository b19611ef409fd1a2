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
  const float* fixed; float dt0;       // [2][heads] decays and their logarithms that hold for every token, with dt0 as every token's dt (the rows then end behind C; nullptr: per token)
  const float* skip;                   // [heads] (nullptr: none)
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
// Operands travel straight from memory to registers (every wave reads its own state rows only): B of a block is asked for at the block's start and used at its end,
// C and the Gram rows of the next block replace the present ones as soon as these are used up, so nothing is held twice.  Rows past the
// entry's end are clamped to its last one (what is read there twice meets dt = 0 or is not stored).
template <int NW>
__global__ __launch_bounds__(256, NW == 1 ? 2 : 1) void ssd_block_kernel(StepMeta m, SsdArgs a) {
  constexpr int Q = SSD_BLOCK;
  constexpr double LOG2E = 1.4426950408889634;
  __shared__ float s_x[2][Q][32];
  __shared__ double s_cs[2][Q];        // base-2 logarithms, summed from the block's start
  __shared__ float s_dt[2][Q], s_end[2][Q];      // dt_j, exp(cs_64 - cs_j) dt_j
  __shared__ float s_part[4][Q][33];
  const int e = blockIdx.x, h = blockIdx.y, e0 = blockIdx.z * 32, tid = threadIdx.x, lane = tid & 63, wv = __builtin_amdgcn_readfirstlane(tid >> 6), half = lane >> 5, l31 = lane & 31;
  const int start = m.ent_start[e], cnt = m.ent_count[e], slot = m.ent_row[e], grp = h / (a.heads / a.groups);
  const bool fresh = m.tok_pos[start] == 0;
  const int ld = (int)a.ld, oX = h * a.E + e0, oB = a.heads * a.E + grp * a.N, oC = oB + a.groups * a.N, oD = a.heads * a.E + 2 * a.groups * a.N + h, oL = oD + 2 * a.heads;
  const float* base = a.row + (size_t)start * ld;
  const float* gram = a.gram + ((size_t)ssd_first_block(start, e) * a.groups + grp) * (Q * Q);
  float* Sg = a.S + ((size_t)slot * a.heads + h) * (size_t)a.N * a.E;
  const bool colok = e0 + l31 < a.E;
  const int xcol = colok ? l31 : 0, n0 = 32 * wv * NW;
  f32x16 S[NW];
#pragma unroll
  for (int w = 0; w < NW; w++)
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int n = n0 + 32 * w + (r & 3) + 8 * (r >> 2) + 4 * half;
      S[w][r] = (!fresh && n < a.N && colok) ? Sg[(size_t)n * a.E + e0 + l31] : 0.f;
    }
  auto at = [](const float* p, unsigned int bytes) -> const float* { return reinterpret_cast<const float*>(reinterpret_cast<const char*>(p) + bytes); };
  // byte offset of row t0 + k of a block with `left` rows, clamped to its last one (ld < 2^21 floats: the factors fit 24 bits); the constant k stays out of registers
  auto row_off = [&](int t0, int k, int left) -> unsigned int { return (unsigned int)(4 * (__mul24(t0, ld) + __mul24(min(k, left - 1 - t0), ld))); };
  float B[NW][32], x[8], dt = 0.f, la = 0.f;      // B[n][j]: j = kk + 32 half
  f32x4 C[NW][2][4], G[2][2];                     // C[i][n]: four channels at a time; the Gram rows of this wave's sixteen keys j = 16 wv + 8 half + 0 .. 7
  // (what stands in state rows beyond N is finite and meets a factor of zero)
  auto fetch_B = [&](int b) {
    const float* p = base + (size_t)b * Q * ld + oB;
    const int left = cnt - b * Q;
#pragma unroll
    for (int w = 0; w < NW; w++) {
      const int n = min(n0 + 32 * w + l31, a.N - 1);
#pragma unroll
      for (int kk = 0; kk < 32; kk++) B[w][kk] = *at(p, row_off(32 * half, kk, left) + 4 * n);
    }
  };
  auto fetch_C = [&](int b) {
    const float* p = base + (size_t)b * Q * ld + oC;
    const int left = cnt - b * Q;
#pragma unroll
    for (int w = 0; w < NW; w++)
#pragma unroll
      for (int it = 0; it < 2; it++)
#pragma unroll
        for (int q = 0; q < 4; q++) {
          const int n = n0 + 32 * w + 8 * q + 4 * half;
          C[w][it][q] = *reinterpret_cast<const f32x4*>(at(p, row_off(l31, 32 * it, left) + 4 * min(n, a.N - 4)));
        }
  };
  auto fetch_G = [&](int b) {
    const float* p = gram + (size_t)b * a.groups * (Q * Q);
#pragma unroll
    for (int it = 0; it < 2; it++)
      if (16 * wv <= 32 * it + 31)
#pragma unroll
        for (int q = 0; q < 2; q++) G[it][q] = *reinterpret_cast<const f32x4*>(at(p, 4u * (unsigned int)((32 * it + l31) * Q + 16 * wv + 8 * half + 4 * q)));
  };
  auto fetch_x = [&](int b) {
    const float* p = base + (size_t)b * Q * ld;
    const int left = cnt - b * Q;
#pragma unroll
    for (int u = 0; u < 8; u++) x[u] = *at(p, row_off(tid >> 5, 8 * u, left) + 4 * (oX + xcol));
    if (wv == 0 && !a.fixed) { const unsigned int off = row_off(lane, 0, left); dt = *at(p + oD, off); la = *at(p + oL, off); }
  };
  auto stage = [&](int b) {
    const int buf = b & 1, left = cnt - b * Q;
#pragma unroll
    for (int u = 0; u < 8; u++) s_x[buf][(tid >> 5) + 8 * u][l31] = x[u];
    if (wv == 0) {
      double v = lane < left ? (double)la * LOG2E : 0.0;
      const float d = lane < left ? dt : 0.f;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) { const double p = __shfl_up(v, o, 64); if (lane >= o) v += p; }
      const double end = __shfl(v, 63, 64);
      s_cs[buf][lane] = v; s_dt[buf][lane] = d; s_end[buf][lane] = d * __builtin_amdgcn_exp2f((float)(end - v));
    }
  };
  if (a.fixed) { dt = a.dt0; la = a.fixed[a.heads + h]; }
  const float Dh = a.skip ? a.skip[h] : 0.f;
  const int nblk = (cnt + Q - 1) / Q;
  fetch_x(0); fetch_C(0); fetch_G(0);
  stage(0);
  for (int b = 0; b < nblk; b++) {
    const int buf = b & 1, t0 = b * Q;
    const bool more = b + 1 < nblk;
    __syncthreads();      // the block's columns and sums stand; the shares of the block before have been read
    fetch_B(b);
    if (more) fetch_x(b + 1);
    __builtin_amdgcn_sched_barrier(0);      // (the phases stay apart: operands of a later one must not take registers early)
    f32x16 acc[2];
#pragma unroll
    for (int it = 0; it < 2; it++)
#pragma unroll
      for (int r = 0; r < 16; r++) acc[it][r] = 0.f;
    double csi[2];
    float ei[2];
#pragma unroll
    for (int it = 0; it < 2; it++) { csi[it] = s_cs[buf][32 * it + l31]; ei[it] = __builtin_amdgcn_exp2f((float)csi[it]); }
    // exp(cs_i) S_in^T C_i over this wave's state rows
#pragma unroll
    for (int w = 0; w < NW; w++)
      if (n0 + 32 * w < a.N)      // (wave-uniform)
#pragma unroll
        for (int r = 0; r < 16; r++) {
          const bool in = n0 + 32 * w + 8 * (r >> 2) + 4 * half < a.N;
#pragma unroll
          for (int it = 0; it < 2; it++) acc[it] = __builtin_amdgcn_mfma_f32_32x32x2f32(C[w][it][r >> 2][r & 3] * (in ? ei[it] : 0.f), S[w][r], acc[it], 0, 0, 0);
        }
    if (more) fetch_C(b + 1);
    __builtin_amdgcn_sched_barrier(0);
    // the block's own tokens: this wave's sixteen keys
    int ahead = l31 - 16 * wv - 8 * half;      // key k of this lane lies ahead of row 32 it + l31 when k > ahead + 32 it
    asm volatile("" : "+v"(ahead));            // (not hoisted into sixteen lane masks)
#pragma unroll
    for (int k = 0; k < 8; k++) {
      const int j = 16 * wv + 8 * half + k;
      const double csj = s_cs[buf][j];
      const float xj = s_x[buf][j][l31] * s_dt[buf][j];
#pragma unroll
      for (int it = 0; it < 2; it++) {
        // (for two of the waves all keys lie ahead of the first 32 rows: they multiply zeros while the others, whom they would wait for, do not)
        const float mij = k <= ahead + 32 * it ? G[it][k >> 2][k & 3] * __builtin_amdgcn_exp2f((float)(csi[it] - csj)) : 0.f;
        acc[it] = __builtin_amdgcn_mfma_f32_32x32x2f32(mij, xj, acc[it], 0, 0, 0);
      }
    }
    if (more) fetch_G(b + 1);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int it = 0; it < 2; it++)
#pragma unroll
      for (int r = 0; r < 16; r++) s_part[wv][32 * it + (r & 3) + 8 * (r >> 2) + 4 * half][l31] = acc[it][r];
    __builtin_amdgcn_sched_barrier(0);
    // S_out
    const float ge = __builtin_amdgcn_exp2f((float)s_cs[buf][Q - 1]);
#pragma unroll
    for (int w = 0; w < NW; w++)
#pragma unroll
      for (int r = 0; r < 16; r++) S[w][r] *= ge;
    if (n0 < a.N)
#pragma unroll
      for (int kk = 0; kk < 32; kk++) {
        const int j = kk + 32 * half;
        const float xs = s_x[buf][j][l31] * s_end[buf][j];
#pragma unroll
        for (int w = 0; w < NW; w++) S[w] = __builtin_amdgcn_mfma_f32_32x32x2f32(B[w][kk], xs, S[w], 0, 0, 0);
      }
    __builtin_amdgcn_sched_barrier(0);
    if (more) stage(b + 1);
    __syncthreads();
#pragma unroll
    for (int u = 0; u < 8; u++) {
      const int t = (tid >> 5) + 8 * u;
      if (t0 + t < cnt && colok)
        a.out[(size_t)(start + t0 + t) * a.ldo + oX + l31] = fmaf(Dh, s_x[buf][t][l31], s_part[0][t][l31] + s_part[1][t][l31] + s_part[2][t][l31] + s_part[3][t][l31]);
    }
  }
#pragma unroll
  for (int w = 0; w < NW; w++)
#pragma unroll
    for (int r = 0; r < 16; r++) {
      const int n = n0 + 32 * w + (r & 3) + 8 * (r >> 2) + 4 * half;
      if (n < a.N && colok) Sg[(size_t)n * a.E + e0 + l31] = S[w][r];
    }
}

}  // namespace tgx
