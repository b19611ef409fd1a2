// stack_ssm.h — row-wise kernels of the layered designs whose norms stand behind the sublayers only and whose mixers are state-space recurrences (Nusovik).
// Same conventions as stack.h / stack_seq.h: a step's T tokens are the concatenated entries of a ragged batch (StepMeta), all arithmetic here is fp32, every
// reduction has a fixed order.
//   post_norm_add_kernel     x += y / sqrt(mean(y^2) + eps) * w: the seam behind every sublayer
//   conv_silu_kernel         causal depth-wise convolution (with bias) + silu over any number of channels, tails per slot; the step sizes and decays of a
//                            scalar-decay recurrence in the same launch
//   selective_scan_kernel    the recurrence of a selective scan: one decay per (channel, state number), read-out, skip and silu gate
//   part_norm_gate_kernel    y * silu(z), RMS norm in equal parts, times a weight
// The scalar-decay recurrence itself is rec_scan_kernel<DPER, REC_SSD> (stack_rec.h) and, for long portions, the chunked form of stack_ssd_mfma.h.
#pragma once
#include "stack.h"

namespace tgx {

// ---- x[t] += y[t] / sqrt(mean(y[t]^2) + eps) * w.  One workgroup per token; widths up to 256 * 4 * POST_REG (in whole vectors of four) stay in registers.
struct PostNormArgs { float* x; const float* y; const float* w; int W; float eps; };
constexpr int POST_REG = 4;
__global__ __launch_bounds__(256) void post_norm_add_kernel(PostNormArgs a) {
  __shared__ float s4[4];
  const size_t t = blockIdx.x;
  float* __restrict__ x = a.x + t * a.W;
  const float* __restrict__ y = a.y + t * a.W;
  const float* __restrict__ w = a.w;
  if ((a.W & 3) == 0 && a.W <= 1024 * POST_REG) {
    f32x4 v[POST_REG], xv[POST_REG], wv[POST_REG];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < POST_REG; k++) {
      const int c = 4 * threadIdx.x + 1024 * k;
      if (c < a.W) { v[k] = *reinterpret_cast<const f32x4*>(y + c); xv[k] = *reinterpret_cast<const f32x4*>(x + c); wv[k] = *reinterpret_cast<const f32x4*>(w + c); }
    }
#pragma unroll
    for (int k = 0; k < POST_REG; k++)
      if (4 * (int)threadIdx.x + 1024 * k < a.W)
#pragma unroll
        for (int u = 0; u < 4; u++) ss = fmaf(v[k][u], v[k][u], ss);
    ss = block_sum_256(ss, s4);
    const float r = 1.0f / sqrtf(ss / (float)a.W + a.eps);
#pragma unroll
    for (int k = 0; k < POST_REG; k++) {
      const int c = 4 * threadIdx.x + 1024 * k;
      if (c >= a.W) continue;
#pragma unroll
      for (int u = 0; u < 4; u++) xv[k][u] = fmaf(v[k][u] * r, wv[k][u], xv[k][u]);
      *reinterpret_cast<f32x4*>(x + c) = xv[k];
    }
    return;
  }
  float ss = 0.f;
  for (int c = threadIdx.x; c < a.W; c += 256) ss = fmaf(y[c], y[c], ss);
  ss = block_sum_256(ss, s4);
  const float r = 1.0f / sqrtf(ss / (float)a.W + a.eps);
  for (int c = threadIdx.x; c < a.W; c += 256) x[c] = fmaf(y[c] * r, w[c], x[c]);
}

// ---- out[t][c] = silu(b[c] + sum_j w[c][j] * raw[t - taps + 1 + j][c]) on the C channels that start at column col0 of the projections' row; the taps - 1 rows
// before come from the step's own rows, the slot's tails (raw rows, double-buffered by step parity like the other per-slot rows) or are zero before the
// sequence's start.  A thread owns one channel of `tile` consecutive tokens; with TAPS > 0 the rows it still needs ride in registers from token to token.
// heads > 0: one more workgroup column turns the projections' step-size columns into out[t][C + h] = dt = softplus(raw + dt_bias[h]), out[t][C + heads + h] =
// exp(-exp(a_log[h]) dt) and out[t][C + 2 heads + h] = -exp(a_log[h]) dt.   Grid: (tokens / tile, C / 256 (+ 1)).
struct ConvSiluArgs {
  const float* proj; long long ldp; int col0;
  const float* cw;       // [C][taps], last column: the current token's
  const float* cb;       // [C]
  float* out; long long ldo;
  float* state;          // [2][slots][taps - 1][C] (nullptr when taps == 1)
  size_t state_buf;
  int C, taps, tile;
  int heads, dt_col;     // heads 0: no step sizes
  const float *dt_bias, *a_log;
};
__device__ __forceinline__ float silu_f(float v) { return v / (1.0f + expf(-v)); }
__device__ __forceinline__ float softplus_f(float v) { return v > 20.f ? v : log1pf(expf(v)); }
template <int TAPS>      // 0: any number
__global__ __launch_bounds__(256) void conv_silu_kernel(StepMeta m, ConvSiluArgs a) {
  const int t0 = blockIdx.x * a.tile, t1 = min(m.T, t0 + a.tile), taps = TAPS ? TAPS : a.taps, nb = taps - 1;
  if (a.heads > 0 && blockIdx.y == gridDim.y - 1) {
    for (int i = threadIdx.x; i < (t1 - t0) * a.heads; i += 256) {
      const int t = t0 + i / a.heads, h = i % a.heads;
      const float dt = softplus_f(a.proj[(size_t)t * a.ldp + a.dt_col + h] + a.dt_bias[h]), la = -expf(a.a_log[h]) * dt;
      float* o = a.out + (size_t)t * a.ldo + a.C;
      o[h] = dt; o[a.heads + h] = expf(la); o[2 * a.heads + h] = la;
    }
    return;
  }
  const int c = blockIdx.y * 256 + threadIdx.x;
  if (c >= a.C) return;
  const float* __restrict__ raw = a.proj + a.col0 + c;
  const float* __restrict__ old_all = a.state;
  float* __restrict__ new_all = a.state;
  float* __restrict__ out = a.out + c;
  const float* __restrict__ cw = a.cw + (size_t)c * taps;
  const float b = a.cb[c];
  constexpr int NH = TAPS > 1 ? TAPS - 1 : 1;
  float w[TAPS ? TAPS : 1], hist[NH];      // hist[d - 1]: the row d back
  if constexpr (TAPS > 0) {
#pragma unroll
    for (int j = 0; j < TAPS; j++) w[j] = cw[j];
  }
  for (int t = t0; t < t1; t++) {
    const int i = m.tok_idx[t], cnt = m.tok_cnt[t], pos = m.tok_pos[t], par = m.tok_par[t];
    const size_t srow = (size_t)m.tok_row[t] * nb * a.C + c;
    const float* st_old = a.state ? old_all + (size_t)par * a.state_buf + srow : nullptr;
    float* st_new = a.state ? new_all + (size_t)(par ^ 1) * a.state_buf + srow : nullptr;
    auto back = [&](int d) -> float {      // the raw row d positions back
      if (d <= i) return raw[(size_t)(t - d) * a.ldp];
      return pos - d >= 0 ? st_old[(size_t)(nb - (d - i)) * a.C] : 0.f;      // tail slot s holds position past - nb + s, past = pos - i
    };
    const float x0 = raw[(size_t)t * a.ldp];
    float acc = b;
    if constexpr (TAPS > 0) {
      if (t == t0 || i == 0) {
#pragma unroll
        for (int d = 1; d < TAPS; d++) hist[d - 1] = back(d);
      }
      acc = fmaf(w[TAPS - 1], x0, acc);
#pragma unroll
      for (int d = 1; d < TAPS; d++) acc = fmaf(w[TAPS - 1 - d], hist[d - 1], acc);
#pragma unroll
      for (int d = TAPS - 1; d > 1; d--) hist[d - 1] = hist[d - 2];
      if (TAPS > 1) hist[0] = x0;
    } else {
      acc = fmaf(cw[nb], x0, acc);
      for (int d = 1; d <= nb; d++) acc = fmaf(cw[nb - d], back(d), acc);
    }
    out[(size_t)t * a.ldo] = silu_f(acc);
    if (st_new) {
      const int s = nb - (cnt - i);                        // row i of cnt lands in tail slot nb - (cnt - i) ...
      if (s >= 0) st_new[(size_t)s * a.C] = x0;
      if (i == 0)                                          // ... and an entry shorter than the tails keeps the end of the old ones
        for (int k = 0; k + cnt < nb; k++) st_new[(size_t)k * a.C] = (pos - (nb - cnt - k) >= 0) ? st_old[(size_t)(k + cnt) * a.C] : 0.f;
    }
  }
}

// ---- selective scan.  Per channel c and state number n:  S[c][n] <- 2^(dt_c A2[c][n]) S[c][n] + dt_c x_c B[n];  y_c = sum_n S[c][n] C[n] + D_c x_c;
// out = y * silu(z).  A2 = -exp(A_log) * log2(e).  One workgroup per (entry, 256 / LPC channels): LPC adjacent lanes share a channel, each keeps SPL of its
// state numbers in registers (SPL LPC >= N).  The tokens are taken in order, a block of TB at a time: (dt, dt x) and (x, z) of the workgroup's channels and (B, C)
// of the block are staged in LDS while the next block's loads are in flight.  Inside a block LPC tokens are advanced without any lane exchange, then their LPC
// partial read-outs are summed over the channel's lanes by halving (each step hands half of the tokens to the partner), which leaves token l with lane l:
// skip, gate and store happen once per token.  Blocks past the end are advanced by dt = 0, which leaves the state as it is.
struct SelScanArgs {
  const float* dt; long long ldt;
  const float* x; long long ldx;
  const float* z; long long ldz;
  const float* bc; long long ldbc; int ccol;      // per token: B [N] at bc, C [N] at bc + ccol
  const float* A2;       // [C][N]
  const float* D;        // [C]
  float* S;              // [slots][C][N]
  float* out; long long ldo;
  int C, N;
};
template <int SPL, int LPC>
__global__ __launch_bounds__(256) void selective_scan_kernel(StepMeta m, SelScanArgs a) {
  constexpr int CPW = 256 / LPC, NP = SPL * LPC, TB = NP <= 32 ? 64 : NP <= 64 ? 32 : 16, NX = (TB * CPW + 255) / 256, NB = TB * NP / 256 > 0 ? (TB * NP + 255) / 256 : 1;
  typedef float f2 __attribute__((ext_vector_type(2)));
  __shared__ __attribute__((aligned(16))) f2 s_bc[TB][NP];
  __shared__ f2 s_dx[TB][CPW], s_xz[TB][CPW + 1];
  // neighbouring channel tiles share 128-byte lines: they are dealt to the same XCD (workgroup index modulo 8)
  const int nt = gridDim.x, tile = (nt & 7) == 0 ? (blockIdx.x & 7) * (nt >> 3) + (blockIdx.x >> 3) : blockIdx.x;
  const int e = blockIdx.y, tid = threadIdx.x, l = tid % LPC, cl = tid / LPC, c0 = tile * CPW, c = c0 + cl;
  const int start = m.ent_start[e], cnt = m.ent_count[e], row = m.ent_row[e];
  const bool fresh = m.tok_pos[start] == 0, on = c < a.C;
  float* Sg = a.S + ((size_t)row * a.C + (on ? c : 0)) * a.N;
  float S[SPL], A2[SPL];
#pragma unroll
  for (int k = 0; k < SPL; k++) {
    const int n = l * SPL + k;
    S[k] = (!fresh && on && n < a.N) ? Sg[n] : 0.f;
    A2[k] = (on && n < a.N) ? a.A2[(size_t)c * a.N + n] : 0.f;
  }
  const float Dc = on ? a.D[c] : 0.f;
  float rdt[NX], rx[NX], rz[NX], rb[NB], rc[NB];
  auto fetch = [&](int t0) {
    const int nb = min(TB, cnt - t0);
#pragma unroll
    for (int u = 0; u < NX; u++) {
      const int i = tid + 256 * u, t = i / CPW, cc = c0 + i % CPW;
      const bool in = t < nb && cc < a.C;
      const size_t tok = (size_t)(start + t0 + (in ? t : 0));
      const int ca = in ? cc : c0;
      rdt[u] = in ? a.dt[tok * a.ldt + ca] : 0.f; rx[u] = in ? a.x[tok * a.ldx + ca] : 0.f; rz[u] = in ? a.z[tok * a.ldz + ca] : 0.f;
    }
#pragma unroll
    for (int u = 0; u < NB; u++) {
      const int i = tid + 256 * u, t = i / NP, n = i % NP;
      const bool in = t < nb && n < a.N;
      const float* p = a.bc + (size_t)(start + t0 + (in ? t : 0)) * a.ldbc;
      rb[u] = in ? p[n] : 0.f; rc[u] = in ? p[a.ccol + n] : 0.f;
    }
  };
  fetch(0);
  for (int t0 = 0; t0 < cnt; t0 += TB) {
    const int nb = min(TB, cnt - t0);
    if (t0 > 0) {      // the block before leaves: its outputs stand in s_xz[..][..].y
      __syncthreads();
#pragma unroll
      for (int u = 0; u < NX; u++) {
        const int i = tid + 256 * u, t = i / CPW, cc = i % CPW;
        if (t < TB && c0 + cc < a.C) a.out[(size_t)(start + t0 - TB + t) * a.ldo + c0 + cc] = s_xz[t][cc].y;
      }
      __syncthreads();
    }
#pragma unroll
    for (int u = 0; u < NX; u++) {
      const int i = tid + 256 * u, t = i / CPW, cc = i % CPW;
      if (t < TB) { s_dx[t][cc] = f2{rdt[u], rdt[u] * rx[u]}; s_xz[t][cc] = f2{rx[u], rz[u]}; }
    }
#pragma unroll
    for (int u = 0; u < NB; u++) { const int i = tid + 256 * u; if (i < TB * NP) s_bc[i / NP][i % NP] = f2{rb[u], rc[u]}; }
    __syncthreads();
    if (t0 + TB < cnt) fetch(t0 + TB);
    auto advance = [&](int t) -> float {
      const f2 d = s_dx[t][cl];
      float acc = 0.f;
#pragma unroll
      for (int k = 0; k < SPL; k++) {
        const f2 bc = s_bc[t][l * SPL + k];
        S[k] = fmaf(__builtin_amdgcn_exp2f(d.x * A2[k]), S[k], d.y * bc.x);
        acc = fmaf(S[k], bc.y, acc);
      }
      return acc;
    };
    auto finish = [&](int t, float y) {
      const f2 xz = s_xz[t][cl];
      s_xz[t][cl].y = fmaf(Dc, xz.x, y) * silu_f(xz.y);
    };
    for (int g = 0; g < nb; g += LPC) {
      if (nb - g == 1) {      // one token left (a decode step): every lane gets the sum, the first one finishes
        const float y = row_group_sum<LPC>(advance(g));
        if (l == 0) finish(g, y);
        break;
      }
      float p[LPC];
#pragma unroll
      for (int j = 0; j < LPC; j++) p[j] = advance(g + j);
      // halving: the partner lane (row mirror, half-row mirror, quad swaps) differs in the bit that says which half of the tokens this lane keeps
      if constexpr (LPC == 16) {
        const bool hi = l & 8;
#pragma unroll
        for (int j = 0; j < 8; j++) { const float keep = hi ? p[j + 8] : p[j], give = hi ? p[j] : p[j + 8]; p[j] = keep + dpp_mov<0x140, 0xf>(give); }
      }
      {
        const bool hi = l & 4;
#pragma unroll
        for (int j = 0; j < 4; j++) { const float keep = hi ? p[j + 4] : p[j], give = hi ? p[j] : p[j + 4]; p[j] = keep + dpp_mov<0x141, 0xf>(give); }
      }
      {
        const bool hi = l & 2;
#pragma unroll
        for (int j = 0; j < 2; j++) { const float keep = hi ? p[j + 2] : p[j], give = hi ? p[j] : p[j + 2]; p[j] = keep + dpp_mov<0x4E, 0xf>(give); }
      }
      const float keep = (l & 1) ? p[1] : p[0], give = (l & 1) ? p[0] : p[1];
      finish(g + l, keep + dpp_mov<0xB1, 0xf>(give));
    }
  }
  __syncthreads();
  const int tl = (cnt - 1) / TB * TB;
#pragma unroll
  for (int u = 0; u < NX; u++) {
    const int i = tid + 256 * u, t = i / CPW, cc = i % CPW;
    if (t < cnt - tl && c0 + cc < a.C) a.out[(size_t)(start + tl + t) * a.ldo + c0 + cc] = s_xz[t][cc].y;
  }
#pragma unroll
  for (int k = 0; k < SPL; k++) { const int n = l * SPL + k; if (on && n < a.N) Sg[n] = S[k]; }
}

// ---- u = y * silu(z) in `parts` equal parts of n channels; out = u / sqrt(mean over the part of u^2 + eps) * w * scale.  Grid: (tokens, parts).
struct PartNormArgs { const float* y; long long ldy; const float* z; long long ldz; const float* w; float* out; long long ldo; int n; float eps, scale; };
constexpr int PART_REG = 8;      // parts up to 256 * PART_REG channels stay in registers
__global__ __launch_bounds__(256) void part_norm_gate_kernel(PartNormArgs a) {
  __shared__ float s4[4];
  const size_t t = blockIdx.x;
  const int c0 = blockIdx.y * a.n;
  const float* __restrict__ y = a.y + t * a.ldy + c0;
  const float* __restrict__ z = a.z + t * a.ldz + c0;
  const float* __restrict__ w = a.w + c0;
  float* __restrict__ out = a.out + t * a.ldo + c0;
  float ss = 0.f;
  if (a.n <= 256 * PART_REG) {
    float u[PART_REG], g[PART_REG], wk[PART_REG];      // all loads first
#pragma unroll
    for (int k = 0; k < PART_REG; k++) {
      const int c = threadIdx.x + 256 * k;
      u[k] = c < a.n ? y[c] : 0.f; g[k] = c < a.n ? z[c] : 0.f; wk[k] = c < a.n ? w[c] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < PART_REG; k++) { u[k] *= silu_f(g[k]); ss = fmaf(u[k], u[k], ss); }
    ss = block_sum_256(ss, s4);
    const float r = a.scale / sqrtf(ss / (float)a.n + a.eps);
#pragma unroll
    for (int k = 0; k < PART_REG; k++) { const int c = threadIdx.x + 256 * k; if (c < a.n) out[c] = u[k] * r * wk[k]; }
    return;
  }
  for (int c = threadIdx.x; c < a.n; c += 256) { const float u = y[c] * silu_f(z[c]); ss = fmaf(u, u, ss); }
  ss = block_sum_256(ss, s4);
  const float r = a.scale / sqrtf(ss / (float)a.n + a.eps);
  for (int c = threadIdx.x; c < a.n; c += 256) out[c] = y[c] * silu_f(z[c]) * r * w[c];
}

}  // namespace tgx
