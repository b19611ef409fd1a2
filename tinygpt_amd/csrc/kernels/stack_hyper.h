// stack_hyper.h — row-wise kernels of the layered designs whose residual is several streams joined by learned mixes (hyper-connections), whose embedding adds a row per
// pair of neighbouring tokens, and whose attention subtracts one score map from another (Keronex).  Same conventions as stack.h: a step's T tokens are the concatenated
// entries of a ragged batch (StepMeta), all arithmetic here is fp32, every reduction has a fixed order.
//   pair_embed_kernel       embedding row * scale + the row of the pair (token before, token), into every stream; the first sublayer's normed input; the slot's last token
//   hyper_seam_kernel       the seam between two sublayers: the streams take the sublayer's output and each other's shares, the next sublayer's normed input leaves
//   map_difference_kernel   o_1 - lambda o_2 of a head's two maps, RMS norm over the head, constant factor
//   map_difference_merge_kernel   the same on the records of an attention whose keys were divided between workgroups
#pragma once
#include "stack_seq.h"

namespace tgx {

constexpr int HYPER_MAX_STREAMS = 16;
constexpr int PAIR_REG = 16;      // channels a thread of the embedding kernel keeps
constexpr int HYPER_REG = 4;      // vectors of four channels a thread keeps between the passes: widths up to 4096

// u_t = sum_s w_in[s] x_s, out_t = u_t / sqrt(mean(u_t^2) + eps) * (1 + w_norm)
struct HyperIn { const float *w_in, *w_norm; float* out; float eps; };

// ---- x_s[t] = embed[id] * scale (+ pair[row]) for all n streams.  row = (id_before * mul_before + id * mul) mod buckets, and `buckets` itself for a sequence's first
// token.  The token before is the entry's own, or the slot's last one (double-buffered with the slot's step parity like the other per-slot rows).  One workgroup per token.
struct PairEmbedArgs {
  const void* embed; const void* pair;      // pair nullptr: no pair rows
  int* last;                                // [2][slots]
  int slots, buckets;
  long long mul_before, mul;
  float scale;
  float* xs;                                // [T][n][W]
  int n, W;
  HyperIn in;
};
template <int DT>
__global__ __launch_bounds__(256) void pair_embed_kernel(StepMeta m, PairEmbedArgs a) {
  __shared__ float s4[4];
  const int t = blockIdx.x, i = m.tok_idx[t], row = m.tok_row[t], par = m.tok_par[t], id = m.tok_id[t];
  const elem_t<DT>* er = reinterpret_cast<const elem_t<DT>*>(a.embed) + (size_t)id * a.W;
  const elem_t<DT>* pr = nullptr;
  if (a.pair) {
    const int before = i > 0 ? m.tok_id[t - 1] : a.last[(size_t)par * a.slots + row];
    const long long b = m.tok_pos[t] == 0 ? a.buckets : ((long long)before * a.mul_before + (long long)id * a.mul) % a.buckets;
    pr = reinterpret_cast<const elem_t<DT>*>(a.pair) + (size_t)b * a.W;
    if (i == m.tok_cnt[t] - 1 && threadIdx.x == 0) a.last[(size_t)(par ^ 1) * a.slots + row] = id;
  }
  float* __restrict__ x = a.xs + (size_t)t * a.n * a.W;
  float* __restrict__ out = a.in.out + (size_t)t * a.W;
  float sum = 0.f, ss = 0.f, v[PAIR_REG];
  for (int s = 0; s < a.n; s++) sum += a.in.w_in[s];
  auto value = [&](int c) -> float { return fmaf(elem_to_f32<DT>(er[c]), a.scale, pr ? elem_to_f32<DT>(pr[c]) : 0.f); };
#pragma unroll
  for (int k = 0; k < PAIR_REG; k++) { const int c = threadIdx.x + 256 * k; v[k] = c < a.W ? value(c) : 0.f; }
#pragma unroll
  for (int k = 0; k < PAIR_REG; k++) ss = fmaf(sum * v[k], sum * v[k], ss);
  for (int c = threadIdx.x + 256 * PAIR_REG; c < a.W; c += 256) { const float u = sum * value(c); ss = fmaf(u, u, ss); }      // (channels beyond the registers are read again below)
  ss = block_sum_256(ss, s4);
  const float r = sum / sqrtf(ss / (float)a.W + a.in.eps);
  auto store = [&](int c, float val) {
    for (int s = 0; s < a.n; s++) x[(size_t)s * a.W + c] = val;
    out[c] = val * r * (1.0f + a.in.w_norm[c]);
  };
#pragma unroll
  for (int k = 0; k < PAIR_REG; k++) { const int c = threadIdx.x + 256 * k; if (c < a.W) store(c, v[k]); }
  for (int c = threadIdx.x + 256 * PAIR_REG; c < a.W; c += 256) store(c, value(c));
}

// ---- the seam.  y_t = the sublayer's output: one row, or the sum of the token's `top` expert rows, plus the shared expert's row.  All streams at once from the old
// ones: x_k <- sum_s mix[s][k] x_s + w_out[k] y; then the next sublayer's input (HyperIn).  Behind the last sublayer (in.w_in nullptr) the streams end: only their sum
// leaves, in in.out.  One workgroup per token; a thread keeps its channels, so only the norm's sum crosses threads.  NS >= n.
struct HyperSeamArgs {
  float* xs;                 // [T][n][W]
  const float* y; int top;   // [T * top][W]
  const float* ysh;          // [T][W] (nullptr: none)
  const float *mix, *w_out;  // [n][n] (from, to), [n]
  int n, W;
  HyperIn in;
};
template <int NS>
__global__ __launch_bounds__(256) void hyper_seam_kernel(HyperSeamArgs a) {
  __shared__ float s4[4];
  const size_t t = blockIdx.x;
  float* __restrict__ xs = a.xs + t * a.n * a.W;
  const float* __restrict__ y = a.y + t * a.top * a.W;
  const float* __restrict__ ysh = a.ysh ? a.ysh + t * a.W : nullptr;
  float* __restrict__ out = a.in.out + t * a.W;
  const bool end = !a.in.w_in;
  float mix[NS][NS], wo[NS], wi[NS];
#pragma unroll
  for (int s = 0; s < NS; s++) {
    wo[s] = s < a.n ? a.w_out[s] : 0.f;
    wi[s] = s < a.n ? (end ? 1.f : a.in.w_in[s]) : 0.f;
#pragma unroll
    for (int k = 0; k < NS; k++) mix[s][k] = s < a.n && k < a.n ? a.mix[s * a.n + k] : 0.f;
  }
  if ((a.W & 3) == 0 && a.W <= 1024 * HYPER_REG) {
    f32x4 u[HYPER_REG];
    float ss = 0.f;
    auto quad = [&](int k) {
      const int c = 4 * threadIdx.x + 1024 * k;
      if (c >= a.W) return;
      f32x4 v[NS], yv = *reinterpret_cast<const f32x4*>(y + c);
#pragma unroll
      for (int s = 0; s < NS; s++) v[s] = s < a.n ? *reinterpret_cast<const f32x4*>(xs + (size_t)s * a.W + c) : f32x4{0.f, 0.f, 0.f, 0.f};
      for (int e = 1; e < a.top; e++) { const f32x4 z = *reinterpret_cast<const f32x4*>(y + (size_t)e * a.W + c); for (int i = 0; i < 4; i++) yv[i] += z[i]; }
      if (ysh) { const f32x4 z = *reinterpret_cast<const f32x4*>(ysh + c); for (int i = 0; i < 4; i++) yv[i] += z[i]; }
      f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int d = 0; d < NS; d++) {
        f32x4 o;
#pragma unroll
        for (int i = 0; i < 4; i++) {
          float x = wo[d] * yv[i];
#pragma unroll
          for (int s = 0; s < NS; s++) x = fmaf(mix[s][d], v[s][i], x);
          o[i] = x;
          acc[i] = fmaf(wi[d], x, acc[i]);
        }
        if (!end && d < a.n) *reinterpret_cast<f32x4*>(xs + (size_t)d * a.W + c) = o;
      }
      u[k] = acc;
#pragma unroll
      for (int i = 0; i < 4; i++) ss = fmaf(acc[i], acc[i], ss);
    };
#pragma unroll
    for (int k = 0; k < HYPER_REG; k++) quad(k);
    if (end) {
#pragma unroll
      for (int k = 0; k < HYPER_REG; k++) { const int c = 4 * threadIdx.x + 1024 * k; if (c < a.W) *reinterpret_cast<f32x4*>(out + c) = u[k]; }
      return;
    }
    ss = block_sum_256(ss, s4);
    const float r = 1.0f / sqrtf(ss / (float)a.W + a.in.eps);
#pragma unroll
    for (int k = 0; k < HYPER_REG; k++) {
      const int c = 4 * threadIdx.x + 1024 * k;
      if (c >= a.W) continue;
      const f32x4 w = *reinterpret_cast<const f32x4*>(a.in.w_norm + c);
      f32x4 o;
#pragma unroll
      for (int i = 0; i < 4; i++) o[i] = u[k][i] * r * (1.0f + w[i]);
      *reinterpret_cast<f32x4*>(out + c) = o;
    }
    return;
  }
  float ss = 0.f;
  for (int c = threadIdx.x; c < a.W; c += 256) {
    float v[NS], yv = y[c], acc = 0.f;
#pragma unroll
    for (int s = 0; s < NS; s++) v[s] = s < a.n ? xs[(size_t)s * a.W + c] : 0.f;
    for (int e = 1; e < a.top; e++) yv += y[(size_t)e * a.W + c];
    if (ysh) yv += ysh[c];
#pragma unroll
    for (int d = 0; d < NS; d++) {
      float x = wo[d] * yv;
#pragma unroll
      for (int s = 0; s < NS; s++) x = fmaf(mix[s][d], v[s], x);
      if (!end && d < a.n) xs[(size_t)d * a.W + c] = x;
      acc = fmaf(wi[d], x, acc);
    }
    out[c] = acc;
    ss = fmaf(acc, acc, ss);
  }
  if (end) return;
  ss = block_sum_256(ss, s4);
  const float r = 1.0f / sqrtf(ss / (float)a.W + a.in.eps);
  for (int c = threadIdx.x; c < a.W; c += 256) out[c] *= r * (1.0f + a.in.w_norm[c]);
}

// ---- out[t][h] = d / sqrt(mean(d^2) + eps) * scale, d = o_1 - lambda o_2 of the head's two maps.  One wave per (token, head); vdim <= 64 GQA_MAX_RPL.
struct MapDifferenceArgs { const float* maps; float* out; int pairs, vdim; float lambda, eps, scale; };      // maps [T][heads][2][vdim], out [T][heads][vdim], pairs = T heads
__global__ __launch_bounds__(256) void map_difference_kernel(MapDifferenceArgs a) {
  const int p = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (p >= a.pairs) return;
  const float* r = a.maps + (size_t)p * 2 * a.vdim;
  float d[GQA_MAX_RPL], ss = 0.f;
#pragma unroll
  for (int k = 0; k < GQA_MAX_RPL; k++) {
    const int c = lane + 64 * k;
    d[k] = c < a.vdim ? fmaf(-a.lambda, r[a.vdim + c], r[c]) : 0.f;
  }
#pragma unroll
  for (int k = 0; k < GQA_MAX_RPL; k++) ss = fmaf(d[k], d[k], ss);
  const float f = a.scale / sqrtf(wave_sum(ss) / (float)a.vdim + a.eps);
#pragma unroll
  for (int k = 0; k < GQA_MAX_RPL; k++) { const int c = lane + 64 * k; if (c < a.vdim) a.out[(size_t)p * a.vdim + c] = d[k] * f; }
}

// ---- the same behind a divided attention: the split records (m, l, acc[vdim]) of both maps of one (token, head) are merged in split order first
struct MapDifferenceMergeArgs { const float* part; int nsplit; float* out; int heads, vdim; float lambda, eps, scale; };      // part [T][heads][2][nsplit][vdim + 2]
__global__ __launch_bounds__(256) void map_difference_merge_kernel(MapDifferenceMergeArgs a) {
  __shared__ float s_f[2][64], s_inv[2], s4[4];
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
  const size_t rs = (size_t)(a.vdim + 2);
  const float* rec = a.part + ((size_t)t * a.heads + h) * 2 * a.nsplit * rs;
  if (wv < 2) {      // a wave per map, a lane per record
    const float* r = rec + (size_t)wv * a.nsplit * rs;
    const float ms = lane < a.nsplit ? r[(size_t)lane * rs] : -INFINITY;
    const float M = group_max<64>(ms), f = ms == -INFINITY ? 0.f : expf(ms - M);
    const float L = group_sum<64>(lane < a.nsplit ? r[(size_t)lane * rs + 1] * f : 0.f);
    s_f[wv][lane] = f;
    if (lane == 0) s_inv[wv] = L > 0.f ? 1.0f / L : 0.f;
  }
  __syncthreads();
  const int c = threadIdx.x;      // vdim <= 256
  float d = 0.f;
  if (c < a.vdim) {
    float o[2] = {0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 2; i++)
      for (int s = 0; s < a.nsplit; s++) o[i] = fmaf(rec[((size_t)i * a.nsplit + s) * rs + 2 + c], s_f[i][s], o[i]);
    d = fmaf(-a.lambda, o[1] * s_inv[1], o[0] * s_inv[0]);
  }
  const float f = a.scale / sqrtf(block_sum_256(d * d, s4) / (float)a.vdim + a.eps);
  if (c < a.vdim) a.out[((size_t)t * a.heads + h) * a.vdim + c] = d * f;
}

}  // namespace tgx
