// hyb_latent.hip -- matrix-core kernels of latent attention in bf16 serving (keys and values that expand from one cached row per token, hyb_kernels.hip has the general forms):
//
//   prompt   attention over keys and transposed values that were expanded for the step, sliding window, learned sink, elementwise gate
//   decode   single rows against the cached rows themselves, 16 query heads per workgroup sharing every row, the keys dealt to several workgroups
//   merge    the decode workgroups' sums joined, expanded to value size (the per-head product) and gated in one launch
//
// Scores, maxima, exponentials, weights and all sums are f32: a score is an f32 sum of exact bf16 products; a weight enters its product as THREE bf16 terms that add up to the f32
// number (8 + 8 + 8 significant bits, cut, not rounded), so the weighted sum too is an f32 sum of exact products.  Exponentials are taken in base two: scale and sink come
// multiplied by log2(e).
#include "hyb_mfma.cuh"
#include <float.h>

namespace mrs {
namespace hybc {

static thread_local char g_err[256];
static int fail(const char *m) { snprintf(g_err, sizeof g_err, "%s", m); return 1; }
static int ok_or(const char *what) {
  if (hipGetLastError() == hipSuccess) return 0;
  snprintf(g_err, sizeof g_err, "%s: launch failed", what);
  return 1;
}
using namespace mrs::mfma;
__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + expf(-v)); }

// ---------------------------------------------------------------------------------- prompt
struct FlashArgs {
  const uint16_t *q;     // [rows, H * DK]
  const uint16_t *k;     // [n_rows, H * DK]  the contexts' keys; an entry's positions lie in consecutive rows from its first gathered block on
  const uint16_t *vt;    // [H * Dv, n_rows]  the contexts' values, transposed
  const int *tables;     // [entries, max_blocks]: gathered block of every block of an entry
  const int *tok_pos;
  const int *seg_entry, *seg_row0, *seg_len;  // segments of at most 64 rows
  const float *sink;     // [H], nullable
  const float *gate;     // [rows, ldg], nullable
  uint16_t *out;         // [rows, H * Dv]
  int H, DK, Dv, n_rows, max_blocks, block_size, window, ldg, segments;
  float scale2;          // scale * log2(e)
};
// One workgroup of four waves per (segment of 64 queries, head): wave = (query half, key half).  Keys and values pass through LDS 64 at a time, the next tile's values in registers
// meanwhile.  S^T = K Q^T leaves a lane with ONE query (its column) and sixteen keys, so the softmax needs one exchange between the wave's halves for the maximum, and the weights
// are already the operand of O^T = V^T P^T: the order of the keys inside a product is free, and the V^T fragments are read in the order the lane holds its weights.  The two key
// halves of a query are joined at the end.
template <int NK, int NV> __global__ void __launch_bounds__(256, 2) latent_flash_kernel(FlashArgs a) {
  constexpr int KS = NK * 16 + 8, VS = 64 + 4, KU = (NK + 1) / 2, VU = NV;   // LDS row strides; 16-byte pieces per thread of a tile
  constexpr int TILE = 64 * KS + NV * 32 * VS, JOIN = 2 * 64 * (NV * 16 + 2) * 2;   // (in 16-bit values)
  __shared__ __attribute__((aligned(16))) uint16_t lds[TILE > JOIN ? TILE : JOIN];
  uint16_t *Ks = lds, *Vs = lds + 64 * KS;
  // workgroups go round robin to the eight dies: every die takes consecutive (head, segment) pairs, so that a head's keys are read through one L2; the longest rows first
  const int n = a.segments * a.H, chunk = gridDim.x >> 3, item = (blockIdx.x & 7) * chunk + (blockIdx.x >> 3);
  if (item >= n) return;
  const int h = item / a.segments, z = a.segments - 1 - item % a.segments;
  const int r0 = a.seg_row0[z], len = a.seg_len[z];
  if (len <= 0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, ql = lane & 31, kh = lane >> 5, qg = wave & 1, kg = wave >> 1;
  const int pos0 = a.tok_pos[r0], hi = pos0 + len - 1;
  const int lo = a.window > 0 && pos0 - a.window + 1 > 0 ? pos0 - a.window + 1 : 0;
  const int b0 = lo / a.block_size;
  const int base = (a.tables[(size_t)a.seg_entry[z] * a.max_blocks + b0] - b0) * a.block_size;   // gathered row of position 0 (only positions >= lo are read)
  const int qi = qg * 32 + ql, t = r0 + (qi < len ? qi : len - 1), pq = pos0 + qi;
  const bool qv = qi < len;
  bf16x8 qf[NK];
#pragma unroll
  for (int ks = 0; ks < NK; ++ks) {
    int4 v = make_int4(0, 0, 0, 0);
    if (ks * 16 + 8 * kh < a.DK) v = *(const int4 *)(a.q + ((size_t)t * a.H + h) * a.DK + ks * 16 + 8 * kh);
    qf[ks] = __builtin_bit_cast(bf16x8, v);
  }
  int4 kr[KU], vr[VU];
  auto fetch = [&](int kt) {
#pragma unroll
    for (int m = 0; m < KU; ++m) {
      const int u = tid + m * 256, row = u / (NK * 2), c = (u - row * (NK * 2)) * 8, g = base + kt + row;
      int4 v = make_int4(0, 0, 0, 0);
      if (row < 64 && c < a.DK && g >= 0 && g < a.n_rows) v = *(const int4 *)(a.k + ((size_t)g * a.H + h) * a.DK + c);
      kr[m] = v;
    }
#pragma unroll
    for (int m = 0; m < VU; ++m) {
      const int u = tid + m * 256, dv = u >> 3, key = kt + (u & 7) * 8, g = base + key;
      int4 v = make_int4(0, 0, 0, 0);
      if (dv < a.Dv && key + 7 >= lo && key <= hi && g >= 0 && g + 8 <= a.n_rows) {
        v = *(const int4 *)(a.vt + (size_t)(h * a.Dv + dv) * a.n_rows + g);
        if (key < lo || key + 7 > hi) {  // (a weight of zero must not meet whatever a page holds past the tokens)
          unsigned w[4] = {(unsigned)v.x, (unsigned)v.y, (unsigned)v.z, (unsigned)v.w};
#pragma unroll
          for (int j = 0; j < 8; ++j)
            if (key + j < lo || key + j > hi) w[j >> 1] &= (j & 1) ? 0x0000ffffu : 0xffff0000u;
          v = make_int4((int)w[0], (int)w[1], (int)w[2], (int)w[3]);
        }
      }
      vr[m] = v;
    }
  };
  auto put = [&]() {
#pragma unroll
    for (int m = 0; m < KU; ++m) {
      const int u = tid + m * 256, row = u / (NK * 2), c = (u - row * (NK * 2)) * 8;
      if (row < 64) *(int4 *)(Ks + row * KS + c) = kr[m];
    }
#pragma unroll
    for (int m = 0; m < VU; ++m) {
      const int u = tid + m * 256;
      int2 *d = (int2 *)(Vs + (u >> 3) * VS + (u & 7) * 8);
      d[0] = make_int2(vr[m].x, vr[m].y);
      d[1] = make_int2(vr[m].z, vr[m].w);
    }
  };
  f32x16 o[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[i][r] = 0.f;
  const bool sunk = a.sink && kg == 0;
  float m = sunk ? a.sink[h] * LOG2E : -FLT_MAX, l = sunk && kh == 0 ? 1.0f : 0.f;   // (l: this half-wave's part)
  const int w_first = pos0 + qg * 32, w_last = w_first + 31 < hi ? w_first + 31 : hi;            // the wave's queries
  const int w_lo = a.window > 0 ? w_first - a.window + 1 : 0;
  const int kt0 = lo & ~31;
  fetch(kt0);
  for (int kt = kt0; kt <= hi; kt += 64) {
    put();
    __syncthreads();
    if (kt + 64 <= hi) fetch(kt + 64);
    const int kb = kt + 32 * kg;
    if (qg * 32 < len && kb <= w_last && kb + 31 >= w_lo) {
      f32x16 s;
#pragma unroll
      for (int r = 0; r < 16; ++r) s[r] = 0.f;
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) {
        const bf16x8 kf = __builtin_bit_cast(bf16x8, *(const int4 *)(Ks + (32 * kg + ql) * KS + ks * 16 + 8 * kh));
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[ks], s, 0, 0, 0);
      }
      // register r: key kb + (r & 3) + 8 (r >> 2) + 4 kh
      const bool whole = kb + 31 <= w_first && (a.window <= 0 || w_last - kb < a.window) && kb >= 0;
      float p[16], mx = -FLT_MAX;
      if (whole) {
#pragma unroll
        for (int r = 0; r < 16; ++r) { p[r] = s[r] * a.scale2; mx = fmaxf(mx, p[r]); }
      } else {
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = kb + (r & 3) + 8 * (r >> 2) + 4 * kh;
          const bool vis = key <= pq && (a.window <= 0 || pq - key < a.window);
          p[r] = vis ? s[r] * a.scale2 : -FLT_MAX;
          mx = fmaxf(mx, p[r]);
        }
      }
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m, mx), alpha = exp2_f(m - mn);
      float sum = 0.f;
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        p[r] = p[r] > -FLT_MAX ? exp2_f(p[r] - mn) : 0.f;
        sum += p[r];
      }
      l = fmaf(l, alpha, sum);
      m = mn;
      if (__any(alpha != 1.0f)) {
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[i][r] *= alpha;
      }
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        bf16x8 pf[3];
        split3(p + 8 * b, pf);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
          const uint16_t *vp = Vs + (i * 32 + ql) * VS + 32 * kg + 16 * b + 4 * kh;
          const int2 v0 = *(const int2 *)vp, v1 = *(const int2 *)(vp + 8);
          const bf16x8 vf = __builtin_bit_cast(bf16x8, make_int4(v0.x, v0.y, v1.x, v1.y));
#pragma unroll
          for (int c = 0; c < 3; ++c) o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf[c], o[i], 0, 0, 0);
        }
      }
    }
    __syncthreads();
  }
  // join the two key halves of every query: lane by lane (same query, same value rows)
  float *jb = (float *)lds + (size_t)qg * 64 * (NV * 16 + 2);
  l += __shfl_xor(l, 32, 64);
  if (kg == 1) {
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
      for (int r = 0; r < 16; ++r) jb[(i * 16 + r) * 64 + lane] = o[i][r];
    jb[NV * 16 * 64 + lane] = m;
    jb[(NV * 16 + 1) * 64 + lane] = l;
  }
  __syncthreads();
  if (kg == 1 || !qv) return;
  const float m1 = jb[NV * 16 * 64 + lane], l1 = jb[(NV * 16 + 1) * 64 + lane];
  const float M = fmaxf(m, m1), e0 = exp2_f(m - M), e1 = exp2_f(m1 - M), inv = 1.0f / fmaf(l, e0, l1 * e1);
  const float *gr = a.gate ? a.gate + (size_t)t * a.ldg + (size_t)h * a.Dv : nullptr;
  uint16_t *op = a.out + ((size_t)t * a.H + h) * a.Dv;
#pragma unroll
  for (int i = 0; i < NV; ++i)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int dv = i * 32 + 8 * q4 + 4 * kh;
      if (dv >= a.Dv) continue;
      uint16_t w[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int r = 4 * q4 + j;
        float v = fmaf(o[i][r], e0, jb[(i * 16 + r) * 64 + lane] * e1) * inv;
        if (gr) v *= sigmoid_f(gr[dv + j]);
        w[j] = from_f<bf16_t>(v).v;
      }
      *(int2 *)(op + dv) = make_int2((int)(w[0] | ((unsigned)w[1] << 16)), (int)(w[2] | ((unsigned)w[3] << 16)));
    }
}

// ---------------------------------------------------------------------------------- decode
struct LatentDecodeArgs {
  const uint16_t *q;      // [rows, H * E], E = R + rot: queries against cached rows
  const uint16_t *cache;  // [blocks, block_size, E]
  const int *block_tables, *tok_seq, *tok_pos;
  float *part;            // [splits, rows, H, R]: un-normalised weighted sums of the rows' first R values
  float *ml;              // [splits, rows, H, 2]: running maximum (base two), sum
  int rows, H, R, E, block_size, max_blocks, window, splits;
  float scale2;
};
// One workgroup of four waves per (share of the keys, 16 heads, row).  A tile is 32 keys.  Scores S^T [key][head]: wave w takes every fourth run of 32 row values (its fragments come
// straight from the pages: lane (i, g) holds keys 2 i and 2 i + 1, values 8 g .. 8 g + 7 of the run), the waves' partial scores meet in LDS, and every wave repeats the softmax of
// the 16 x 32 tile.  The same fragments leave transposed for LDS, [value][key], two neighbouring keys per write; the weighted sums O^T [value][head] are dealt to the waves
// by 16-value blocks.  The fragments of the next tile are requested before that product.
template <int NF, int NB> __global__ void __launch_bounds__(256) latent_decode_kernel(LatentDecodeArgs a) {
  extern __shared__ __attribute__((aligned(16))) char dl[];
  float4 *Sp = (float4 *)dl;                    // [wave][tile of two][lane]
  uint16_t *Ct = (uint16_t *)(dl + 4 * 2 * 64 * 16);   // [R][40]: 32 keys, padded
  constexpr int CS = 40;
  const int split = blockIdx.x, h0 = blockIdx.y * 16, t = blockIdx.z, tid = threadIdx.x, w = tid >> 6, lane = tid & 63, i = lane & 15, g = lane >> 4;
  const int pos = a.tok_pos[t], lo = a.window > 0 && pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  const int tiles = (pos - lo + 32) >> 5, per = (tiles + a.splits - 1) / a.splits;
  const int k_first = lo + split * per * 32;
  int k_end = k_first + per * 32;
  k_end = k_end > pos + 1 ? pos + 1 : k_end;
  const int h = h0 + i;
  const bool hv = h < a.H;
  float *mlp = a.ml + (((size_t)split * a.rows + t) * a.H + (hv ? h : 0)) * 2;
  if (k_first >= k_end) {   // nothing for this share (its sums are not read)
    if (w == 0 && g == 0 && hv) { mlp[0] = -FLT_MAX; mlp[1] = 0.f; }
    return;
  }
  const int *bt = a.block_tables + (size_t)a.tok_seq[t] * a.max_blocks;
  bf16x8 qf[NF];
#pragma unroll
  for (int f = 0; f < NF; ++f) {
    const int e = 32 * (w + 4 * f) + 8 * g;
    int4 v = make_int4(0, 0, 0, 0);
    if (hv && e < a.E) v = *(const int4 *)(a.q + ((size_t)t * a.H + h) * a.E + e);
    qf[f] = __builtin_bit_cast(bf16x8, v);
  }
  int4 kf[NF][2];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const int key = k0 + 2 * i + c;
      const bool on = key < k_end;
      const uint16_t *row = a.cache + (on ? ((size_t)bt[key / a.block_size] * a.block_size + key % a.block_size) * a.E : 0);
#pragma unroll
      for (int f = 0; f < NF; ++f) {
        const int e = 32 * (w + 4 * f) + 8 * g;
        kf[f][c] = (on && e < a.E) ? *(const int4 *)(row + e) : make_int4(0, 0, 0, 0);
      }
    }
  };
  f32x4 o[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b) o[b] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = -FLT_MAX, l = 0.f;
  fetch(k_first);
  for (int k0 = k_first; k0 < k_end; k0 += 32) {
    f32x4 s[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int f = 0; f < NF; ++f)
#pragma unroll
      for (int c = 0; c < 2; ++c) s[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, kf[f][c]), qf[f], s[c], 0, 0, 0);
#pragma unroll
    for (int f = 0; f < NF; ++f) {
      const int e = 32 * (w + 4 * f) + 8 * g;
      const unsigned x[4] = {(unsigned)kf[f][0].x, (unsigned)kf[f][0].y, (unsigned)kf[f][0].z, (unsigned)kf[f][0].w};
      const unsigned y[4] = {(unsigned)kf[f][1].x, (unsigned)kf[f][1].y, (unsigned)kf[f][1].z, (unsigned)kf[f][1].w};
      if (e < a.R) {   // (the value size is a multiple of 16)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          *(unsigned *)(Ct + (e + 2 * j) * CS + 2 * i) = (x[j] & 0xffffu) | (y[j] << 16);
          *(unsigned *)(Ct + (e + 2 * j + 1) * CS + 2 * i) = (x[j] >> 16) | (y[j] & 0xffff0000u);
        }
      }
    }
#pragma unroll
    for (int c = 0; c < 2; ++c) Sp[(w * 2 + c) * 64 + lane] = make_float4(s[c][0], s[c][1], s[c][2], s[c][3]);
    __syncthreads();
    float p[8], mx = -FLT_MAX;   // p[2 r + c]: key k0 + 8 g + 2 r + c of head h
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      float v[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const float4 x = Sp[(q * 2 + c) * 64 + lane];
        v[0] += x.x; v[1] += x.y; v[2] += x.z; v[3] += x.w;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        p[2 * r + c] = k0 + 8 * g + 2 * r + c < k_end ? v[r] * a.scale2 : -FLT_MAX;
        mx = fmaxf(mx, p[2 * r + c]);
      }
    }
    if (k0 + 32 < k_end) fetch(k0 + 32);
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx), alpha = exp2_f(m - mn);
    float sum = 0.f;
#pragma unroll
    for (int r = 0; r < 8; ++r) {
      p[r] = p[r] > -FLT_MAX ? exp2_f(p[r] - mn) : 0.f;
      sum += p[r];
    }
    l = fmaf(l, alpha, sum);   // (this lane's keys only)
    m = mn;
    bf16x8 pf[3];
    split3(p, pf);
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const int rb = (w + 4 * b) * 16;
      if (rb < a.R) {
        const bf16x8 cf = __builtin_bit_cast(bf16x8, *(const int4 *)(Ct + (rb + i) * CS + 8 * g));
#pragma unroll
        for (int r = 0; r < 4; ++r) o[b][r] *= alpha;
#pragma unroll
        for (int c = 0; c < 3; ++c) o[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cf, pf[c], o[b], 0, 0, 0);
      }
    }
    __syncthreads();
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (!hv) return;
  if (w == 0 && g == 0) { mlp[0] = m; mlp[1] = l; }
  float *op = a.part + (((size_t)split * a.rows + t) * a.H + h) * a.R;
#pragma unroll
  for (int b = 0; b < NB; ++b) {
    const int rb = (w + 4 * b) * 16;
    if (rb < a.R) *(float4 *)(op + rb + 4 * g) = make_float4(o[b][0], o[b][1], o[b][2], o[b][3]);
  }
}
// The shares of a (row, head) joined (with the sink), rounded to bf16, multiplied by the head's expansion w_uv [Dv, R] and the gate: out [rows, H * Dv]
struct LatentMergeArgs {
  const float *part, *ml, *sink, *gate;
  const uint16_t *w_uv;   // [H, Dv, R]
  uint16_t *out;
  int rows, H, R, Dv, splits, ldg;
};
__global__ void __launch_bounds__(1024) latent_merge_kernel(LatentMergeArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];  // o [R] | weight of every share
  const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  float *o = sm, *ws = sm + a.R;
  const size_t step = (size_t)a.rows * a.H, at = (size_t)t * a.H + h;
  const float sv = a.sink ? a.sink[h] * LOG2E : -FLT_MAX;
  float mm = lane < a.splits ? a.ml[(lane * step + at) * 2] : -FLT_MAX;   // (at most 64 shares; every wave does the same)
  const float M = fmaxf(wave_max(mm), sv);
  float e = lane < a.splits ? exp2_f(mm - M) : 0.f;
  const float L = wave_sum(lane < a.splits ? a.ml[(lane * step + at) * 2 + 1] * e : 0.f) + (a.sink ? exp2_f(sv - M) : 0.f);
  if (wave == 0 && lane < a.splits) ws[lane] = e / L;
  __syncthreads();
  const int nthr = blockDim.x, nw = nthr >> 6;
  for (int r = tid; r < a.R; r += nthr) {
    float acc = 0.f;
#pragma unroll 8
    for (int s = 0; s < a.splits; ++s) {   // (an empty share's sums were never written: whatever is read there is dropped)
      const float w = ws[s], v = a.part[(s * step + at) * a.R + r];
      acc = w != 0.f ? fmaf(w, v, acc) : acc;
    }
    o[r] = round_to<bf16_t>(acc);
  }
  __syncthreads();
#pragma unroll 4
  for (int dv = wave; dv < a.Dv; dv += nw) {
    const uint16_t *w = a.w_uv + ((size_t)h * a.Dv + dv) * a.R;
    float acc = 0.f;
    for (int r = lane * 8; r < a.R; r += 512) {
      const int4 v = *(const int4 *)(w + r);
      const unsigned u[4] = {(unsigned)v.x, (unsigned)v.y, (unsigned)v.z, (unsigned)v.w};
      const float4 x0 = *(const float4 *)(o + r), x1 = *(const float4 *)(o + r + 4);
      const float x[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        acc = fmaf(x[2 * j], __uint_as_float(u[j] << 16), acc);
        acc = fmaf(x[2 * j + 1], __uint_as_float(u[j] & 0xffff0000u), acc);
      }
    }
    acc = wave_sum(acc);
    if (lane == 0) {
      if (a.gate) acc *= sigmoid_f(a.gate[(size_t)t * a.ldg + (size_t)h * a.Dv + dv]);
      a.out[at * a.Dv + dv] = from_f<bf16_t>(acc).v;
    }
  }
}

}  // namespace hybc
}  // namespace mrs

using namespace mrs::hybc;
#define S_(s) ((hipStream_t)(s))

extern "C" const char *mrs_hyb_latent_mfma_last_error() { return g_err; }

/* bf16 only.  q [rows, H * DK], k [n_rows, H * DK], vt [H * Dv, n_rows]: the contexts' expanded keys and transposed values in gathered blocks, an entry's blocks one after the
 * other (tables [entries, max_blocks] of gathered block numbers); segment table of at most 64 rows per segment; sink [H] and gate [rows, ldg] nullable; out [rows, H * Dv].
 * DK a multiple of 8 up to 256, Dv a multiple of 8 up to 128, block_size a multiple of 8. */
extern "C" int mrs_hyb_latent_mfma_prompt(const void *q, const void *k, const void *vt, const int *tables, const int *tok_pos, const int *seg_entry, const int *seg_row0,
                                          const int *seg_len, int segments, int seg_rows, const float *sink, const float *gate, int ldg, void *out, int rows, int H, int DK, int Dv,
                                          int n_rows, int max_blocks, int block_size, int window, float scale, void *stream) {
  if (rows <= 0 || segments <= 0) return 0;
  if (H <= 0 || DK <= 0 || DK % 8 || DK > 256 || Dv <= 0 || Dv % 8 || Dv > 128) return fail("mrs_hyb_latent_mfma_prompt: key size a multiple of 8 up to 256, value size a multiple of 8 up to 128");
  if (seg_rows > 64 || block_size <= 0 || block_size % 8 || n_rows % 8) return fail("mrs_hyb_latent_mfma_prompt: segments of at most 64 rows, blocks of a multiple of 8 tokens");
  if (gate && ldg < H * Dv) return fail("mrs_hyb_latent_mfma_prompt: gate rows shorter than heads * value size");
  if (((uintptr_t)q | (uintptr_t)k | (uintptr_t)vt) % 16 || ((uintptr_t)out) % 8) return fail("mrs_hyb_latent_mfma_prompt: unaligned operands");
  const long long n = (long long)segments * H;
  if (n > (1 << 24)) return fail("mrs_hyb_latent_mfma_prompt: too many segments for one launch");
  FlashArgs a{(const uint16_t *)q, (const uint16_t *)k, (const uint16_t *)vt, tables, tok_pos, seg_entry, seg_row0, seg_len, sink, gate, (uint16_t *)out, H, DK, Dv, n_rows, max_blocks,
              block_size, window, ldg, segments, scale * LOG2E};
  dim3 grid((unsigned)((n + 7) / 8 * 8));
  const int nk = (DK + 15) / 16, nv = (Dv + 31) / 32;
#define MRS_LF(NK_, NV_) hipLaunchKernelGGL((latent_flash_kernel<NK_, NV_>), grid, dim3(256), 0, S_(stream), a)
#define MRS_LFK(NK_) do { if (nv <= 1) MRS_LF(NK_, 1); else if (nv <= 2) MRS_LF(NK_, 2); else MRS_LF(NK_, 4); } while (0)
  if (nk <= 4) MRS_LFK(4); else if (nk <= 6) MRS_LFK(6); else if (nk <= 8) MRS_LFK(8); else if (nk <= 12) MRS_LFK(12); else MRS_LFK(16);
#undef MRS_LFK
#undef MRS_LF
  return ok_or("mrs_hyb_latent_mfma_prompt");
}

/* bf16 only.  Single rows: q [rows, H * E] against the pages cache [blocks, block_size, E], value = the first R of a row's E values.  part [splits, rows, H, R] and ml [splits, rows,
 * H, 2]: f32 scratch.  Then out [rows, H * Dv] = gate * (w_uv [H, Dv, R] . joined).  E a multiple of 8 up to 640, R a multiple of 16 up to 512; 1 .. 64 splits. */
extern "C" int mrs_hyb_latent_mfma_decode(const void *q, const void *cache, const int *block_tables, const int *tok_seq, const int *tok_pos, float *part, float *ml, int rows, int H, int R,
                                          int E, int block_size, int max_blocks, int window, int splits, float scale, void *stream) {
  if (rows <= 0) return 0;
  if (H <= 0 || R <= 0 || R % 16 || R > 512 || E < R || E % 8 || E > 640) return fail("mrs_hyb_latent_mfma_decode: latent size a multiple of 16 up to 512, row size a multiple of 8 up to 640");
  if (splits < 1 || splits > 64 || rows > 65535 || block_size <= 0) return fail("mrs_hyb_latent_mfma_decode: 1 .. 64 shares");
  if (((uintptr_t)q | (uintptr_t)cache | (uintptr_t)part) % 16) return fail("mrs_hyb_latent_mfma_decode: unaligned operands");
  LatentDecodeArgs a{(const uint16_t *)q, (const uint16_t *)cache, block_tables, tok_seq, tok_pos, part, ml, rows, H, R, E, block_size, max_blocks, window, splits, scale * LOG2E};
  const size_t lds = 4 * 2 * 64 * 16 + (size_t)R * 80;
  dim3 grid(splits, (H + 15) / 16, rows);
  const int nf = ((E + 31) / 32 + 3) / 4, nb = (R / 16 + 3) / 4;
#define MRS_LD(NF_, NB_) hipLaunchKernelGGL((latent_decode_kernel<NF_, NB_>), grid, dim3(256), lds, S_(stream), a)
  if (nf <= 2 && nb <= 2) MRS_LD(2, 2); else if (nf <= 3 && nb <= 4) MRS_LD(3, 4); else MRS_LD(5, 8);
#undef MRS_LD
  return ok_or("mrs_hyb_latent_mfma_decode");
}
extern "C" int mrs_hyb_latent_mfma_merge(const float *part, const float *ml, const float *sink, const void *w_uv, const float *gate, int ldg, void *out, int rows, int H, int R, int Dv,
                                         int splits, void *stream) {
  if (rows <= 0) return 0;
  if (H <= 0 || R <= 0 || R % 8 || R > 8192 || Dv <= 0 || splits < 1 || splits > 64 || rows > 65535) return fail("mrs_hyb_latent_mfma_merge: sizes (1 .. 64 shares)");
  if (gate && ldg < H * Dv) return fail("mrs_hyb_latent_mfma_merge: gate rows shorter than heads * value size");
  if (((uintptr_t)w_uv) % 16) return fail("mrs_hyb_latent_mfma_merge: unaligned operands");
  LatentMergeArgs a{part, ml, sink, gate, (const uint16_t *)w_uv, (uint16_t *)out, rows, H, R, Dv, splits, ldg};
  const int nthr = (long long)rows * H >= 1024 ? 256 : 1024;   // few (row, head) pairs: more loads of the expansion in flight per compute unit
  hipLaunchKernelGGL(latent_merge_kernel, dim3(H, rows), dim3(nthr), (size_t)(a.R + 64) * 4, S_(stream), a);
  return ok_or("mrs_hyb_latent_mfma_merge");
}
