// hyb_attn_mfma.hip -- softmax attention over paged keys and values for steps with prompt portions, bf16, on the matrix cores (hyb_kernels.hip has the general forms): grouped heads,
// key and value sizes of their own, every earlier token / a sliding window / position chunks, a learned sink per head, a gate per head or per output value.
//
// Scores, maxima, exponentials, weights and all sums are f32: a score is an f32 sum of exact bf16 products; a weight enters its product as THREE bf16 terms that add up to the f32
// number, so the weighted sum too is an f32 sum of exact products.  Exponentials are taken in base two: scale and sink come multiplied by log2(e).
#include "hyb_mfma.cuh"
#include <float.h>

namespace mrs {
namespace hyba {

static thread_local char g_err[256];
static int fail(const char *m) { snprintf(g_err, sizeof g_err, "%s", m); return 1; }
static int ok_or(const char *what) {
  if (hipGetLastError() == hipSuccess) return 0;
  snprintf(g_err, sizeof g_err, "%s: launch failed", what);
  return 1;
}
using namespace mrs::mfma;
__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + expf(-v)); }

struct PagedFlashArgs {
  const uint16_t *q;          // [rows, H * D]
  const uint16_t *k_cache;    // [blocks, G, block_size, D]
  const uint16_t *v_cache;    // [blocks, G, block_size, Dv]
  const int *tables;          // [entries, max_blocks]
  const int *tok_pos;
  const int *seg_entry, *seg_row0, *seg_len;  // segments of at most 64 rows
  const float *sink;          // [H], nullable
  const float *gate;          // nullable: one logit per (row, head) at column h, or (gate_each) one per output value at column h * Dv + d
  uint16_t *out;              // [rows, H * Dv]
  int H, G, D, Dv, max_blocks, block_size, window, chunk, ldg, gate_each, segments;
  float scale2;               // scale * log2(e)
};
// first key that position p sees
__device__ __forceinline__ int first_key(const PagedFlashArgs &a, int p) {
  if (a.chunk > 0) return (p / a.chunk) * a.chunk;
  return a.window > 0 && p - a.window + 1 > 0 ? p - a.window + 1 : 0;
}
// One workgroup of four waves per (segment of 64 queries, head): wave = (query half, key half).  Keys and values pass through LDS 64 at a time, the next tile's in registers meanwhile
// and the tile's after that with its page rows looked up; values are transposed on the way in (two keys' values side by side per write).  S^T = K Q^T leaves a lane with ONE query
// (its column) and sixteen keys, so the softmax needs one exchange between the wave's halves for the maximum, and the weights are already the operand of O^T = V^T P^T: the order
// of the keys inside a product is free, and the V^T fragments are read in the order the lane holds its weights.  The two key halves of a query are joined at the end.
template <int NK, int NV> __global__ void __launch_bounds__(256, NK > 8 || NV > 4 ? 1 : 2) paged_flash_kernel(PagedFlashArgs a) {
  constexpr int KS = NK * 16 + 8, VS = 64 + 4, KU = (NK + 1) / 2, VU = (NV + 1) / 2;   // LDS row strides; pieces per thread of a tile (16 bytes of a key, of two keys' values)
  constexpr int JP = NV > 4 ? 2 : 1, JV = (NV + JP - 1) / JP;                           // the join runs in JP parts of JV value blocks
  constexpr int TILE = 64 * KS + VU * 64 * VS, JOIN = 2 * 64 * (JV * 16 + 2) * 2;      // (in 16-bit values)
  __shared__ __attribute__((aligned(16))) uint16_t lds[TILE > JOIN ? TILE : JOIN];
  __shared__ int rows_at[2][64];   // page row of every key of a tile (-1: not read)
  uint16_t *Ks = lds, *Vs = lds + 64 * KS;
  // workgroups go round robin to the eight dies: every die takes consecutive (head, segment) pairs, so that a head's keys are read through one L2; the longest rows first
  const int n = a.segments * a.H, chunk = gridDim.x >> 3, item = (blockIdx.x & 7) * chunk + (blockIdx.x >> 3);
  if (item >= n) return;
  const int h = item / a.segments, z = a.segments - 1 - item % a.segments, g = h / (a.H / a.G);
  const int r0 = a.seg_row0[z], len = a.seg_len[z];
  if (len <= 0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, ql = lane & 31, kh = lane >> 5, qg = wave & 1, kg = wave >> 1;
  const int pos0 = a.tok_pos[r0], hi = pos0 + len - 1, lo = first_key(a, pos0);
  const int *bt = a.tables + (size_t)a.seg_entry[z] * a.max_blocks;
  const int qi = qg * 32 + ql, t = r0 + (qi < len ? qi : len - 1), pq = pos0 + qi, q_lo = first_key(a, pq);
  const bool qv = qi < len;
  bf16x8 qf[NK];
#pragma unroll
  for (int ks = 0; ks < NK; ++ks) {
    int4 v = make_int4(0, 0, 0, 0);
    if (ks * 16 + 8 * kh < a.D) v = *(const int4 *)(a.q + ((size_t)t * a.H + h) * a.D + ks * 16 + 8 * kh);
    qf[ks] = __builtin_bit_cast(bf16x8, v);
  }
  auto page_row = [&](int key) -> int {
    if (key < lo || key > hi) return -1;
    return (bt[key / a.block_size] * a.G + g) * a.block_size + key % a.block_size;
  };
  int4 kr[KU], vr[VU][2];
  auto fetch = [&](const int *at) {
#pragma unroll
    for (int m = 0; m < KU; ++m) {
      const int u = tid + m * 256, row = u / (NK * 2), c = (u - row * (NK * 2)) * 8, r = row < 64 ? at[row] : -1;
      int4 v = make_int4(0, 0, 0, 0);
      if (r >= 0 && c < a.D) v = *(const int4 *)(a.k_cache + (size_t)r * a.D + c);
      kr[m] = v;
    }
#pragma unroll
    for (int m = 0; m < VU; ++m) {
      const int pair = tid >> 3, dv = m * 64 + (tid & 7) * 8;
#pragma unroll
      for (int j = 0; j < 2; ++j) {
        const int r = at[2 * pair + j];
        int4 v = make_int4(0, 0, 0, 0);   // (a weight of zero must not meet whatever a page holds beside the keys)
        if (r >= 0 && dv < a.Dv) v = *(const int4 *)(a.v_cache + (size_t)r * a.Dv + dv);
        vr[m][j] = v;
      }
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
      const int pair = tid >> 3, dv = m * 64 + (tid & 7) * 8;
      const unsigned x[4] = {(unsigned)vr[m][0].x, (unsigned)vr[m][0].y, (unsigned)vr[m][0].z, (unsigned)vr[m][0].w};
      const unsigned y[4] = {(unsigned)vr[m][1].x, (unsigned)vr[m][1].y, (unsigned)vr[m][1].z, (unsigned)vr[m][1].w};
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        *(unsigned *)(Vs + (dv + 2 * j) * VS + 2 * pair) = (x[j] & 0xffffu) | (y[j] << 16);
        *(unsigned *)(Vs + (dv + 2 * j + 1) * VS + 2 * pair) = (x[j] >> 16) | (y[j] & 0xffff0000u);
      }
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
  const int w_lo = first_key(a, w_first), w_hi_lo = first_key(a, w_last);                       // first keys of the first and of the last of them
  const int kt0 = lo & ~31;
  if (tid < 64) rows_at[0][tid] = page_row(kt0 + tid);
  __syncthreads();
  fetch(rows_at[0]);
  int next_row = tid < 64 ? page_row(kt0 + 64 + tid) : -1, flip = 0;
  for (int kt = kt0; kt <= hi; kt += 64) {
    put();
    flip ^= 1;
    if (tid < 64) rows_at[flip][tid] = next_row;
    __syncthreads();
    if (kt + 64 <= hi) {
      fetch(rows_at[flip]);
      if (tid < 64) next_row = page_row(kt + 128 + tid);
    }
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
      const bool whole = kb + 31 <= w_first && kb >= w_hi_lo;
      float p[16], mx = -FLT_MAX;
      if (whole) {
#pragma unroll
        for (int r = 0; r < 16; ++r) { p[r] = s[r] * a.scale2; mx = fmaxf(mx, p[r]); }
      } else {
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const int key = kb + (r & 3) + 8 * (r >> 2) + 4 * kh;
          p[r] = key <= pq && key >= q_lo ? s[r] * a.scale2 : -FLT_MAX;
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
  float *jb = (float *)lds + (size_t)qg * 64 * (JV * 16 + 2);
  l += __shfl_xor(l, 32, 64);
  const float *gr = a.gate ? a.gate + (size_t)t * a.ldg + (a.gate_each ? (size_t)h * a.Dv : (size_t)h) : nullptr;
  uint16_t *op = a.out + ((size_t)t * a.H + h) * a.Dv;
#pragma unroll
  for (int jp = 0; jp < JP; ++jp) {
    if (kg == 1) {
#pragma unroll
      for (int i = 0; i < JV; ++i)
#pragma unroll
        for (int r = 0; r < 16; ++r)
          if (jp * JV + i < NV) jb[(i * 16 + r) * 64 + lane] = o[jp * JV + i < NV ? jp * JV + i : 0][r];
      jb[JV * 16 * 64 + lane] = m;
      jb[(JV * 16 + 1) * 64 + lane] = l;
    }
    __syncthreads();
    if (kg == 0 && qv) {
      const float m1 = jb[JV * 16 * 64 + lane], l1 = jb[(JV * 16 + 1) * 64 + lane];
      const float M = fmaxf(m, m1), e0 = exp2_f(m - M), e1 = exp2_f(m1 - M), inv = 1.0f / fmaf(l, e0, l1 * e1);
#pragma unroll
      for (int i = 0; i < JV; ++i)
#pragma unroll
        for (int q4 = 0; q4 < 4; ++q4) {
          const int dv = (jp * JV + i) * 32 + 8 * q4 + 4 * kh;
          if (jp * JV + i >= NV || dv >= a.Dv) continue;
          uint16_t w[4];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const int r = 4 * q4 + j;
            float v = fmaf(o[jp * JV + i < NV ? jp * JV + i : 0][r], e0, jb[(i * 16 + r) * 64 + lane] * e1) * inv;
            if (gr) v *= sigmoid_f(gr[a.gate_each ? dv + j : 0]);
            w[j] = from_f<bf16_t>(v).v;
          }
          *(int2 *)(op + dv) = make_int2((int)(w[0] | ((unsigned)w[1] << 16)), (int)(w[2] | ((unsigned)w[3] << 16)));
        }
    }
    if (jp + 1 < JP) __syncthreads();
  }
}

}  // namespace hyba
}  // namespace mrs

using namespace mrs::hyba;
#define S_(s) ((hipStream_t)(s))

extern "C" const char *mrs_hyb_attn_mfma_last_error() { return g_err; }

/* bf16 only.  q [rows, H * D], pages k_cache [blocks, G, block_size, D] and v_cache [blocks, G, block_size, Dv]; segment table of at most 64 rows per segment.  window > 0: the last
 * `window` positions, chunk > 0: the positions of the query's own chunk (not both); sink [H] nullable; gate nullable: [rows, ldg] with one logit per head, or per output value
 * (gate_each).  D and Dv multiples of 8 up to 256. */
extern "C" int mrs_hyb_attn_mfma_prompt(const void *q, const void *k_cache, const void *v_cache, const int *tables, const int *tok_pos, const int *seg_entry, const int *seg_row0,
                                        const int *seg_len, int segments, int seg_rows, const float *sink, const float *gate, int ldg, int gate_each, void *out, int rows, int H, int G,
                                        int D, int Dv, int num_blocks, int max_blocks, int block_size, int window, int chunk, float scale, void *stream) {
  if (rows <= 0 || segments <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D <= 0 || D % 8 || D > 256 || Dv <= 0 || Dv % 8 || Dv > 256) return fail("mrs_hyb_attn_mfma_prompt: key and value sizes multiples of 8 up to 256, heads % kv_heads == 0");
  if (seg_rows > 64 || block_size <= 0 || (long long)num_blocks * G * block_size > 0x7fffffffLL) return fail("mrs_hyb_attn_mfma_prompt: segments of at most 64 rows, fewer than 2^31 page rows");
  if (window > 0 && chunk > 0) return fail("mrs_hyb_attn_mfma_prompt: chunks and a sliding window exclude each other");
  if (gate && ldg < (gate_each ? H * Dv : H)) return fail("mrs_hyb_attn_mfma_prompt: gate rows shorter than heads (* value size)");
  if (((uintptr_t)q | (uintptr_t)k_cache | (uintptr_t)v_cache) % 16 || ((uintptr_t)out) % 8) return fail("mrs_hyb_attn_mfma_prompt: unaligned operands");
  const long long n = (long long)segments * H;
  if (n > (1 << 24)) return fail("mrs_hyb_attn_mfma_prompt: too many segments for one launch");
  PagedFlashArgs a{(const uint16_t *)q, (const uint16_t *)k_cache, (const uint16_t *)v_cache, tables, tok_pos, seg_entry, seg_row0, seg_len, sink, gate, (uint16_t *)out, H, G, D, Dv,
                   max_blocks, block_size, window > 0 ? window : 0, chunk > 0 ? chunk : 0, ldg, gate_each ? 1 : 0, segments, scale * LOG2E};
  dim3 grid((unsigned)((n + 7) / 8 * 8));
  const int nk = (D + 15) / 16, nv = (Dv + 31) / 32;
#define MRS_PF(NK_, NV_) hipLaunchKernelGGL((paged_flash_kernel<NK_, NV_>), grid, dim3(256), 0, S_(stream), a)
#define MRS_PFK(NK_) do { if (nv <= 1) MRS_PF(NK_, 1); else if (nv <= 2) MRS_PF(NK_, 2); else if (nv <= 4) MRS_PF(NK_, 4); else if (nv <= 6) MRS_PF(NK_, 6); else MRS_PF(NK_, 8); } while (0)
  if (nk <= 4) MRS_PFK(4); else if (nk <= 6) MRS_PFK(6); else if (nk <= 8) MRS_PFK(8); else if (nk <= 12) MRS_PFK(12); else MRS_PFK(16);
#undef MRS_PFK
#undef MRS_PF
  return ok_or("mrs_hyb_attn_mfma_prompt");
}
