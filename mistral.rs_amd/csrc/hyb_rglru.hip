// hyb_rglru.hip -- the real-gated linear recurrent unit (Griffin's recurrent block) on ragged batches.  u [rows, C] f32: the convolved branch; its channels are cut into `blocks` equal
// parts, part b with two square matrices:
//   r = sigmoid(Wa_b u_b + ba),  i = sigmoid(Wi_b u_b + bi),  log a = -8 r softplus(lam),  S_t = a S_(t-1) + sqrt(1 - a^2) i u,  out = S_t gelu(y + yb)
// Same conventions as hyb_kernels.hip: a step's rows are one flat range, an entry whose first position is 0 reads its slot as zero; state [slots, C] f32.
//
//   gates   one workgroup per (segment of at most 64 rows, 64 channels of a part): both products, the gates, and the recurrence over the segment from zero -- it leaves the local states
//           and the running products of a, so that what came before enters later with one multiply-add per value
//   carry   per channel: the segments of an entry one after the other; every segment's start, the slot's new state
//   out     S = local + product * start, times the GELU branch, rounded once for the out-projection
//   step    steps of single rows: gates, recurrence and output in one launch
//
// Everything that enters the recurrence is f32.  bf16 weights: u enters its matrix-core products as THREE bf16 terms that add up to the f32 number, so a gate's logit is an f32 sum of
// exact products.
#include "hyb_mfma.cuh"
#include <float.h>

namespace mrs {
namespace hybg {

static thread_local char g_err[256];
static int fail(const char *m) { snprintf(g_err, sizeof g_err, "%s", m); return 1; }
static int ok_or(const char *what) {
  if (hipGetLastError() == hipSuccess) return 0;
  snprintf(g_err, sizeof g_err, "%s: launch failed", what);
  return 1;
}
using namespace mrs::mfma;

__device__ __forceinline__ float sigmoid_f(float v) { return 1.0f / (1.0f + expf(-v)); }
__device__ __forceinline__ float softplus_f(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
__device__ __forceinline__ float gelu_tanh_f(float v) { return 0.5f * v * (1.0f + tanhf(0.7978845608028654f * fmaf(0.044715f * v * v, v, v))); }
// from the gates' logits: what the state keeps and what the row brings
__device__ __forceinline__ void recurrence_of(float zr, float zi, float sp, float u, float &a, float &g) {
  const float la = -8.0f * sigmoid_f(zr) * sp;
  a = expf(la);
  g = sqrtf(-expm1f(2.0f * la)) * sigmoid_f(zi) * u;
}

struct GateArgs {
  const float *u;                  // [rows, C]
  const void *wa, *wi;             // [blocks, part, part] (out, in) in T
  const float *ba, *bi, *lam;      // [C]
  const int *seg_row0, *seg_len;
  float *local, *prod;             // [rows, C]: the segment's state from zero after the row, the product of its a's up to the row
  int C, part, tiles;              // tiles: 64-channel tiles of a part
  int vec_ok;
};
constexpr int GT = 64, GK = 32;    // tile: rows and channels; values of the part per step
template <class T> __global__ void __launch_bounds__(256) rglru_gates_kernel(GateArgs a) {
  constexpr bool MC = sizeof(T) == 2;   // bf16: matrix cores
  constexpr int US = GK + 8;
  // staging and logits do not live at the same time
  constexpr int STAGE = MC ? (3 + 2) * GT * US * 2 : 3 * GT * (GK + 4) * 4, LOG = 2 * GT * (GT + 1) * 4;
  __shared__ __attribute__((aligned(16))) char sm[STAGE > LOG ? STAGE : LOG];
  __shared__ float endA[4][GT], endS[4][GT];
  const int z = blockIdx.x, b = blockIdx.y / a.tiles, n0 = (blockIdx.y % a.tiles) * GT, part = a.part;
  const int r0 = a.seg_row0[z], len = a.seg_len[z];
  if (len <= 0) return;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const float *ub = a.u + (size_t)r0 * a.C + (size_t)b * part;
  const T *wa = (const T *)a.wa + (size_t)b * part * part, *wi = (const T *)a.wi + (size_t)b * part * part;
  float *Lr = (float *)sm, *Li = Lr + GT * (GT + 1);
  const int sr = tid >> 2, kc = (tid & 3) * 8;   // this thread stages row sr (of u, of both weights), values kc .. kc + 7
  auto load_u = [&](int k0, float *v) {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = 0.f;
    if (sr >= len) return;
    const float *p = ub + (size_t)sr * a.C + k0 + kc;
    if (a.vec_ok && k0 + kc + 8 <= part) {
      const float4 x = *(const float4 *)p, y = *(const float4 *)(p + 4);
      v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w; v[4] = y.x; v[5] = y.y; v[6] = y.z; v[7] = y.w;
    } else {
#pragma unroll
      for (int j = 0; j < 8; ++j) if (k0 + kc + j < part) v[j] = p[j];
    }
  };
  if constexpr (MC) {
    uint16_t *Us = (uint16_t *)sm, *Ws = Us + 3 * GT * US;   // [term][row][US], [gate][channel][US]
    auto load_w = [&](const T *w, int k0) -> int4 {
      int4 v = make_int4(0, 0, 0, 0);
      if (n0 + sr < part) {
        const T *p = w + (size_t)(n0 + sr) * part + k0 + kc;
        if (a.vec_ok && k0 + kc + 8 <= part) v = *(const int4 *)p;
        else {
          uint16_t t[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) t[j] = k0 + kc + j < part ? p[j].v : (uint16_t)0;
          v = make_int4((int)(t[0] | ((unsigned)t[1] << 16)), (int)(t[2] | ((unsigned)t[3] << 16)), (int)(t[4] | ((unsigned)t[5] << 16)), (int)(t[6] | ((unsigned)t[7] << 16)));
        }
      }
      return v;
    };
    const int ql = lane & 31, kh = lane >> 5, wm = (wave & 1) * 32, wn = (wave >> 1) * 32;
    f32x16 cr, ci;
#pragma unroll
    for (int r = 0; r < 16; ++r) cr[r] = ci[r] = 0.f;
    float uv[8];
    int4 wv[2];
    load_u(0, uv);
    wv[0] = load_w(wa, 0); wv[1] = load_w(wi, 0);
    for (int k0 = 0; k0 < part; k0 += GK) {
      bf16x8 ut[3];
      split3(uv, ut);
#pragma unroll
      for (int c = 0; c < 3; ++c) *(int4 *)(Us + (c * GT + sr) * US + kc) = __builtin_bit_cast(int4, ut[c]);
#pragma unroll
      for (int c = 0; c < 2; ++c) *(int4 *)(Ws + (c * GT + sr) * US + kc) = wv[c];
      __syncthreads();
      if (k0 + GK < part) { load_u(k0 + GK, uv); wv[0] = load_w(wa, k0 + GK); wv[1] = load_w(wi, k0 + GK); }
#pragma unroll
      for (int ks = 0; ks < GK; ks += 16) {
        const bf16x8 fr = __builtin_bit_cast(bf16x8, *(const int4 *)(Ws + (wn + ql) * US + ks + 8 * kh)), fi = __builtin_bit_cast(bf16x8, *(const int4 *)(Ws + (GT + wn + ql) * US + ks + 8 * kh));
#pragma unroll
        for (int c = 0; c < 3; ++c) {
          const bf16x8 fu = __builtin_bit_cast(bf16x8, *(const int4 *)(Us + (c * GT + wm + ql) * US + ks + 8 * kh));
          cr = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fu, fr, cr, 0, 0, 0);
          ci = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fu, fi, ci, 0, 0, 0);
        }
      }
      __syncthreads();
    }
#pragma unroll
    for (int r = 0; r < 16; ++r) {   // register r: row (r & 3) + 8 (r >> 2) + 4 kh of the wave's quadrant, channel ql
      const int m = wm + (r & 3) + 8 * (r >> 2) + 4 * kh;
      Lr[m * (GT + 1) + wn + ql] = cr[r];
      Li[m * (GT + 1) + wn + ql] = ci[r];
    }
  } else {
    float *Us = (float *)sm, *Wr = Us + GT * (GK + 4), *Wi = Wr + GT * (GK + 4);
    const int tn = tid & 15, tm = tid >> 4;   // rows tm + 16 i, channels tn + 16 j
    float cr[4][4], ci[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) cr[i][j] = ci[i][j] = 0.f;
    for (int k0 = 0; k0 < part; k0 += GK) {
      float uv[8];
      load_u(k0, uv);
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const bool on = n0 + sr < part && k0 + kc + j < part;
        Us[sr * (GK + 4) + kc + j] = uv[j];
        Wr[sr * (GK + 4) + kc + j] = on ? to_f<T>(wa[(size_t)(n0 + sr) * part + k0 + kc + j]) : 0.f;
        Wi[sr * (GK + 4) + kc + j] = on ? to_f<T>(wi[(size_t)(n0 + sr) * part + k0 + kc + j]) : 0.f;
      }
      __syncthreads();
      for (int k = 0; k < GK; ++k) {
        float x[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) x[i] = Us[(tm + 16 * i) * (GK + 4) + k];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float wr = Wr[(tn + 16 * j) * (GK + 4) + k], wv = Wi[(tn + 16 * j) * (GK + 4) + k];
#pragma unroll
          for (int i = 0; i < 4; ++i) { cr[i][j] = fmaf(x[i], wr, cr[i][j]); ci[i][j] = fmaf(x[i], wv, ci[i][j]); }
        }
      }
      __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        Lr[(tm + 16 * i) * (GT + 1) + tn + 16 * j] = cr[i][j];
        Li[(tm + 16 * i) * (GT + 1) + tn + 16 * j] = ci[i][j];
      }
  }
  __syncthreads();
  // a thread = one channel of sixteen rows: gates, the states from zero, the products; the quarters of the segment then take in what is before them
  const int n = lane, ch = b * part + n0 + n, m0 = wave * 16;
  const bool live = n0 + n < part;
  const int chc = live ? ch : b * part;
  const float sp = softplus_f(a.lam[chc]), ba = a.ba[chc], bi = a.bi[chc];
  float S[16], P[16], s = 0.f, p = 1.0f;
#pragma unroll
  for (int k = 0; k < 16; ++k) {
    const int m = m0 + k;
    if (m < len && live) {
      float av, gv;
      recurrence_of(Lr[m * (GT + 1) + n] + ba, Li[m * (GT + 1) + n] + bi, sp, a.u[(size_t)(r0 + m) * a.C + ch], av, gv);
      s = fmaf(av, s, gv);
      p *= av;
    }
    S[k] = s; P[k] = p;
  }
  endA[wave][n] = p; endS[wave][n] = s;
  __syncthreads();
  float s0 = 0.f, p0 = 1.0f;
  for (int w = 0; w < wave; ++w) { s0 = fmaf(endA[w][n], s0, endS[w][n]); p0 *= endA[w][n]; }
#pragma unroll
  for (int k = 0; k < 16; ++k) {
    const int m = m0 + k;
    if (m >= len || !live) break;
    a.local[(size_t)(r0 + m) * a.C + ch] = fmaf(P[k], s0, S[k]);
    a.prod[(size_t)(r0 + m) * a.C + ch] = P[k] * p0;
  }
}

// start [segments, C]: the state in front of every segment; the slot takes the state behind the entry's last one
__global__ void __launch_bounds__(256) rglru_carry_kernel(const float *__restrict__ local, const float *__restrict__ prod, float *__restrict__ start, float *__restrict__ state,
                                                          const int *__restrict__ seq_pos0, const int *__restrict__ seq_slot, const int *__restrict__ seg_row0, const int *__restrict__ seg_len,
                                                          const int *__restrict__ ent_seg0, int C) {
  const int c = blockIdx.x * 256 + threadIdx.x, s = blockIdx.y;
  if (c >= C) return;
  float *st = state + (size_t)seq_slot[s] * C + c;
  float cur = seq_pos0[s] > 0 ? *st : 0.f;
  const int z0 = ent_seg0[s], z1 = ent_seg0[s + 1];
#pragma unroll 8
  for (int z = z0; z < z1; ++z) {
    start[(size_t)z * C + c] = cur;
    const int len = seg_len[z];
    const size_t at = (size_t)(seg_row0[z] + (len > 0 ? len - 1 : 0)) * C + c;
    const float p = prod[at], l = local[at];
    cur = len > 0 ? fmaf(p, cur, l) : cur;
  }
  *st = cur;
}
template <class T, int V> __global__ void __launch_bounds__(256) rglru_out_kernel(const float *__restrict__ local, const float *__restrict__ prod, const float *__restrict__ start,
                                                                                  const float *__restrict__ y, int ldy, const float *__restrict__ yb, T *__restrict__ out,
                                                                                  const int *__restrict__ seg_row0, const int *__restrict__ seg_len, int C, int rows_per) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * V, z = blockIdx.z, m0 = blockIdx.y * rows_per;
  if (c >= C) return;
  const int len = seg_len[z], r0 = seg_row0[z], m1 = m0 + rows_per < len ? m0 + rows_per : len;
  float st[V], bb[V];
#pragma unroll
  for (int j = 0; j < V; ++j) { st[j] = start[(size_t)z * C + c + j]; bb[j] = yb[c + j]; }
  for (int m = m0; m < m1; ++m) {
    const size_t t = r0 + m;
    float l[V], p[V], g[V];
    if (V == 4) {
      const float4 l4 = *(const float4 *)(local + t * C + c), p4 = *(const float4 *)(prod + t * C + c), y4 = *(const float4 *)(y + t * ldy + c);
      l[0] = l4.x; l[V > 1 ? 1 : 0] = l4.y; l[V > 2 ? 2 : 0] = l4.z; l[V > 3 ? 3 : 0] = l4.w;
      p[0] = p4.x; p[V > 1 ? 1 : 0] = p4.y; p[V > 2 ? 2 : 0] = p4.z; p[V > 3 ? 3 : 0] = p4.w;
      g[0] = y4.x; g[V > 1 ? 1 : 0] = y4.y; g[V > 2 ? 2 : 0] = y4.z; g[V > 3 ? 3 : 0] = y4.w;
    } else {
      l[0] = local[t * C + c]; p[0] = prod[t * C + c]; g[0] = y[t * ldy + c];
    }
#pragma unroll
    for (int j = 0; j < V; ++j) out[t * C + c + j] = from_f<T>(fmaf(p[j], st[j], l[j]) * gelu_tanh_f(g[j] + bb[j]));
  }
}

// Steps of single rows: a wave makes both logits of one channel for up to MR entries (the matrices are read once for all of them), lane m then steps the channel of entry m.
struct StepArgs {
  const float *u;                  // [rows, C]
  const void *wa, *wi;
  const float *ba, *bi, *lam;
  const float *y;                  // [rows, ldy]
  const float *yb;
  float *state;
  void *out;                       // [rows, C] in T
  const int *seq_start, *seq_pos0, *seq_slot;
  int C, part, ldy, entries, vec_ok;
};
template <class T> struct W8;
template <> struct W8<bf16_t> {
  static __device__ __forceinline__ void load(const bf16_t *p, float *o) {
    const int4 v = *(const int4 *)p;
    const unsigned u[4] = {(unsigned)v.x, (unsigned)v.y, (unsigned)v.z, (unsigned)v.w};
#pragma unroll
    for (int j = 0; j < 4; ++j) { o[2 * j] = __uint_as_float(u[j] << 16); o[2 * j + 1] = __uint_as_float(u[j] & 0xffff0000u); }
  }
};
template <> struct W8<float> {
  static __device__ __forceinline__ void load(const float *p, float *o) {
    const float4 a = *(const float4 *)p, b = *(const float4 *)(p + 4);
    o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
  }
};
template <class T, int MR> __global__ void __launch_bounds__(256) rglru_step_kernel(StepArgs a) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, ch = blockIdx.x * 4 + wave, s0 = blockIdx.y * MR;
  if (ch >= a.C) return;
  const int cnt = a.entries - s0 < MR ? a.entries - s0 : MR, b = ch / a.part, n = ch - b * a.part;
  const T *wa = (const T *)a.wa + ((size_t)b * a.part + n) * a.part, *wi = (const T *)a.wi + ((size_t)b * a.part + n) * a.part;
  const float *ub = a.u + (size_t)b * a.part;
  float zr[MR], zi[MR];
#pragma unroll
  for (int m = 0; m < MR; ++m) zr[m] = zi[m] = 0.f;
  if (a.vec_ok) {
    for (int k = lane * 8; k < a.part; k += 512) {
      float x[8], wr[8], wv[8];
      W8<T>::load(wa + k, wr);
      W8<T>::load(wi + k, wv);
#pragma unroll
      for (int m = 0; m < MR; ++m)
        if (m < cnt) {
          W8<float>::load(ub + (size_t)a.seq_start[s0 + m] * a.C + k, x);
#pragma unroll
          for (int j = 0; j < 8; ++j) { zr[m] = fmaf(wr[j], x[j], zr[m]); zi[m] = fmaf(wv[j], x[j], zi[m]); }
        }
    }
  } else {
    for (int k = lane; k < a.part; k += 64) {
      const float wr = to_f<T>(wa[k]), wv = to_f<T>(wi[k]);
#pragma unroll
      for (int m = 0; m < MR; ++m)
        if (m < cnt) {
          const float x = ub[(size_t)a.seq_start[s0 + m] * a.C + k];
          zr[m] = fmaf(wr, x, zr[m]);
          zi[m] = fmaf(wv, x, zi[m]);
        }
    }
  }
  float mr = 0.f, mi = 0.f;
#pragma unroll
  for (int m = 0; m < MR; ++m) {
    const float x = wave_sum(zr[m]), y = wave_sum(zi[m]);
    if (lane == m) { mr = x; mi = y; }
  }
  if (lane >= cnt) return;
  const int s = s0 + lane;
  const size_t t = a.seq_start[s];
  float av, gv;
  recurrence_of(mr + a.ba[ch], mi + a.bi[ch], softplus_f(a.lam[ch]), a.u[t * a.C + ch], av, gv);
  float *st = a.state + (size_t)a.seq_slot[s] * a.C + ch;
  const float S = fmaf(av, a.seq_pos0[s] > 0 ? *st : 0.f, gv);
  *st = S;
  ((T *)a.out)[t * a.C + ch] = from_f<T>(S * gelu_tanh_f(a.y[t * a.ldy + ch] + a.yb[ch]));
}

}  // namespace hybg
}  // namespace mrs

using namespace mrs::hybg;
#define S_(s) ((hipStream_t)(s))

extern "C" const char *mrs_hyb_rglru_last_error() { return g_err; }

/* u [rows, C] f32 (the convolved branch), wa / wi [blocks, C / blocks, C / blocks] (dtype), ba / bi / lam [C]; y [rows, ldy] f32 and yb [C]: the GELU branch before its bias.
 * Segment table of at most 64 rows per segment; local, prod [rows, C] and start [segments, C]: f32 scratch; out [rows, C] (dtype) = state * gelu(y + yb). */
extern "C" int mrs_hyb_rglru_scan(const float *u, const void *wa, const void *wi, const float *ba, const float *bi, const float *lam, const float *y, int ldy, const float *yb,
                                  float *state, float *local, float *prod, float *start, void *out, const int *seq_pos0, const int *seq_slot, const int *seg_row0, const int *seg_len,
                                  const int *ent_seg0, int rows, int entries, int segments, int seg_rows, int C, int blocks, int dtype, void *stream) {
  if (rows <= 0 || entries <= 0 || segments <= 0) return 0;
  if (C <= 0 || blocks <= 0 || C % blocks || ldy < C) return fail("mrs_hyb_rglru_scan: width % blocks must be 0; rows shorter than the width");
  if (seg_rows > GT || entries > 65535 || segments > 65535) return fail("mrs_hyb_rglru_scan: segments of at most 64 rows, at most 65535 segments");
  if (dtype != 1 && dtype != 2) return fail("mrs_hyb_rglru_scan: dtype");
  const int part = C / blocks, tiles = (part + GT - 1) / GT;
  if ((long long)blocks * tiles > 65535) return fail("mrs_hyb_rglru_scan: too many channel tiles for one launch");
  const int vec = part % 8 == 0 && ((uintptr_t)u % 16) == 0 && ((uintptr_t)wa % 16) == 0 && ((uintptr_t)wi % 16) == 0;
  GateArgs a{u, wa, wi, ba, bi, lam, seg_row0, seg_len, local, prod, C, part, tiles, vec};
  const dim3 grid(segments, blocks * tiles);
  if (dtype == 1) hipLaunchKernelGGL(rglru_gates_kernel<mrs::bf16_t>, grid, dim3(256), 0, S_(stream), a);
  else hipLaunchKernelGGL(rglru_gates_kernel<float>, grid, dim3(256), 0, S_(stream), a);
  hipLaunchKernelGGL(rglru_carry_kernel, dim3((C + 255) / 256, entries), dim3(256), 0, S_(stream), local, prod, start, state, seq_pos0, seq_slot, seg_row0, seg_len, ent_seg0, C);
  const bool v4 = C % 4 == 0 && ldy % 4 == 0 && (((uintptr_t)local | (uintptr_t)prod | (uintptr_t)y) % 16) == 0;
  constexpr int PER = 8;   // rows per workgroup of the output pass
  const dim3 go((C / (v4 ? 4 : 1) + 255) / 256, (seg_rows + PER - 1) / PER, segments);
#define MRS_RGO(T) do { if (v4) hipLaunchKernelGGL((rglru_out_kernel<T, 4>), go, dim3(256), 0, S_(stream), local, prod, start, y, ldy, yb, (T *)out, seg_row0, seg_len, C, PER); \
                        else hipLaunchKernelGGL((rglru_out_kernel<T, 1>), go, dim3(256), 0, S_(stream), local, prod, start, y, ldy, yb, (T *)out, seg_row0, seg_len, C, PER); } while (0)
  if (dtype == 1) MRS_RGO(mrs::bf16_t); else MRS_RGO(float);
#undef MRS_RGO
  return ok_or("mrs_hyb_rglru_scan");
}

/* steps of single rows (rows == entries) */
extern "C" int mrs_hyb_rglru_step(const float *u, const void *wa, const void *wi, const float *ba, const float *bi, const float *lam, const float *y, int ldy, const float *yb,
                                  float *state, void *out, const int *seq_start, const int *seq_pos0, const int *seq_slot, int rows, int entries, int C, int blocks, int dtype,
                                  void *stream) {
  if (rows <= 0) return 0;
  if (rows != entries) return fail("mrs_hyb_rglru_step: one row per entry");
  if (C <= 0 || blocks <= 0 || C % blocks || ldy < C) return fail("mrs_hyb_rglru_step: width % blocks must be 0; rows shorter than the width");
  const int part = C / blocks;
  const int vec = part % 8 == 0 && ((uintptr_t)u % 16) == 0 && ((uintptr_t)wa % 16) == 0 && ((uintptr_t)wi % 16) == 0;
  StepArgs a{u, wa, wi, ba, bi, lam, y, yb, state, out, seq_start, seq_pos0, seq_slot, C, part, ldy, entries, vec};
  const int mr = entries <= 1 ? 1 : entries <= 2 ? 2 : entries <= 4 ? 4 : 8;
  const dim3 grid((C + 3) / 4, (entries + mr - 1) / mr);
  if (grid.y > 65535) return fail("mrs_hyb_rglru_step: too many entries for one launch");
#define MRS_RGS_(T, M_) hipLaunchKernelGGL((rglru_step_kernel<T, M_>), grid, dim3(256), 0, S_(stream), a)
#define MRS_RGS(T) do { if (mr == 1) MRS_RGS_(T, 1); else if (mr == 2) MRS_RGS_(T, 2); else if (mr == 4) MRS_RGS_(T, 4); else MRS_RGS_(T, 8); } while (0)
  if (dtype == 1) MRS_RGS(mrs::bf16_t);
  else if (dtype == 2) MRS_RGS(float);
  else return fail("mrs_hyb_rglru_step: dtype");
#undef MRS_RGS
#undef MRS_RGS_
  return ok_or("mrs_hyb_rglru_step");
}
