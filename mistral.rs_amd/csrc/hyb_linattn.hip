// hyb_linattn.hip -- linear attention with a decayed outer-product state (f32 [slot, head, D, Dv], carried per sequence slot), in three forms:
//   channel decays   alpha = sigmoid(z + bias)^(1 / tau);   S <- diag(alpha) S + k v^T;   o = S^T (q q_mult)                    (gated linear attention)
//   bonus            alpha = exp(-exp(z + bias));   o = (S + diag(u) k v^T)^T q;   S <- diag(alpha) S + k v^T                   (time mixing: the current token enters o through u)
//   head decays      S <- decay_h S + silu(k) silu(v)^T;   o = S^T silu(q)                                                       (one constant per head, SiLU operands)
// Same conventions as hyb_kernels.hip: a step's rows are one flat range, entry s owns rows [seq_start[s], seq_start[s + 1]) at positions seq_pos0[s] + i and state slot
// seq_slot[s]; an entry whose first position is 0 reads its slot as zero.
//
//   scan   steps with portions: entries as chains, or the segments of long portions side by side (end states and decay products from zero, a carry, the outputs)
//   step   steps of single rows: the second step of the decay's projection, the decays, the state update, the read-out, the per-head output norm and the SiLU gate in one launch
//          (head decays: the state update and the read-out; the norm over all heads follows)
//   shift  the operands of time mixing: every row mixed with its predecessor, five mixes per row, the last row of an entry into its slot
//
// Everything here is f32 arithmetic on f32 operands; T is only the type the results are rounded to for the next product (and the type of a weight).
#include "common.cuh"
#include <float.h>

namespace mrs {
namespace hybl {

static thread_local char g_err[256];
static int fail(const char *m) { snprintf(g_err, sizeof g_err, "%s", m); return 1; }
static int ok_or(const char *what) {
  if (hipGetLastError() == hipSuccess) return 0;
  snprintf(g_err, sizeof g_err, "%s: launch failed", what);
  return 1;
}

enum { FORM_CHANNEL = 0, FORM_BONUS = 1, FORM_HEAD = 2 };
__device__ __forceinline__ float silu_f(float v) { return v / (1.0f + expf(-v)); }
// SiLU in the loop that stages operands: hardware exponential and reciprocal (one unit in the last place each)
__device__ __forceinline__ float silu_quick(float v) { return v * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(v * -1.4426950408889634f)); }
__device__ __forceinline__ float softplus_f(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
// sigmoid(z)^(1 / tau) through its logarithm, -softplus(-z) / tau: no cancellation at either end
__device__ __forceinline__ float channel_decay(float z, float inv_tau) { return expf(-softplus_f(-z) * inv_tau); }

// sum over groups of R consecutive lanes (R = 4, 8, 16, groups aligned to R) with data-parallel-primitive moves inside a row of 16 lanes
template <int CTRL> __device__ __forceinline__ float dpp_add(float x) {
  return x + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xf, 0xf, true));
}
template <int R> __device__ __forceinline__ float group_sum(float x) {
  static_assert(R == 4 || R == 8 || R == 16, "groups of 4, 8 or 16 lanes");
  x = dpp_add<0xB1>(x);               // quad_perm [1, 0, 3, 2]
  x = dpp_add<0x4E>(x);               // quad_perm [2, 3, 0, 1]
  if (R == 8) x = dpp_add<0x141>(x);  // row_half_mirror: the other quad of the eight
  if (R == 16) {
    x = dpp_add<0x124>(x);            // row_ror 4
    x = dpp_add<0x128>(x);            // row_ror 8
  }
  return x;
}

struct GlaArgs {
  const float *u;       // [rows, ldu]: v [H * Dv] at 0, k [H * D] at k_col, q [H * D] at q_col
  const float *dec;     // [rows, H * D]: the decays
  float *state;         // [slots, H, D, Dv]
  float *out;           // [rows, H * Dv]
  const int *seq_pos0, *seq_slot;
  const int *seg_entry, *seg_row0, *seg_len, *ent_seg0;  // segment table: entry, first row, rows; first segment of every entry (+ the total)
  float *carry;         // [segments, H, D, Dv]: a segment's end state from zero, then the state the next segment starts from
  float *decay;         // [segments, H, D]: the products of a segment's decays
  int ldu, k_col, q_col, H, D, Dv;
  float q_mult;
  const float *bonus;       // [H, D]       (bonus form)
  const float *head_decay;  // [H]          (head form; `dec` is not read)
};
// decays of all rows, in place: z [rows, n] (the products W_a2 a1) -> sigmoid(z + b)^(1 / tau); V values per access
// (inv_tau 0: exp(-exp(z + b)))
__device__ __forceinline__ float decay_of(float z, float inv_tau) { return inv_tau > 0.f ? channel_decay(z, inv_tau) : expf(-expf(z)); }
template <int V> __global__ void __launch_bounds__(256) gla_decays_kernel(float *__restrict__ z, const float *__restrict__ b, int n, size_t total, float inv_tau) {
  const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= total) return;
  const int c = (int)(i % n);
  if (V == 4) {
    float4 v = *(const float4 *)(z + i);
    v.x = decay_of(v.x + b[c], inv_tau); v.y = decay_of(v.y + b[c + 1], inv_tau);
    v.z = decay_of(v.z + b[c + 2], inv_tau); v.w = decay_of(v.w + b[c + 3], inv_tau);
    *(float4 *)(z + i) = v;
  } else {
    z[i] = decay_of(z[i] + b[c], inv_tau);
  }
}

// The recurrence is linear in S and a row scales the state's rows by numbers of its own, so a long portion can run its segments side by side:
//   A  every segment but an entry's last, from zero: its end state L_k and the channel products d_k                        (LOCAL; parallel over segments)
//   B  init_(k+1) = diag(d_k) init_k + L_k, init_0 = the slot's state (zero for an entry that starts at position 0)      (gla_carry_kernel)
//   C  every segment from its init state: the outputs; an entry's last segment leaves the slot's new state               (parallel over segments)
// An entry of one segment is pass C alone.
// A workgroup owns one (segment, head) and 64 / R * 4 value columns per wave.  A lane holds a register tile of the state: 4 columns times K = 4 J rows n = 4 (j R + r) + i (r = its
// place in the group of R lanes): per row of tokens it reads 3 J + 1 16-byte groups (k, q, decays, v) from LDS for 12 K multiply-adds, lanes of a group at adjacent
// addresses, and the four column sums close with data-parallel-primitive adds inside the group.  Token rows are staged TC at a time, key sizes and columns zero-padded to the tile
// so that the loop has no guards; the next stage's values travel in registers while the current one is consumed.
// The bonus form reads the state before a row's product enters it and adds the row's own value times sum_n u_n k_n q_n, one number per row that the lanes of a group add up
// next to the read-out; the head form carries no decays through LDS and takes the SiLU of its operands on the way in.
template <int R, int J, bool LOCAL, int NT, int FORM> __global__ void __launch_bounds__(NT) gla_scan_kernel(GlaArgs a, int TC, int vec) {
  extern __shared__ __attribute__((aligned(16))) float sm[];  // [2][TC][k Dp | q Dp | decay Dp (not in the head form) | v PC]
  constexpr int K = 4 * J, Dp = R * K, CW = 64 / R * 4, MAXV = 4, VO = (FORM == FORM_HEAD ? 2 : 3) * Dp;   // VO: where the values start
  const int tid = threadIdx.x, nthr = blockDim.x, wave = tid >> 6, lane = tid & 63, r = lane % R, pl = lane / R;
  const int h = blockIdx.y, z = blockIdx.z, PC = (nthr >> 6) * CW, p0 = blockIdx.x * PC;
  const int s = a.seg_entry[z], r0 = a.seg_row0[z], len = a.seg_len[z], D = a.D, Dv = a.Dv;
  const bool first = z == a.ent_seg0[s], last = z == a.ent_seg0[s + 1] - 1;
  if (len <= 0 || (LOCAL && last)) return;
  const int pc = wave * CW + pl * 4, p = p0 + pc;    // this lane's first column: in the workgroup, in the head
  const size_t np = (size_t)D * Dv;
  float *st = a.state + ((size_t)a.seq_slot[s] * a.H + h) * np;
  const float *init = LOCAL ? nullptr : (first ? (a.seq_pos0[s] > 0 ? st : nullptr) : a.carry + ((size_t)(z - 1) * a.H + h) * np);
  float S[K][4], prod[LOCAL ? K : 1], ub[FORM == FORM_BONUS ? K : 1];
  const float hd = FORM == FORM_HEAD ? a.head_decay[h] : 0.f;
#pragma unroll
  for (int k = 0; k < K; ++k) {
    const int n = 4 * ((k >> 2) * R + r) + (k & 3);
#pragma unroll
    for (int c = 0; c < 4; ++c) S[k][c] = (init && n < D && p + c < Dv) ? init[(size_t)n * Dv + p + c] : 0.f;
    if (LOCAL) prod[k] = 1.0f;
    if (FORM == FORM_BONUS) ub[FORM == FORM_BONUS ? k : 0] = n < D ? a.bonus[h * D + n] : 0.f;
  }
  // a stage = TC rows of U groups of four values, dealt to the threads flat; where a group comes from is worked out once
  const int U = (VO + PC) >> 2, stage_n = TC * U, rowlen = 4 * U, stage = TC * rowlen;
  float4 stg[MAXV];
  int src[MAXV], info[MAXV];   // offset in u or z of the group in the first stage; what (0 nothing, 1 plain, 2 query, 3 decay) | values << 2 | row << 5
#pragma unroll
  for (int m = 0; m < MAXV; ++m) {
    const int e = tid + m * nthr;
    src[m] = info[m] = 0;
    if (e >= stage_n) continue;
    const int i = e / U, j = 4 * (e - i * U), row = r0 + i;
    int what = 1, left;
    if (j < VO) {
      const int which = j / Dp, n = j - which * Dp;
      left = D - n;
      what = 1 + which;
      src[m] = which < 2 ? row * a.ldu + (which ? a.q_col : a.k_col) + h * D + n : row * a.H * D + h * D + n;
    } else {
      const int c = p0 + j - VO;
      left = Dv - c;
      src[m] = row * a.ldu + h * Dv + c;
    }
    left = left > 4 ? 4 : left;
    if (left > 0) info[m] = what | (left << 2) | (i << 5);
  }
  auto fetch = [&](int c0) {
#pragma unroll
    for (int m = 0; m < MAXV; ++m) {
      float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
      const int what = info[m] & 3, left = (info[m] >> 2) & 7, i = info[m] >> 5;
      if (what && c0 + i < len) {
        const float *q = what == 3 ? a.dec + (src[m] + c0 * a.H * D) : a.u + (src[m] + c0 * a.ldu);
        if (vec && left == 4) v = *(const float4 *)q;
        else {
          v.x = q[0];
          if (left > 1) v.y = q[1];
          if (left > 2) v.z = q[2];
          if (left > 3) v.w = q[3];
        }
      }
      stg[m] = v;
    }
  };
  auto put = [&](float *buf) {
#pragma unroll
    for (int m = 0; m < MAXV; ++m) {
      const int e = tid + m * nthr, what = info[m] & 3;
      if (e >= stage_n) continue;
      float4 v = stg[m];
      if (FORM == FORM_HEAD) { v.x = silu_quick(v.x); v.y = silu_quick(v.y); v.z = silu_quick(v.z); v.w = silu_quick(v.w); }
      if (what == 2) { v.x *= a.q_mult; v.y *= a.q_mult; v.z *= a.q_mult; v.w *= a.q_mult; }
      *(float4 *)(buf + 4 * e) = v;
    }
  };
  fetch(0);
  put(sm);
  __syncthreads();
  const bool out_vec = vec && p + 4 <= Dv;
  int flip = 0;
  for (int c0 = 0; c0 < len; c0 += TC, flip ^= 1) {
    const float *cur = sm + flip * stage;
    const bool more = c0 + TC < len;
    if (more) fetch(c0 + TC);
    const int cnt = len - c0 < TC ? len - c0 : TC;
    for (int i = 0; i < cnt; ++i) {
      const float *row = cur + i * rowlen;
      const float4 v4 = *(const float4 *)(row + VO + pc);
      const float vv[4] = {v4.x, v4.y, v4.z, v4.w};
      float o[4] = {0.f, 0.f, 0.f, 0.f}, own = 0.f;
#pragma unroll
      for (int j = 0; j < J; ++j) {
        const int n = 4 * (j * R + r);
        const float4 k4 = *(const float4 *)(row + n);
        float4 a4 = make_float4(hd, hd, hd, hd);
        if (FORM != FORM_HEAD) a4 = *(const float4 *)(row + 2 * Dp + n);
        float4 q4 = make_float4(0.f, 0.f, 0.f, 0.f);
        if (!LOCAL) q4 = *(const float4 *)(row + Dp + n);
        const float kk[4] = {k4.x, k4.y, k4.z, k4.w}, aa[4] = {a4.x, a4.y, a4.z, a4.w}, qq[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int i4 = 0; i4 < 4; ++i4) {
          float *Sr = S[4 * j + i4];
          if (FORM == FORM_BONUS && !LOCAL) own = fmaf(ub[FORM == FORM_BONUS ? 4 * j + i4 : 0] * kk[i4], qq[i4], own);
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            if (FORM == FORM_BONUS && !LOCAL) o[c] = fmaf(Sr[c], qq[i4], o[c]);
            Sr[c] = fmaf(aa[i4], Sr[c], kk[i4] * vv[c]);
            if (FORM != FORM_BONUS && !LOCAL) o[c] = fmaf(Sr[c], qq[i4], o[c]);
          }
          if (LOCAL) prod[LOCAL ? 4 * j + i4 : 0] *= aa[i4];
        }
      }
      if (!LOCAL) {
#pragma unroll
        for (int c = 0; c < 4; ++c) o[c] = group_sum<R>(FORM == FORM_BONUS ? fmaf(own, vv[c], o[c]) : o[c]);
        if (r == 0) {
          float *op = a.out + (size_t)(r0 + c0 + i) * a.H * Dv + (size_t)h * Dv + p;
          if (out_vec) *(float4 *)op = make_float4(o[0], o[1], o[2], o[3]);
          else {
#pragma unroll
            for (int c = 0; c < 4; ++c)
              if (p + c < Dv) op[c] = o[c];
          }
        }
      }
    }
    if (more) put(sm + (flip ^ 1) * stage);
    __syncthreads();
  }
  if (LOCAL) {
    if (blockIdx.x == 0 && wave == 0 && pl == 0)
#pragma unroll
      for (int k = 0; k < K; ++k) {
        const int n = 4 * ((k >> 2) * R + r) + (k & 3);
        if (n < D) a.decay[((size_t)z * a.H + h) * D + n] = prod[LOCAL ? k : 0];
      }
    st = a.carry + ((size_t)z * a.H + h) * np;
  }
  if (LOCAL || last)
#pragma unroll
    for (int k = 0; k < K; ++k) {
      const int n = 4 * ((k >> 2) * R + r) + (k & 3);
      if (n >= D) continue;
      float *d = st + (size_t)n * Dv + p;
      if (out_vec) *(float4 *)d = make_float4(S[k][0], S[k][1], S[k][2], S[k][3]);
      else {
#pragma unroll
        for (int c = 0; c < 4; ++c)
          if (p + c < Dv) d[c] = S[k][c];
      }
    }
}
__global__ void __launch_bounds__(256) gla_carry_kernel(GlaArgs a) {
  const int e = blockIdx.x * 256 + threadIdx.x, h = blockIdx.y, s = blockIdx.z;
  const int np = a.D * a.Dv;
  if (e >= np) return;
  const int z0 = a.ent_seg0[s], z1 = a.ent_seg0[s + 1], n = e / a.Dv;
  if (z1 - z0 < 2) return;
  float cur = a.seq_pos0[s] > 0 ? a.state[((size_t)a.seq_slot[s] * a.H + h) * np + e] : 0.f;
  for (int z = z0; z < z1 - 1; ++z) {
    float *c = a.carry + ((size_t)z * a.H + h) * np + e;
    cur = fmaf(a.decay[((size_t)z * a.H + h) * a.D + n], cur, *c);
    *c = cur;
  }
}

// Steps of single rows: one workgroup per (entry, head).  z = W_a2 a1 (a1: the row's `rank` values at a1_col of u, rounded to T as the product would read them), decays, then
// thread (y, x) owns the columns 4 x .. 4 x + 3 (VP = 4) or x (VP = 1) of the state rows y, y + Y, ..: it updates them in place and adds up its part of the read-out; the parts
// meet in LDS, the head is divided by its root mean square, multiplied by the weight `norm` [Dv] and by silu(gate).
// Bonus form: a1 is tanh of the row's values (rounded to T), decays exp(-exp(z)), the read-out before the update plus the row's own value through u, `norm` [H * Dv].
// Head form: operands through SiLU, one decay, the read-out in f32 to out32; grid.z workgroups of `span` columns each share a head.
struct GlaStepArgs {
  const float *u;           // [rows, ldu]: v | k | q | gate [H * Dv] at g_col | a1 [rank] at a1_col
  const void *wa2;          // [H * D, rank] in T
  const float *zb, *norm;
  float *state;
  const int *seq_start, *seq_pos0, *seq_slot;
  void *out;                // [rows, H * Dv] in T
  int ldu, k_col, q_col, g_col, a1_col, rank, H, D, Dv;
  float q_mult, inv_tau, eps;
  const float *a1;          // nullable: the decay projection's first step in rows of its own, [rows, rank], instead of columns of u
  const float *bonus, *head_decay;
  float *out32;
  int span;
};
template <class T, int VP, int FORM> __global__ void __launch_bounds__(1024) gla_step_kernel(GlaStepArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];  // k [Dq] | q [Dq] | decay [Dq] | a1 [rank padded] | o [Dv padded] | parts [Y][X * VP]
  __shared__ float red[16];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, nthr = blockDim.x, D = a.D, Dv = a.Dv, t = a.seq_start[s];
  if (a.seq_start[s + 1] - t != 1) return;
  const int Dq = (D + 3) & ~3, rp = (a.rank + 3) & ~3, vp = (Dv + 3) & ~3;
  float *ks = sm, *qs = ks + Dq, *as = qs + Dq, *a1 = as + Dq, *os = a1 + rp, *parts = os + vp;
  const float *ur = a.u + (size_t)t * a.ldu;
  const float *ar = a.a1 ? a.a1 + (size_t)t * a.rank : ur + a.a1_col;
  for (int j = tid; j < a.rank; j += nthr) a1[j] = round_to<T>(FORM == FORM_BONUS ? tanhf(ar[j]) : ar[j]);
  for (int n = tid; n < D; n += nthr) {
    float kn = ur[a.k_col + h * D + n], qn = ur[a.q_col + h * D + n];
    if (FORM == FORM_HEAD) { kn = silu_quick(kn); qn = silu_quick(qn); as[n] = a.head_decay[h]; }
    ks[n] = kn; qs[n] = qn * a.q_mult;
  }
  __syncthreads();
  if (FORM != FORM_HEAD) for (int n = tid; n < D; n += nthr) {
    const T *w = (const T *)a.wa2 + (size_t)(h * D + n) * a.rank;
    float z = 0.f;
    for (int j = 0; j < a.rank; ++j) z = fmaf(a1[j], to_f<T>(w[j]), z);
    as[n] = decay_of(z + a.zb[h * D + n], FORM == FORM_BONUS ? 0.f : a.inv_tau);
  }
  float own = 0.f;   // what the row's own value weighs in the read-out (the same sum in every wave)
  if (FORM == FORM_BONUS) {
    for (int n = tid & 63; n < D; n += 64) own = fmaf(a.bonus[h * D + n] * ks[n], qs[n], own);
    own = wave_sum(own);
  }
  __syncthreads();
  const bool carried = a.seq_pos0[s] > 0;
  float *st = a.state + ((size_t)a.seq_slot[s] * a.H + h) * D * Dv;
  const int cf = FORM == FORM_HEAD ? blockIdx.z * a.span : 0, ce = FORM == FORM_HEAD && cf + a.span < Dv ? cf + a.span : Dv;   // this workgroup's columns
  const int cols = (ce - cf + VP - 1) / VP, X = cols < nthr ? cols : nthr, Y = nthr / X, x = tid % X, y = tid / X;
  for (int cb = 0; cb < cols; cb += X) {
    const int c = cf + (cb + x) * VP;
    float o[VP], v[VP];
#pragma unroll
    for (int j = 0; j < VP; ++j) o[j] = 0.f;
    if (y < Y && cb + x < cols) {
#pragma unroll
      for (int j = 0; j < VP; ++j) {
        v[j] = ur[h * Dv + c + j];
        if (FORM == FORM_HEAD) v[j] = silu_quick(v[j]);
        if (FORM == FORM_BONUS && y == 0) o[j] = own * v[j];
      }
#pragma unroll 4
      for (int n = y; n < D; n += Y) {
        float *sp = st + (size_t)n * Dv + c, S[VP];
        if (VP == 4) {
          const float4 s4 = carried ? *(const float4 *)sp : make_float4(0.f, 0.f, 0.f, 0.f);
          S[0] = s4.x; S[VP > 1 ? 1 : 0] = s4.y; S[VP > 2 ? 2 : 0] = s4.z; S[VP > 3 ? 3 : 0] = s4.w;
        } else {
          S[0] = carried ? *sp : 0.f;
        }
        const float kn = ks[n], qn = qs[n], an = as[n];
#pragma unroll
        for (int j = 0; j < VP; ++j) {
          if (FORM == FORM_BONUS) o[j] = fmaf(S[j], qn, o[j]);
          S[j] = fmaf(an, S[j], kn * v[j]);
          if (FORM != FORM_BONUS) o[j] = fmaf(S[j], qn, o[j]);
        }
        if (VP == 4) *(float4 *)sp = make_float4(S[0], S[VP > 1 ? 1 : 0], S[VP > 2 ? 2 : 0], S[VP > 3 ? 3 : 0]);
        else *sp = S[0];
      }
    }
    __syncthreads();   // the previous column block's parts have been read
    if (y < Y)
#pragma unroll
      for (int j = 0; j < VP; ++j) parts[(y * X + x) * VP + j] = o[j];
    __syncthreads();
    for (int e = tid; e < X * VP; e += nthr) {
      if (cf + cb * VP + e >= ce) continue;
      float sum = 0.f;
      for (int q = 0; q < Y; ++q) sum += parts[q * X * VP + e];
      os[cf + cb * VP + e] = sum;
    }
  }
  __syncthreads();
  if (FORM == FORM_HEAD) {
    for (int d = cf + tid; d < ce; d += nthr) a.out32[((size_t)t * a.H + h) * Dv + d] = os[d];
    return;
  }
  float ss = 0.f;
  for (int d = tid; d < Dv; d += nthr) ss = fmaf(os[d], os[d], ss);
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  float tot = 0.f;
  for (int w = 0; w < (nthr >> 6); ++w) tot += red[w];
  const float inv = 1.0f / sqrtf(tot / (float)Dv + a.eps);
  for (int d = tid; d < Dv; d += nthr) ((T *)a.out)[((size_t)t * a.H + h) * Dv + d] = from_f<T>(os[d] * inv * a.norm[(FORM == FORM_BONUS ? h * Dv : 0) + d] * silu_f(ur[a.g_col + h * Dv + d]));
}

// Time mixing's operands: out[m][t] = h_t + (h_(t-1) - h_t) mu[m] rounded to T, m = 0 .. n - 1, h_(t-1) the row before (the slot's row at an entry's start, zeros at position 0).
// The workgroups of an entry's first row are the only readers of its slot; they leave the entry's last row there (h itself holds it already).
template <class T> __global__ void __launch_bounds__(256) token_shift_kernel(const float *__restrict__ h, const float *__restrict__ mu, float *__restrict__ state, T *__restrict__ out,
                                                                             const int *__restrict__ tok_seq, const int *__restrict__ seq_start, const int *__restrict__ seq_pos0,
                                                                             const int *__restrict__ seq_slot, int rows, int W, int n) {
  const int t = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  if (c >= W) return;
  const int s = tok_seq[t], r0 = seq_start[s];
  const float cur = h[(size_t)t * W + c];
  float prev;
  if (t == r0) {
    float *st = state + (size_t)seq_slot[s] * W + c;
    prev = seq_pos0[s] > 0 ? *st : 0.f;
    *st = h[(size_t)(seq_start[s + 1] - 1) * W + c];
  } else {
    prev = h[(size_t)(t - 1) * W + c];
  }
  const float d = prev - cur;
  for (int m = 0; m < n; ++m) out[((size_t)m * rows + t) * W + c] = from_f<T>(fmaf(d, mu[(size_t)m * W + c], cur));
}
// out = tanh(x) rounded to T
template <class T> __global__ void __launch_bounds__(256) tanh_round_kernel(const float *__restrict__ x, T *__restrict__ out, size_t n) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) out[i] = from_f<T>(tanhf(x[i]));
}

}  // namespace hybl
}  // namespace mrs

using namespace mrs::hybl;
#define S_(s) ((hipStream_t)(s))

extern "C" const char *mrs_hyb_linattn_last_error() { return g_err; }

/* z [rows, n] -> sigmoid(z + b [n])^inv_tau, in place; inv_tau 0: exp(-exp(z + b)) */
extern "C" int mrs_hyb_gla_decays(float *z, const float *b, int rows, int n, float inv_tau, void *stream) {
  const size_t total = (size_t)rows * n;
  if (rows <= 0 || n <= 0) return 0;
  if (n % 4 == 0 && ((uintptr_t)z % 16) == 0) hipLaunchKernelGGL(gla_decays_kernel<4>, dim3((unsigned)((total / 4 + 255) / 256)), dim3(256), 0, S_(stream), z, b, n, total, inv_tau);
  else hipLaunchKernelGGL(gla_decays_kernel<1>, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, S_(stream), z, b, n, total, inv_tau);
  return ok_or("mrs_hyb_gla_decays");
}
/* form 0: one decay per head and key channel (`dec`), 1: the same with a bonus [H, D] for the current row, 2: one decay per head (head_decay [H]) and SiLU operands.
 * u [rows, ldu] = v [H * Dv] | ... with k [H * D] at k_col and q [H * D] at q_col; dec [rows, H * D] the decays.
 * Segment table as for the other scans; carry [segments, H, D, Dv] and decay [segments, H, D] are scratch, needed when segments > entries. */
static int scan_launch(int form, const float *bonus, const float *head_decay, const float *u, int ldu, int k_col, int q_col, const float *dec, float *state, float *out, const int *seq_pos0, const int *seq_slot,
                                const int *seg_entry, const int *seg_row0, const int *seg_len, const int *ent_seg0, float *carry, float *decay, int rows, int entries, int segments,
                                int H, int D, int Dv, float q_mult, void *stream) {
  if (rows <= 0 || entries <= 0 || segments <= 0) return 0;
  if (H <= 0 || D <= 0 || Dv <= 0 || D > 512) return fail("mrs_hyb_gla_scan: head sizes (key size 1 .. 512)");
  if (entries > 65535 || segments > 65535 || H > 65535) return fail("mrs_hyb_gla_scan: more than 65535 entries, segments or heads");
  if (k_col < H * Dv || q_col < H * Dv || ldu < k_col + H * D || ldu < q_col + H * D) return fail("mrs_hyb_gla_scan: rows shorter than v | k | q");
  if (segments > entries && (!carry || !decay)) return fail("mrs_hyb_gla_scan: segmented entries need the carry scratch");
  GlaArgs a{u, dec, state, out, seq_pos0, seq_slot, seg_entry, seg_row0, seg_len, ent_seg0, carry, decay, ldu, k_col, q_col, H, D, Dv, q_mult, bonus, head_decay};
  const int vec = (ldu % 4 == 0 && k_col % 4 == 0 && q_col % 4 == 0 && D % 4 == 0 && Dv % 4 == 0 && ((uintptr_t)u % 16) == 0 && ((uintptr_t)dec % 16) == 0 &&
                   ((uintptr_t)state % 16) == 0 && ((uintptr_t)out % 16) == 0 && ((uintptr_t)carry % 16) == 0) ? 1 : 0;
  int R, J;
  if (D <= 32) { R = 4; J = 2; } else if (D <= 64) { R = 8; J = 2; } else if (D <= 128) { R = 16; J = 2; } else if (D <= 256) { R = 16; J = 4; } else { R = 16; J = 8; }
  const int Dp = 4 * R * J, NO = form == FORM_HEAD ? 2 : 3, CW = 64 / R * 4, all = (Dv + CW - 1) / CW;
  // waves: a head's columns in workgroups of at most 16 waves (8 for the large register tiles), and enough of them that two rows fit a stage (4 groups of four values per thread)
  const int most = J >= 4 ? 8 : 16;
  int nblk = (all + most - 1) / most, nw = (all + nblk - 1) / nblk;
  while (nw < most && 2 * (NO * Dp + nw * CW) / 4 > 4 * 64 * nw) ++nw;
  const int U = (NO * Dp + nw * CW) / 4;
  int TC = 4 * 64 * nw / U;
  TC = TC > 16 ? 16 : TC;
  while (TC > 1 && (size_t)2 * TC * U * 16 > 65536) --TC;
  const size_t lds = (size_t)2 * TC * U * 16;
  if ((long long)rows * ldu > 0x7fffffffLL) return fail("mrs_hyb_gla_scan: more than 2^31 projected values in one step");
  if (TC < 1 || lds > 65536) return fail("mrs_hyb_gla_scan: a row of operands does not fit the staging registers / 64 KB of LDS");
  dim3 grid(nblk, H, segments), block(64 * nw);
#define MRS_GLA__(R_, J_, L_, NT_, F_) hipLaunchKernelGGL((gla_scan_kernel<R_, J_, L_, NT_, F_>), grid, block, lds, S_(stream), a, TC, vec)
#define MRS_GLA_(R_, J_, L_, MOST_, F_) do { if (nw <= 4) MRS_GLA__(R_, J_, L_, 256, F_); else if (nw <= 8) MRS_GLA__(R_, J_, L_, 512, F_); else MRS_GLA__(R_, J_, L_, MOST_, F_); } while (0)
#define MRS_GLAF(L_, F_) do { if (D <= 32) MRS_GLA_(4, 2, L_, 1024, F_); else if (D <= 64) MRS_GLA_(8, 2, L_, 1024, F_); else if (D <= 128) MRS_GLA_(16, 2, L_, 1024, F_); \
                              else if (D <= 256) MRS_GLA_(16, 4, L_, 512, F_); else MRS_GLA_(16, 8, L_, 512, F_); } while (0)
#define MRS_GLA(L_) do { if (form == FORM_CHANNEL) MRS_GLAF(L_, FORM_CHANNEL); else if (form == FORM_BONUS) MRS_GLAF(L_, FORM_BONUS); else MRS_GLAF(L_, FORM_HEAD); } while (0)
  if (segments > entries) {
    MRS_GLA(true);
    hipLaunchKernelGGL(gla_carry_kernel, dim3((unsigned)(((size_t)D * Dv + 255) / 256), H, entries), dim3(256), 0, S_(stream), a);
  }
  MRS_GLA(false);
#undef MRS_GLA
#undef MRS_GLAF
#undef MRS_GLA_
#undef MRS_GLA__
  return ok_or("mrs_hyb_gla_scan");
}

extern "C" int mrs_hyb_gla_scan(const float *u, int ldu, int k_col, int q_col, const float *dec, float *state, float *out, const int *seq_pos0, const int *seq_slot,
                                const int *seg_entry, const int *seg_row0, const int *seg_len, const int *ent_seg0, float *carry, float *decay, int rows, int entries, int segments,
                                int H, int D, int Dv, float q_mult, void *stream) {
  return scan_launch(FORM_CHANNEL, nullptr, nullptr, u, ldu, k_col, q_col, dec, state, out, seq_pos0, seq_slot, seg_entry, seg_row0, seg_len, ent_seg0, carry, decay, rows, entries,
                     segments, H, D, Dv, q_mult, stream);
}
extern "C" int mrs_hyb_bonus_scan(const float *u, int ldu, int k_col, int q_col, const float *dec, const float *bonus, float *state, float *out, const int *seq_pos0,
                                  const int *seq_slot, const int *seg_entry, const int *seg_row0, const int *seg_len, const int *ent_seg0, float *carry, float *decay, int rows,
                                  int entries, int segments, int H, int D, int Dv, void *stream) {
  if (!bonus || !dec) return fail("mrs_hyb_bonus_scan: the rows' decays and the heads' bonus are needed");
  return scan_launch(FORM_BONUS, bonus, nullptr, u, ldu, k_col, q_col, dec, state, out, seq_pos0, seq_slot, seg_entry, seg_row0, seg_len, ent_seg0, carry, decay, rows, entries,
                     segments, H, D, Dv, 1.0f, stream);
}
extern "C" int mrs_hyb_lightning_scan(const float *u, int ldu, int k_col, int q_col, const float *head_decay, float *state, float *out, const int *seq_pos0, const int *seq_slot,
                                      const int *seg_entry, const int *seg_row0, const int *seg_len, const int *ent_seg0, float *carry, float *decay, int rows, int entries,
                                      int segments, int H, int D, int Dv, void *stream) {
  if (!head_decay) return fail("mrs_hyb_lightning_scan: the heads' decays are needed");
  return scan_launch(FORM_HEAD, nullptr, head_decay, u, ldu, k_col, q_col, nullptr, state, out, seq_pos0, seq_slot, seg_entry, seg_row0, seg_len, ent_seg0, carry, decay, rows,
                     entries, segments, H, D, Dv, 1.0f, stream);
}

// (what all single-row forms check and launch; `a` complete but for nothing)
static int step_launch(int form, const GlaStepArgs &a, int rows, int entries, int dtype, void *stream) {
  if (rows <= 0) return 0;
  const int H = a.H, D = a.D, Dv = a.Dv;
  if (rows != entries || entries > 65535) return fail("mrs_hyb_gla_step: one row per entry");
  if (H <= 0 || H > 65535 || D <= 0 || Dv <= 0 || (form != FORM_HEAD && a.rank <= 0)) return fail("mrs_hyb_gla_step: head sizes / decay rank");
  if (a.k_col < H * Dv || a.ldu < a.k_col + H * D || a.ldu < a.q_col + H * D || (form != FORM_HEAD && a.ldu < a.g_col + H * Dv) || (form != FORM_HEAD && !a.a1 && a.ldu < a.a1_col + a.rank))
    return fail("mrs_hyb_gla_step: rows shorter than their columns");
  if (dtype != 1 && dtype != 2) return fail("mrs_hyb_gla_step: dtype");
  const bool v4 = Dv % 4 == 0 && ((uintptr_t)a.state % 16) == 0;
  const int VP = v4 ? 4 : 1, cols = (form == FORM_HEAD ? (a.span < Dv ? a.span : Dv) : Dv) / VP;
  // threads: at most eight state rows each where a head has that many, whole waves
  long long want = (long long)cols * ((D + 7) / 8);
  int nthr = want > 1024 ? 1024 : (int)((want + 63) / 64 * 64);
  if (nthr < 64) nthr = 64;
  const int X = cols < nthr ? cols : nthr, Y = nthr / X;
  const size_t lds = (size_t)(3 * ((D + 3) & ~3) + ((a.rank + 3) & ~3) + ((Dv + 3) & ~3) + Y * X * VP) * 4;
  if (lds > 65536 - 128) return fail("mrs_hyb_gla_step: the head does not fit 64 KB of LDS");
  dim3 grid(entries, H, form == FORM_HEAD ? (Dv + a.span - 1) / a.span : 1);
#define MRS_GLAS_(T, V_) do { if (form == FORM_CHANNEL) hipLaunchKernelGGL((gla_step_kernel<T, V_, FORM_CHANNEL>), grid, dim3(nthr), lds, S_(stream), a); \
                              else if (form == FORM_BONUS) hipLaunchKernelGGL((gla_step_kernel<T, V_, FORM_BONUS>), grid, dim3(nthr), lds, S_(stream), a); \
                              else hipLaunchKernelGGL((gla_step_kernel<T, V_, FORM_HEAD>), grid, dim3(nthr), lds, S_(stream), a); } while (0)
#define MRS_GLAS(T) do { if (v4) MRS_GLAS_(T, 4); else MRS_GLAS_(T, 1); } while (0)
  if (dtype == 1) MRS_GLAS(mrs::bf16_t);
  else MRS_GLAS(float);
#undef MRS_GLAS
#undef MRS_GLAS_
  return ok_or("mrs_hyb_gla_step");
}
/* steps of single rows (rows == entries): u also holds the output gate [H * Dv] at g_col and the decay projection's first step [rank] at a1_col; wa2 [H * D, rank] (dtype);
 * out (dtype) [rows, H * Dv] = o / rms(o) per head * norm [Dv] * silu(gate) */
extern "C" int mrs_hyb_gla_step(const float *u, int ldu, int k_col, int q_col, int g_col, int a1_col, int rank, const void *wa2, const float *zb, const float *norm, float *state,
                                void *out, const int *seq_start, const int *seq_pos0, const int *seq_slot, int rows, int entries, int H, int D, int Dv, float q_mult, float inv_tau,
                                float eps, int dtype, void *stream) {
  const GlaStepArgs a{u, wa2, zb, norm, state, seq_start, seq_pos0, seq_slot, out, ldu, k_col, q_col, g_col, a1_col, rank, H, D, Dv, q_mult, inv_tau, eps, nullptr, nullptr, nullptr, nullptr, 0};
  return step_launch(FORM_CHANNEL, a, rows, entries, dtype, stream);
}
/* the same with a1 [rows, rank] in rows of its own (tanh is taken here), decays exp(-exp(W a1 + zb)), the bonus [H, D] and a norm weight of [H * Dv] */
extern "C" int mrs_hyb_bonus_step(const float *u, int ldu, int k_col, int q_col, int g_col, const float *a1, int rank, const void *wa2, const float *zb, const float *bonus,
                                  const float *norm, float *state, void *out, const int *seq_start, const int *seq_pos0, const int *seq_slot, int rows, int entries, int H, int D,
                                  int Dv, float eps, int dtype, void *stream) {
  if (!a1 || !bonus) return fail("mrs_hyb_bonus_step: the decay projection's first step and the bonus are needed");
  const GlaStepArgs a{u, wa2, zb, norm, state, seq_start, seq_pos0, seq_slot, out, ldu, k_col, q_col, g_col, 0, rank, H, D, Dv, 1.0f, 0.f, eps, a1, bonus, nullptr, nullptr, 0};
  return step_launch(FORM_BONUS, a, rows, entries, dtype, stream);
}
/* single rows with one decay per head and SiLU operands: out (f32) [rows, H * Dv], no norm and no gate */
extern "C" int mrs_hyb_lightning_step(const float *u, int ldu, int k_col, int q_col, const float *head_decay, float *state, float *out, const int *seq_start, const int *seq_pos0,
                                      const int *seq_slot, int rows, int entries, int H, int D, int Dv, void *stream) {
  if (!head_decay) return fail("mrs_hyb_lightning_step: the heads' decays are needed");
  const GlaStepArgs a{u, nullptr, nullptr, nullptr, state, seq_start, seq_pos0, seq_slot, nullptr, ldu, k_col, q_col, 0, 0, 0, H, D, Dv, 1.0f, 0.f, 0.f, nullptr, nullptr, head_decay, out, 32};
  return step_launch(FORM_HEAD, a, rows, entries, 2, stream);
}

/* out [n, rows, W] (dtype): the n mixes of every row of h [rows, W] f32 with the row before it (mu [n, W]); state [slots, W] f32 holds the last row of what came before */
extern "C" int mrs_hyb_token_shift(const float *h, const float *mu, float *state, void *out, const int *tok_seq, const int *seq_start, const int *seq_pos0, const int *seq_slot, int rows,
                                   int W, int n, int dtype, void *stream) {
  if (rows <= 0 || W <= 0 || n <= 0) return 0;
  dim3 grid(rows, (W + 255) / 256);
  if (grid.y > 65535) return fail("mrs_hyb_token_shift: row width");
  if (dtype == 1) hipLaunchKernelGGL(token_shift_kernel<mrs::bf16_t>, grid, dim3(256), 0, S_(stream), h, mu, state, (mrs::bf16_t *)out, tok_seq, seq_start, seq_pos0, seq_slot, rows, W, n);
  else if (dtype == 2) hipLaunchKernelGGL(token_shift_kernel<float>, grid, dim3(256), 0, S_(stream), h, mu, state, (float *)out, tok_seq, seq_start, seq_pos0, seq_slot, rows, W, n);
  else return fail("mrs_hyb_token_shift: dtype");
  return ok_or("mrs_hyb_token_shift");
}
/* out (dtype) = tanh(x), n values */
extern "C" int mrs_hyb_tanh_round(const float *x, void *out, int rows, int cols, int dtype, void *stream) {
  const size_t n = (size_t)rows * cols;
  if (rows <= 0 || cols <= 0) return 0;
  const dim3 grid((unsigned)((n + 255) / 256));
  if (dtype == 1) hipLaunchKernelGGL(tanh_round_kernel<mrs::bf16_t>, grid, dim3(256), 0, S_(stream), x, (mrs::bf16_t *)out, n);
  else if (dtype == 2) hipLaunchKernelGGL(tanh_round_kernel<float>, grid, dim3(256), 0, S_(stream), x, (float *)out, n);
  else return fail("mrs_hyb_tanh_round: dtype");
  return ok_or("mrs_hyb_tanh_round");
}
