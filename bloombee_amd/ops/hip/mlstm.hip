// Matrix memory with exponential gates (mLSTM) over ragged batches: per head a
// 32-bit state S (dim x vdim), a normalizer n (dim) and a running maximum m, and
// for every token, with log gates i and f (one of each per head),
//     m' = max(f + m, i),  S <- e^(f + m - m') S + e^(i - m') k v^T,
//     n <- e^(f + m - m') n + e^(i - m') k,
//     o = S^T q / (max(|n . q|, e^-m') + 1e-6)
// then o RMS-normed over vdim, times the norm weight and sigmoid of the output
// gate. i = cap tanh(z / cap), f = log sigmoid(cap tanh(z / cap)). A sequence
// whose portion starts at position 0 starts from zero, whatever its slot holds.
//
//  mlstm_step_kernel   token by token, everything fused: decoded tokens, and any
//                      sizes and types.
//  mlstm_gates_kernel  prompts in chunks of C = 64 tokens, a wave each: with b the
//                      cumulated f, a = i - b and g the running maximum of a, so
//                      that m_t = b_t + M_t, M_t = max(m_0, g_t)
//  mlstm_scan_kernel   chunk after chunk, a slice of value columns each: leaves S
//                      and n for the chunk, then
//                      S <- e^(m_0 - M) S + k^T (e^(a - M) v),  M = M_last.
//                      n is the state's column of a value that is always one.
//  mlstm_out_kernel    all chunks side by side:
//                        A[t][s] = (q_t . k_s) e^(a_s - M_t)     (s <= t)
//                        o = (A v + e^(m_0 - M_t) q S) / den, norm and gate
//
// Every exponent of the chunk form is <= 0. Chunk products run on bf16 MFMAs with
// weighted operands and states split into two bf16 (the value and what its
// rounding lost). Exponents are in units of log 2 inside.

#pragma once
#include "common.h"
#include "rows.hip"
#include "latent.hip"
#include "gla.hip"

static constexpr float MLSTM_FLOOR = 1e-6f;
static constexpr int MLSTM_C = 64;

// cap * tanh(z / cap)
DEVINL float soft_cap(float z, float cap) { return cap * tanhf(z / cap); }
DEVINL float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

struct MlstmArgs {
  Parts y;            // q, k, v, output gate columns
  Parts g;            // f32; i_off: first of H input gates, then H forget gates
  const float* gb;    // (2 H,) their biases
  const float* nw;    // (H * vdim,)
  float* S;           // (slots, H, dim, vdim)
  float* n;           // (slots, H, dim)
  float* m;           // (slots, H)
  void* out;          // row stride ldo, H * vdim columns
  const int* slots;   // (S,)
  const int* tok_pos;
  const int* cu;
  const int* list;
  long ldo;
  int q_off, k_off, v_off, g_off, i_off, H, dim, vdim;
  float qscale, cap, eps;
};

// grid (H, listed sequences). LDS: q, k (dim each), partial sums (B * V), v, o
// (vdim each).
template <typename TP, typename T, int V, int B>
__global__ __launch_bounds__(B) void mlstm_step_kernel(MlstmArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds_mem[];
  __shared__ float red[B / WAVE], red2[B / WAVE];
  const int h = blockIdx.x, s = a.list[blockIdx.y], tid = threadIdx.x;
  float* qs = lds_mem;
  float* ks = qs + a.dim;
  float* part = lds_mem + ((2 * a.dim + 3) & ~3);
  float* vs = part + B * V;
  float* os = vs + ((a.vdim + 3) & ~3);
  const int VQ = a.vdim / V, CW = min(VQ, B), RG = B / CW;
  const int rg = tid / CW, cq = tid % CW;
  const int t0 = a.cu[s], t1 = a.cu[s + 1];
  const long head = (long)a.slots[s] * a.H + h;
  float* S = a.S + head * a.dim * a.vdim;
  float* n = a.n + head * a.dim;
  const float bi = a.gb[h], bf = a.gb[a.H + h];
  float m = 0.f;
  bool any = false;
  for (int t = t0; t < t1; ++t) {
    const int pos = a.tok_pos[t];
    if (pos < 0) continue;  // empty slot
    if (!any && pos > 0) m = a.m[head];
    any = true;
    float zi[1], zf[1];
    fold_parts<float, 1>(a.g, t, a.i_off + h, zi);
    fold_parts<float, 1>(a.g, t, a.i_off + a.H + h, zf);
    const float li = soft_cap(zi[0] + bi, a.cap);
    const float lf = log_sigmoid(soft_cap(zf[0] + bf, a.cap));
    const float mn = fmaxf(lf + m, li);
    const float keep = expf(lf + m - mn), add = expf(li - mn);
    m = mn;
    __syncthreads();
    float dot = 0.f;
    for (int d = tid; d < a.dim; d += B) {
      float v[1];
      const int c = h * a.dim + d;
      fold_parts<TP, 1>(a.y, t, a.q_off + c, v);
      const float q = v[0] * a.qscale;
      fold_parts<TP, 1>(a.y, t, a.k_off + c, v);
      const float nn = (pos > 0 ? n[d] * keep : 0.f) + add * v[0];
      n[d] = nn;
      dot += nn * q;
      qs[d] = q;
      ks[d] = add * v[0];
    }
    dot = wave_reduce_sum(dot);
    if ((tid & (WAVE - 1)) == 0) red2[tid / WAVE] = dot;
    for (int i = tid; i < a.vdim; i += B)
      fold_parts<TP, 1>(a.y, t, a.v_off + h * a.vdim + i, vs + i);
    __syncthreads();
    dot = 0.f;
#pragma unroll
    for (int i = 0; i < B / WAVE; ++i) dot += red2[i];
    const float den = 1.f / (fmaxf(fabsf(dot), expf(-m)) + MLSTM_FLOOR);
    for (int cb = 0; cb < VQ; cb += CW) {
      const int c = (cb + cq) * V;
      float o[V];
#pragma unroll
      for (int j = 0; j < V; ++j) o[j] = 0.f;
      if (rg < RG && c < a.vdim) {
        float vv[V];
#pragma unroll
        for (int j = 0; j < V; ++j) vv[j] = vs[c + j];
#pragma unroll 8
        for (int d = rg; d < a.dim; d += RG) {
          float x[V];
          float* p = S + (long)d * a.vdim + c;
          if (pos > 0) {
            ldv<V>(p, x);
          } else {
#pragma unroll
            for (int j = 0; j < V; ++j) x[j] = 0.f;
          }
          const float kk = ks[d], qq = qs[d];
#pragma unroll
          for (int j = 0; j < V; ++j) {
            x[j] = keep * x[j] + kk * vv[j];
            o[j] += x[j] * qq;
          }
          stv<V>(p, x);
        }
      }
#pragma unroll
      for (int j = 0; j < V; ++j) part[tid * V + j] = o[j];
      __syncthreads();
      if (tid < CW && c < a.vdim) {
        for (int g = 1; g < RG; ++g)
#pragma unroll
          for (int j = 0; j < V; ++j) o[j] += part[(g * CW + tid) * V + j];
#pragma unroll
        for (int j = 0; j < V; ++j) os[c + j] = o[j] * den;
      }
      __syncthreads();
    }
    float ss = 0.f;
    for (int i = tid; i < a.vdim; i += B) ss += os[i] * os[i];
    ss = wave_reduce_sum(ss);
    if ((tid & (WAVE - 1)) == 0) red[tid / WAVE] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < B / WAVE; ++i) ss += red[i];
    const float inv = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
    T* op = (T*)a.out + t * a.ldo + h * a.vdim;
    for (int i = tid; i < a.vdim; i += B) {
      float g[1];
      const int c = h * a.vdim + i;
      fold_parts<TP, 1>(a.y, t, a.g_off + c, g);
      stf(op + i, os[i] * inv * a.nw[c] * sigmoid_f(g[0]));
    }
  }
  if (any && tid == 0) a.m[head] = m;
}

struct MlstmChunkArgs {
  const unsigned short* y;  // (N, ldy) bf16
  const float* g;           // (N, ldg), i_off
  const float* gb;
  const float* nw;
  float* St;                // states, as MlstmArgs
  float* n;
  float* m;
  const float* mprev;       // (S, H): m before the step, sequence by sequence
  float* b;                 // (chunks, H, 3, C): b, a, g in units of log 2
  float* m0;                // (chunks, H): m before the chunk, the same units
  float* n0;                // (chunks, H, DP): n before the chunk
  unsigned short* S;        // (chunks, H, VT, 2, DP / 32, 64, 8): fragments of
                            // the state before each chunk, high and low part
  unsigned short* out;      // (N, ldo)
  const int* row0;          // (chunks,) first row
  const int* len;           // (chunks,) tokens
  const int* ccu;           // (listed + 1,) first chunk of each sequence
  const int* list;
  const int* slots;
  const int* q_start;
  long ldo;
  int ldy, ldg, q_off, k_off, v_off, g_off, i_off, H, dim, vdim, VT;
  float qscale, cap, eps;
};

// grid (chunks, H), one wave, a token a lane
__global__ __launch_bounds__(64) void mlstm_gates_kernel(MlstmChunkArgs a) {
  const int ch = blockIdx.x, h = blockIdx.y, t = threadIdx.x;
  float li = NEG_BIG, lf = 0.f;
  if (t < a.len[ch]) {
    const float* g = a.g + (a.row0[ch] + t) * (long)a.ldg + a.i_off + h;
    li = soft_cap(g[0] + a.gb[h], a.cap) * LOG2E;
    lf = log_sigmoid(soft_cap(g[a.H] + a.gb[a.H + h], a.cap)) * LOG2E;
  }
  float b = lf;
#pragma unroll
  for (int d = 1; d < WAVE; d <<= 1) {
    const float o = __shfl_up(b, d);
    if (t >= d) b += o;
  }
  const float as = li - b;
  float g = as;
#pragma unroll
  for (int d = 1; d < WAVE; d <<= 1) {
    const float o = __shfl_up(g, d);
    if (t >= d) g = fmaxf(g, o);
  }
  float* p = a.b + ((long)ch * a.H + h) * 3 * MLSTM_C + t;
  p[0] = b;
  p[MLSTM_C] = as;
  p[2 * MLSTM_C] = g;
}

// grid ((vdim + 1) / 64, H, listed sequences); a wave owns 16 value columns and
// the state's whole column. The state's accumulators hold rows in the order
//     tile 2g + n, row x*4 + y  <->  channel g*32 + x*8 + n*4 + y
// so that a lane's registers of two tiles are eight consecutive channels: an
// operand fragment as it is. Column vdim is n.
template <int DP, bool VEC>
__global__ __launch_bounds__(256) void mlstm_scan_kernel(MlstmChunkArgs a) {
  constexpr int C = MLSTM_C, NG = DP / 32, NC = C / 32;
  // rows 16 banks apart (mod 64): the permuted column reads do not collide
  constexpr int LDD = DP == 32 ? 96 : DP + 32, LDV = 64 + 8;
  constexpr int PD = C * DP / 8 / 256;   // 16 B pieces a thread
  constexpr int PV = C * 64 / 8 / 256;
  constexpr int BUF = C * LDD + 2 * C * LDV;  // 16-bit elements
  static_assert(PD >= 1 && PV >= 1, "chunk smaller than the workgroup");
  extern __shared__ __attribute__((aligned(16))) unsigned short lds_ms[];
  const int h = blockIdx.y, i = blockIdx.z, s = a.list[i], tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int v0 = blockIdx.x * 64, vt = blockIdx.x * 4 + wave;
  const int col = v0 + wave * 16 + li;
  const bool live = col < a.vdim, norm = col == a.vdim;
  const long head = (long)a.slots[s] * a.H + h;
  // n is a column of stride one
  float* S = norm ? a.n + head * a.dim
                  : a.St + head * a.dim * a.vdim + min(col, a.vdim - 1);
  const long rs = norm ? 1 : a.vdim;

  f32x4 acc[2 * NG];
  const bool started = a.q_start[s] != 0;
  const bool kept = started && (live || norm);
#pragma unroll
  for (int n = 0; n < 2 * NG; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc[n][r] = S[min((n >> 1) * 32 + hi * 8 + (n & 1) * 4 + r, a.dim - 1) * rs];
  // all loads first, then the choice: else each waits behind a branch
  __builtin_amdgcn_sched_barrier(0);
#pragma unroll
  for (int n = 0; n < 2 * NG; ++n) asm volatile("" : "+v"(acc[n]));
#pragma unroll
  for (int n = 0; n < 2 * NG; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (!kept || (n >> 1) * 32 + hi * 8 + (n & 1) * 4 + r >= a.dim)
        acc[n][r] = 0.f;

  const int c0 = a.ccu[i], c1 = a.ccu[i + 1];
  if (c0 >= c1) return;
  // a sequence's chunks lie one after the other
  const long first = a.row0[c0];
  const int total = (c1 - c0 - 1) * C + a.len[c1 - 1];

  short8 rk[PD], rv[PV];
  float ra[PV], rb = 0.f, rg = 0.f;
  auto fetch = [&](int ch) {
    const long row0 = first + (long)(ch - c0) * C;
    const int len = min(C, total - (ch - c0) * C);
    const float* bp = a.b + ((long)ch * a.H + h) * 3 * C;
#pragma unroll
    for (int n = 0; n < PD; ++n) {
      const int idx = tid + n * 256, t = idx / (DP / 8);
      rk[n] = load_row8<VEC>(a.y + (row0 + min(t, len - 1)) * a.ldy + a.k_off +
                                 h * a.dim, idx % (DP / 8) * 8, a.dim, t < len);
    }
#pragma unroll
    for (int n = 0; n < PV; ++n) {
      const int idx = tid + n * 256, t = idx / 8;
      rv[n] = load_row8<VEC>(a.y + (row0 + min(t, len - 1)) * a.ldy + a.v_off +
                                 h * a.vdim, v0 + idx % 8 * 8, a.vdim, t < len);
      ra[n] = bp[C + t];
    }
    rb = bp[C - 1];
    rg = bp[3 * C - 1];
  };
  // m before the chunk to be staged, and the state's factor in the staged one.
  // All workgroups of a head follow m; one writes it (they read a copy).
  float mb = started ? a.mprev[(long)s * a.H + h] * LOG2E : 0.f, fac = 1.f;
  auto stage = [&](unsigned short* buf, int ch) {
    const float M = fmaxf(mb, rg);
    fac = fast_exp2(mb - M);
    if (blockIdx.x == 0 && tid == 0) a.m0[(long)ch * a.H + h] = mb;
    mb = rb + M;
#pragma unroll
    for (int n = 0; n < PD; ++n) {
      const int idx = tid + n * 256;
      *reinterpret_cast<short8*>(buf + idx / (DP / 8) * LDD + idx % (DP / 8) * 8) =
          rk[n];
    }
    unsigned short* vb = buf + C * LDD;
#pragma unroll
    for (int n = 0; n < PV; ++n) {
      const int idx = tid + n * 256, c = v0 + idx % 8 * 8;
      const float w = fast_exp2(ra[n] - M);
      float v[8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        v[j] = (c + j == a.vdim ? 1.f : bf2f((unsigned short)rv[n][j])) * w;
      short8 vh, vl;
      split8(v, vh, vl);
      unsigned short* p = vb + idx / 8 * LDV + idx % 8 * 8;
      *reinterpret_cast<short8*>(p) = vh;
      *reinterpret_cast<short8*>(p + C * LDV) = vl;
    }
  };

  fetch(c0);
  stage(lds_ms, c0);
  if (c0 + 1 < c1) fetch(c0 + 1);
  for (int ch = c0; ch < c1; ++ch) {
    const unsigned short* buf = lds_ms + ((ch - c0) & 1) * BUF;
    const float f = fac;
    __syncthreads();   // buf is written, the other one is read
    // registers hold the next chunk since an iteration ago
    if (ch + 1 < c1) stage(lds_ms + ((ch + 1 - c0) & 1) * BUF, ch + 1);
    if (ch + 2 < c1) fetch(ch + 2);
    // the state as it stands, for the chunk's outputs
    if (vt < a.VT) {
      unsigned short* sp =
          a.S + ((((long)ch * a.H + h) * a.VT + vt) * 2 * NG) * 512 + lane * 8;
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        float sv[8];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          sv[r] = live ? acc[2 * g][r] : 0.f;
          sv[4 + r] = live ? acc[2 * g + 1][r] : 0.f;
        }
        short8 sh, sl;
        split8(sv, sh, sl);
        *reinterpret_cast<short8*>(sp + g * 512) = sh;
        *reinterpret_cast<short8*>(sp + (NG + g) * 512) = sl;
      }
    }
    if (norm) {
      float* np = a.n0 + ((long)ch * a.H + h) * DP + hi * 8;
#pragma unroll
      for (int n = 0; n < 2 * NG; ++n)
        *reinterpret_cast<f32x4*>(np + (n >> 1) * 32 + (n & 1) * 4) = acc[n];
    }
    const unsigned short* vb = buf + C * LDD;
    bf16x8 vf[2][NC];
#pragma unroll
    for (int p = 0; p < 2; ++p)
#pragma unroll
      for (int k = 0; k < NC; ++k)
        vf[p][k] = column_frag(vb + p * C * LDV, LDV, k * 32,
                               wave * 16 + (li & 3) * 4, li, hi);
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int n = 0; n < 2; ++n) {
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[2 * g + n][r] *= f;
#pragma unroll
        for (int k = 0; k < NC; ++k) {
          const bf16x8 kf = column_frag(buf, LDD, k * 32,
                                        g * 32 + (li & 3) * 8 + n * 4, li, hi);
#pragma unroll
          for (int p = 0; p < 2; ++p)
            acc[2 * g + n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                kf, vf[p][k], acc[2 * g + n], 0, 0, 0);
        }
      }
  }
  if (live || norm) {
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = g * 32 + hi * 8 + n * 4 + r;
          if (d < a.dim) S[d * rs] = acc[2 * g + n][r];
        }
  }
  if (blockIdx.x == 0 && tid == 0) a.m[head] = mb / LOG2E;
}

// grid (chunks, H), eight waves; a wave owns every eighth tile of 16 value
// columns. Outputs are made transposed, o^T = S^T q^T + v^T A^T: a lane holds
// four consecutive columns of one token. LDS: k, later v; q; A.
template <int DP, int NCT, bool VEC>
__global__ __launch_bounds__(512) void mlstm_out_kernel(MlstmChunkArgs a) {
  constexpr int C = MLSTM_C, LDD = DP + 8, LDA = C + 8, NG = DP / 32;
  constexpr int NT = C / 16, NC = C / 32, NB = C / 16, VC = NCT * 128;
  constexpr int LDV = VC + 24;   // rows 12 banks apart, for column reads
  constexpr int FIRST = C * (LDD > LDV ? LDD : LDV);
  constexpr int PQ = C * DP / 8 / 512 > 0 ? C * DP / 8 / 512 : 1;
  constexpr int PV = C * VC / 8 / 512;
  // the states, too, are asked for ahead, where there are registers for them
  constexpr bool EARLY = VEC && NCT * NG <= 8;
  constexpr int NS = EARLY ? NCT : 1;
  extern __shared__ __attribute__((aligned(16))) unsigned short lds_mo[];
  __shared__ float ssum[8][C], rsum[NB][C], n0s[DP];
  __shared__ float as_[C], ms[C], ct[C], fl[C], dn[C];
  unsigned short* ks = lds_mo;               // (C, LDD)
  unsigned short* vs = lds_mo;               // (C, LDV)
  unsigned short* qs = lds_mo + FIRST;       // (C, LDD)
  unsigned short* As = qs + C * LDD;         // (2, C, LDA)
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const long row0 = a.row0[ch], base = (long)ch * a.H + h;
  const int len = a.len[ch];

  // everything that comes from memory is asked for up front
  short8 rq[PQ], rk[PQ], rv[PV];
  bf16x8 sh[NS][NG], sl[NS][NG];
  auto load_state = [&](int c, bf16x8 (&u)[NG], bf16x8 (&v)[NG]) {
    // waves beyond the last tile read that one again and drop what they make
    const int vt = min(c * 8 + wave, a.VT - 1);
    const unsigned short* sp = a.S + ((base * a.VT + vt) * 2 * NG) * 512 + lane * 8;
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      u[g] = as_bf16x8(*reinterpret_cast<const short8*>(sp + g * 512));
      v[g] = as_bf16x8(*reinterpret_cast<const short8*>(sp + (NG + g) * 512));
    }
  };
#pragma unroll
  for (int n = 0; n < PQ; ++n) {
    const int idx = min(tid + n * 512, C * DP / 8 - 1);
    const int t = idx / (DP / 8), d = idx % (DP / 8) * 8;
    const unsigned short* row = a.y + (row0 + min(t, len - 1)) * a.ldy + h * a.dim;
    rq[n] = load_row8<VEC>(row + a.q_off, d, a.dim, t < len);
    rk[n] = load_row8<VEC>(row + a.k_off, d, a.dim, t < len);
  }
#pragma unroll
  for (int n = 0; n < PV; ++n) {
    const int idx = tid + n * 512, t = idx / (VC / 8);
    rv[n] = load_row8<VEC>(a.y + (row0 + min(t, len - 1)) * a.ldy + a.v_off +
                               h * a.vdim, idx % (VC / 8) * 8, a.vdim, t < len);
  }
  if constexpr (EARLY) {
#pragma unroll
    for (int c = 0; c < NCT; ++c) load_state(c, sh[c], sl[c]);
  }
  if (tid < DP) n0s[tid] = a.n0[base * DP + tid];
  if (tid < C) {
    const float* bp = a.b + base * 3 * C + tid;
    const float m0 = a.m0[base], M = fmaxf(m0, bp[2 * C]);
    as_[tid] = bp[C];
    ms[tid] = M;
    ct[tid] = a.qscale * fast_exp2(m0 - M);   // of the state, query scale in it
    fl[tid] = fast_exp2(-(bp[0] + M));        // floor of the normalizer
  }
#pragma unroll
  for (int n = 0; n < PQ; ++n) {
    const int idx = tid + n * 512;
    if (idx >= C * DP / 8) continue;
    const int at = idx / (DP / 8) * LDD + idx % (DP / 8) * 8;
    *reinterpret_cast<short8*>(qs + at) = rq[n];
    *reinterpret_cast<short8*>(ks + at) = rk[n];
  }
  __syncthreads();
  for (int pair = wave; pair < NB * NB; pair += 8) {
    const int I = pair / NB, J = pair % NB;
    f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (J <= I && I * 16 < len) {
#pragma unroll
      for (int kk = 0; kk < NG; ++kk)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            as_bf16x8(*reinterpret_cast<const short8*>(
                qs + (I * 16 + li) * LDD + kk * 32 + hi * 8)),
            as_bf16x8(*reinterpret_cast<const short8*>(
                ks + (J * 16 + li) * LDD + kk * 32 + hi * 8)),
            acc, 0, 0, 0);
    }
    const int s = J * 16 + li;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = I * 16 + hi * 4 + r;
      const float v =
          s <= t ? acc[r] * a.qscale * fast_exp2(as_[s] - ms[t]) : 0.f;
      const unsigned short vh = cvt_bf(v);
      As[t * LDA + s] = vh;
      As[(C + t) * LDA + s] = cvt_bf(v - bf2f(vh));
      const float sum = group16_reduce_sum(v);
      if (li == 0) rsum[J][t] = sum;
    }
  }
  {
    // n_0 . q, eight threads a token
    const int t = tid / 8, p = tid % 8;
    float d = 0.f;
    for (int c = p * 8; c < DP; c += 64) {
      float q[8];
      load_bf16x8(qs + t * LDD + c, q);
#pragma unroll
      for (int j = 0; j < 8; ++j) d += q[j] * n0s[c + j];
    }
    d += __shfl_xor(d, 1);
    d += __shfl_xor(d, 2);
    d += __shfl_xor(d, 4);
    if (p == 0) dn[t] = d * ct[t];
  }
  __syncthreads();   // k is read
  if (tid < C) {
    float d = dn[tid];
#pragma unroll
    for (int j = 0; j < NB; ++j) d += rsum[j][tid];
    dn[tid] = 1.f / (fmaxf(fabsf(d), fl[tid]) + MLSTM_FLOOR);
  }
#pragma unroll
  for (int n = 0; n < PV; ++n) {
    const int idx = tid + n * 512;
    *reinterpret_cast<short8*>(vs + idx / (VC / 8) * LDV + idx % (VC / 8) * 8) = rv[n];
  }
  __syncthreads();

  // the states, then v: an operand that is read serves all of the wave's tiles
  f32x4 o[NCT][NT];
#pragma unroll
  for (int c = 0; c < NCT; ++c)
#pragma unroll
    for (int t = 0; t < NT; ++t) o[c][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int c0 = 0; c0 < NCT; c0 += NS) {
    if constexpr (!EARLY) load_state(c0, sh[0], sl[0]);
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const bf16x8 q = as_bf16x8(*reinterpret_cast<const short8*>(
            qs + (t * 16 + li) * LDD + g * 32 + hi * 8));
#pragma unroll
        for (int c = 0; c < NS; ++c) {
          f32x4& r = o[c0 + c][t];
          r = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sh[c][g], q, r, 0, 0, 0);
          r = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sl[c][g], q, r, 0, 0, 0);
        }
      }
  }
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const float f = ct[t * 16 + li];
#pragma unroll
    for (int c = 0; c < NCT; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) o[c][t][r] *= f;
  }
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    bf16x8 vf[NCT];
#pragma unroll
    for (int c = 0; c < NCT; ++c)
      vf[c] = column_frag(vs, LDV, k * 32, (c * 8 + wave) * 16 + (li & 3) * 4, li, hi);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if (k * 32 > t * 16 + 15) continue;  // above the diagonal
#pragma unroll
      for (int p = 0; p < 2; ++p) {
        const bf16x8 af = as_bf16x8(*reinterpret_cast<const short8*>(
            As + (p * C + t * 16 + li) * LDA + k * 32 + hi * 8));
#pragma unroll
        for (int c = 0; c < NCT; ++c)
          o[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[c], af, o[c][t], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NCT; ++c)
    if (c * 8 + wave >= a.VT)
#pragma unroll
      for (int t = 0; t < NT; ++t) o[c][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // columns beyond vdim are zero: they add nothing
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const float den = dn[t * 16 + li];
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < NCT; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        o[c][t][r] *= den;
        ss += o[c][t][r] * o[c][t][r];
      }
    ss += __shfl_xor(ss, 16);
    ss += __shfl_xor(ss, 32);
    if (hi == 0) ssum[wave][t * 16 + li] = ss;
  }
  __syncthreads();
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int tt = t * 16 + li;
    if (tt >= len) continue;
    float ss = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) ss += ssum[w][tt];
    const float inv = 1.f / sqrtf(ss / (float)a.vdim + a.eps);
    const unsigned short* gp = a.y + (row0 + tt) * a.ldy + a.g_off + h * a.vdim;
    const float* nw = a.nw + h * a.vdim;
    unsigned short* op = a.out + (row0 + tt) * a.ldo + h * a.vdim;
#pragma unroll
    for (int c = 0; c < NCT; ++c) {
      const int v0 = (c * 8 + wave) * 16 + hi * 4;
      if (v0 >= a.vdim) continue;
      if constexpr (VEC) {
        float g[4], w[4];
        ldv<4>(gp + v0, g);
        ldv<4>(nw + v0, w);
#pragma unroll
        for (int r = 0; r < 4; ++r) w[r] *= o[c][t][r] * inv * sigmoid_f(g[r]);
        stv<4>(op + v0, w);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (v0 + r >= a.vdim) continue;
          op[v0 + r] =
              cvt_bf(o[c][t][r] * inv * nw[v0 + r] * sigmoid_f(bf2f(gp[v0 + r])));
        }
      }
    }
  }
}
