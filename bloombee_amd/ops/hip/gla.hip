// Gated linear attention over ragged batches: per head a 32-bit state S
// (dim x vdim) and, for every token,
//     S <- diag(alpha) S + k v^T,   o = S^T q,
//     alpha = sigmoid(z)^(1/tau), z = W_a2 a1 + b per key channel,
// then o RMS-normed over vdim, times silu of the output gate. A sequence whose
// portion starts at position 0 starts from a zero state, whatever its slot
// holds.
//
// The same with a forget gate that also decides what is written (HGRN2; WRITES in
// the kernels): alpha = lower + (1 - lower) sigmoid(z + b) and k = 1 - alpha, z a
// projection in f32 like q, which passes through silu; no output gate.
//
//  gla_step_kernel   token by token, everything fused: decoded tokens, and any
//                    sizes and types.
//  gla_prep_kernel   prompts in chunks of C tokens, all chunks side by side:
//                    cumulated log decays b and kd = k 2^(b_last - b)
//  gla_scan_kernel   chunk after chunk, a slice of value columns each: leaves
//                    S for the chunk, then S <- 2^b_last S + kd^T v
//  gla_out_kernel    all chunks side by side:
//                       A[t][s] = sum_d q_t k_s 2^(b_t - b_s)   (s <= t)
//                       o = (q 2^b) S + A v, norm and gate
//  hgrn_prep_kernel  gla_prep_kernel for gates that write
//
// Chunk products run on bf16 MFMAs with decayed operands, weights and states
// split into two bf16 (the value and what its rounding lost). All exponents of
// the chunk form are <= 0 except inside a 16 x 16 diagonal block, which is
// computed pair by pair where its decays span too far.

#pragma once
#include "common.h"
#include "rows.hip"
#include "latent.hip"

// log2 of sigmoid(z), accurate on both sides
DEVINL float log2_sigmoid(float z) {
  const float e = fast_exp2(-fabsf(z) * LOG2E);
  // log(1 + e): the series where 1 + e would drop bits
  const float l = e < 0.01f ? (e - 0.5f * e * e + e * e * e * (1.f / 3)) * LOG2E
                            : __builtin_amdgcn_logf(1.f + e);
  return fminf(z, 0.f) * LOG2E - l;
}

// A forget gate in (lower, 1) and what it leaves room for, 1 - gate.
DEVINL float forget_room(float lower, float z) {
  return (1.f - lower) * sigmoid_f(-z);
}

// log2 of the gate, accurate where it is nearly one. A gate below 2^-64 forgets
// all there is.
DEVINL float log2_forget(float lower, float z, float room) {
  if (room < 0.01f)
    return -room * (1.f + room * (0.5f + room * (1.f / 3))) * LOG2E;
  return __builtin_amdgcn_logf(fmaxf(lower + (1.f - lower) * sigmoid_f(z), 5.4e-20f));
}

struct GlaArgs {
  Parts y;            // q, k, v, g columns; WRITES: q, v
  Parts a1;           // f32; a1_off: first column; WRITES: z
  const float* a2;    // (r, H * dim)
  const float* a2b;   // (H * dim,)
  const float* lower; // (H * dim,), WRITES
  const float* nw;    // (vdim,)
  float* state;       // (slots, H, dim, vdim)
  void* out;          // row stride ldo, H * vdim columns
  const int* slots;   // (S,)
  const int* tok_pos;
  const int* cu;
  const int* list;
  long ldo;
  int q_off, k_off, v_off, g_off, a1_off, r, H, dim, vdim;
  float qscale, inv_tau, eps;
};

// grid (H, listed sequences). LDS: q, k, alpha (dim each), partial sums
// (B * V), v, o (vdim each), a1 (r).
template <typename TP, typename T, int V, int B, bool WRITES = false>
__global__ __launch_bounds__(B) void gla_step_kernel(GlaArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds_gla[];
  __shared__ float red[B / WAVE];
  const int h = blockIdx.x, s = a.list[blockIdx.y], tid = threadIdx.x;
  float* qs = lds_gla;
  float* ks = qs + a.dim;
  float* as = ks + a.dim;
  float* part = lds_gla + ((3 * a.dim + 3) & ~3);
  float* vs = part + B * V;
  float* os = vs + ((a.vdim + 3) & ~3);
  float* a1s = os + ((a.vdim + 3) & ~3);
  const int VQ = a.vdim / V, CW = min(VQ, B), RG = B / CW;
  const int rg = tid / CW, cq = tid % CW;
  const int t0 = a.cu[s], t1 = a.cu[s + 1];
  float* S = a.state + ((long)a.slots[s] * a.H + h) * a.dim * a.vdim;
  for (int t = t0; t < t1; ++t) {
    const int pos = a.tok_pos[t];
    if (pos < 0) continue;  // empty slot
    __syncthreads();
    if constexpr (!WRITES) {
      for (int i = tid; i < a.r; i += B)
        fold_parts<float, 1>(a.a1, t, a.a1_off + i, a1s + i);
      __syncthreads();
    }
    for (int d = tid; d < a.dim; d += B) {
      float v[1];
      const int c = h * a.dim + d;
      fold_parts<TP, 1>(a.y, t, a.q_off + c, v);
      if constexpr (WRITES) {
        float z[1];
        fold_parts<float, 1>(a.a1, t, a.a1_off + c, z);
        z[0] += a.a2b[c];
        const float lo = a.lower[c];
        qs[d] = v[0] / (1.f + expf(-v[0]));
        ks[d] = (1.f - lo) / (1.f + expf(z[0]));
        as[d] = lo + (1.f - lo) / (1.f + expf(-z[0]));
        continue;
      }
      qs[d] = v[0] * a.qscale;
      fold_parts<TP, 1>(a.y, t, a.k_off + c, v);
      ks[d] = v[0];
      float z = a.a2b[c];
      for (int i = 0; i < a.r; ++i) z += a1s[i] * a.a2[(long)i * a.H * a.dim + c];
      const float ls = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
      as[d] = expf(ls * a.inv_tau);
    }
    for (int i = tid; i < a.vdim; i += B)
      fold_parts<TP, 1>(a.y, t, a.v_off + h * a.vdim + i, vs + i);
    __syncthreads();
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
          const float al = as[d], kk = ks[d], qq = qs[d];
#pragma unroll
          for (int j = 0; j < V; ++j) {
            x[j] = al * x[j] + kk * vv[j];
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
        for (int j = 0; j < V; ++j) os[c + j] = o[j];
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
      float v = os[i] * inv * a.nw[i];
      if constexpr (!WRITES) {
        float g[1];
        fold_parts<TP, 1>(a.y, t, a.g_off + h * a.vdim + i, g);
        v *= g[0] * sigmoid_f(g[0]);
      }
      stf(op + i, v);
    }
  }
}

struct GlaChunkArgs {
  const unsigned short* y;  // (N, ldy) bf16
  const float* a1;          // (N, ld1), a1_off; WRITES: z
  const float* a2;          // (r, H * dim)
  const float* a2b;
  const float* lower;       // (H * dim,), WRITES
  const float* nw;
  float* state;
  float* b;                 // (chunks, H, C, DP): cumulated log2 decays
  unsigned short* kd;       // (chunks, H, 2, C, DP): high and low part
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
  int ldy, ld1, q_off, k_off, v_off, g_off, a1_off, r, H, dim, vdim, VT;
  float qscale, inv_tau, eps;
};

DEVINL void split8(const float* v, short8& hi, short8& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const __bf16 h = (__bf16)v[j];
    hi[j] = __builtin_bit_cast(short, h);
    lo[j] = __builtin_bit_cast(short, (__bf16)(v[j] - (float)h));
  }
}

// Eight columns c.. of a head of n columns in row `row`, zero where !live and
// beyond n. VEC: n is a multiple of 8 and rows are aligned. Addresses are
// clamped, so that nothing branches.
template <bool VEC>
DEVINL short8 load_row8(const unsigned short* row, int c, int n, bool live) {
  short8 v;
  if constexpr (VEC) {
    v = *reinterpret_cast<const short8*>(row + min(c, n - 8));
    return live && c < n ? v : short8{};
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = (short)row[min(c + j, n - 1)];
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = live && c + j < n ? v[j] : (short)0;
    return v;
  }
}

// Eight channels of token t's q or k (columns off ..).
template <bool VEC>
DEVINL void load_channels(const GlaChunkArgs& a, long row0, int len, int off,
                          int h, int t, int d, float* v) {
  const short8 u = load_row8<VEC>(
      a.y + (row0 + min(t, len - 1)) * a.ldy + off + h * a.dim, d, a.dim, t < len);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] = bf2f((unsigned short)u[j]);
}

// Eight value columns of token t.
template <bool VEC>
DEVINL short8 load_values(const GlaChunkArgs& a, long row0, int len, int h, int t,
                          int c) {
  return load_row8<VEC>(a.y + (row0 + min(t, len - 1)) * a.ldy + a.v_off +
                            h * a.vdim, c, a.vdim, t < len);
}

// Gates that write: the room eight channels of token t leave, zero where !live
// and beyond the head; l2 gets their log2.
template <bool VEC>
DEVINL void load_gates(const GlaChunkArgs& a, long row0, int len, int h, int t,
                       int d, float* room, float* l2) {
  const float* z = a.a1 + (row0 + min(t, len - 1)) * a.ld1 + a.a1_off + h * a.dim;
  const float* zb = a.a2b + h * a.dim;
  const float* lo = a.lower + h * a.dim;
  float zv[8], bv[8], lv[8];
  if constexpr (VEC) {
    const int c = min(d, a.dim - 8);
    ldv<8>(z + c, zv);
    ldv<8>(zb + c, bv);
    ldv<8>(lo + c, lv);
  } else {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int c = min(d + j, a.dim - 1);
      zv[j] = z[c];
      bv[j] = zb[c];
      lv[j] = lo[c];
    }
  }
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const bool in = t < len && d + j < a.dim;
    const float r = forget_room(lv[j], zv[j] + bv[j]);
    room[j] = in ? r : 0.f;
    if (l2) l2[j] = in ? log2_forget(lv[j], zv[j] + bv[j], r) : 0.f;
  }
}

// Eight channels of token t's silu(q).
template <bool VEC>
DEVINL void load_silu(const GlaChunkArgs& a, long row0, int len, int h, int t,
                      int d, float* v) {
  load_channels<VEC>(a, row0, len, a.q_off, h, t, d, v);
#pragma unroll
  for (int j = 0; j < 8; ++j) v[j] *= sigmoid_f(v[j]);
}

// grid (chunks, H). LDS: b (C x (DP + 4))
template <int DP, int C, bool VEC>
__global__ __launch_bounds__(256) void hgrn_prep_kernel(GlaChunkArgs a) {
  constexpr int LDB = DP + 4, PN = C * DP / 8 / 256;
  extern __shared__ __attribute__((aligned(16))) float lds_b[];
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const long row0 = a.row0[ch];
  const int len = a.len[ch];
  float k[PN][8];
#pragma unroll
  for (int n = 0; n < PN; ++n) {
    const int idx = tid + n * 256;
    const int t = idx / (DP / 8), d = idx % (DP / 8) * 8;
    float l2[8];
    load_gates<VEC>(a, row0, len, h, t, d, k[n], l2);
    stv<8>(lds_b + t * LDB + d, l2);
  }
  __syncthreads();
  const long base = (long)ch * a.H + h;
  if (tid < DP) {
    float s = 0.f;
#pragma unroll 16
    for (int t = 0; t < C; ++t) {
      s += lds_b[t * LDB + tid];
      lds_b[t * LDB + tid] = s;
    }
  }
  __syncthreads();
#pragma unroll
  for (int n = 0; n < PN; ++n) {
    const int idx = tid + n * 256;
    const int t = idx / (DP / 8), d = idx % (DP / 8) * 8;
    float b[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      b[j] = lds_b[t * LDB + d + j];
      k[n][j] *= fast_exp2(lds_b[(C - 1) * LDB + d + j] - b[j]);
    }
    stv<8>(a.b + (base * C + t) * DP + d, b);
    short8 vh, vl;
    split8(k[n], vh, vl);
    const long at = base * 2 * C * DP + t * DP + d;
    *reinterpret_cast<short8*>(a.kd + at) = vh;
    *reinterpret_cast<short8*>(a.kd + at + C * DP) = vl;
  }
}

// grid (chunks, H). LDS: b (C x (DP + 4)), a1 (C x r), a2 of the head (r x DP)
template <int DP, int C, bool VEC>
__global__ __launch_bounds__(256) void gla_prep_kernel(GlaChunkArgs a) {
  constexpr int LDB = DP + 4;
  extern __shared__ __attribute__((aligned(16))) float lds_b[];
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  float* a1s = lds_b + C * LDB;
  float* a2s = a1s + C * a.r;
  const long row0 = a.row0[ch];
  const int len = a.len[ch];
  for (int i = tid; i < C * a.r; i += 256)
    a1s[i] = i / a.r < len
                 ? a.a1[(row0 + i / a.r) * a.ld1 + a.a1_off + i % a.r] : 0.f;
  for (int i = tid; i < a.r * DP; i += 256) {
    const int d = i % DP;
    a2s[i] = d < a.dim ? a.a2[(long)(i / DP) * a.H * a.dim + h * a.dim + d] : 0.f;
  }
  __syncthreads();
  {
    // 256 / DP tokens at a time, one channel a thread
    const int d = tid % DP;
    const float bias = d < a.dim ? a.a2b[h * a.dim + d] : 0.f;
    for (int t = tid / DP; t < C; t += 256 / DP) {
      float z = bias;
      for (int i = 0; i < a.r; ++i) z += a1s[t * a.r + i] * a2s[i * DP + d];
      lds_b[t * LDB + d] =
          d < a.dim && t < len ? log2_sigmoid(z) * a.inv_tau : 0.f;
    }
  }
  __syncthreads();
  const long base = (long)ch * a.H + h;
  if (tid < DP) {
    float s = 0.f;
#pragma unroll 16
    for (int t = 0; t < C; ++t) {
      s += lds_b[t * LDB + tid];
      lds_b[t * LDB + tid] = s;
    }
  }
  __syncthreads();
#pragma unroll
  for (int n = 0; n < C * DP / 8 / 256; ++n) {
    const int idx = tid + n * 256;
    const int t = idx / (DP / 8), d = idx % (DP / 8) * 8;
    float k[8], b[8];
    load_channels<VEC>(a, row0, len, a.k_off, h, t, d, k);
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      b[j] = lds_b[t * LDB + d + j];
      k[j] *= fast_exp2(lds_b[(C - 1) * LDB + d + j] - b[j]);
    }
    stv<8>(a.b + (base * C + t) * DP + d, b);
    short8 vh, vl;
    split8(k, vh, vl);
    const long at = base * 2 * C * DP + t * DP + d;
    *reinterpret_cast<short8*>(a.kd + at) = vh;
    *reinterpret_cast<short8*>(a.kd + at + C * DP) = vl;
  }
}

// grid (vdim / 64, H, listed sequences); a wave owns 16 value columns and the
// state's whole column. The state's accumulators hold rows in the order
//     tile 2g + n, row x*4 + y  <->  channel g*32 + x*8 + n*4 + y
// so that a lane's registers of two tiles are eight consecutive channels: an
// operand fragment as it is.
template <int DP, int C, bool VEC>
__global__ __launch_bounds__(256) void gla_scan_kernel(GlaChunkArgs a) {
  constexpr int NG = DP / 32, NC = C / 32;
  // rows 16 banks apart (mod 64): the permuted column reads do not collide
  constexpr int LDD = DP == 32 ? 96 : DP + 32, LDV = 64 + 8;
  constexpr int PD = C * DP / 8 / 256;   // 16 B pieces a thread and plane
  constexpr int PV = C * 64 / 8 / 256;
  constexpr int BUF = 2 * C * LDD + C * LDV + 2 * DP;  // 16-bit elements
  static_assert(PD >= 1 && PV >= 1, "chunk smaller than the workgroup");
  extern __shared__ __attribute__((aligned(16))) unsigned short lds_scan[];
  const int h = blockIdx.y, i = blockIdx.z, s = a.list[i], tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int v0 = blockIdx.x * 64, vt = blockIdx.x * 4 + wave;
  const int col = v0 + wave * 16 + li;
  const bool live = col < a.vdim;
  float* S = a.state + ((long)a.slots[s] * a.H + h) * a.dim * a.vdim;

  f32x4 acc[2 * NG];
  const bool kept = a.q_start[s] != 0 && live;
#pragma unroll
  for (int n = 0; n < 2 * NG; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc[n][r] = S[(long)min((n >> 1) * 32 + hi * 8 + (n & 1) * 4 + r, a.dim - 1) *
                        a.vdim + min(col, a.vdim - 1)];
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

  short8 rk[2][PD], rv[PV];
  float rd = 0.f;
  auto fetch = [&](int ch) {
    const long base = (long)ch * a.H + h;
#pragma unroll
    for (int p = 0; p < 2; ++p)
#pragma unroll
      for (int n = 0; n < PD; ++n)
        rk[p][n] = *reinterpret_cast<const short8*>(
            a.kd + (base * 2 + p) * C * DP + (tid + n * 256) * 8);
    const long row0 = first + (long)(ch - c0) * C;
    const int len = min(C, total - (ch - c0) * C);
#pragma unroll
    for (int n = 0; n < PV; ++n) {
      const int idx = tid + n * 256;
      rv[n] = load_values<VEC>(a, row0, len, h, idx / 8, v0 + idx % 8 * 8);
    }
    rd = a.b[(base * C + C - 1) * DP + tid % DP];
  };
  auto stage = [&](unsigned short* buf) {
#pragma unroll
    for (int p = 0; p < 2; ++p)
#pragma unroll
      for (int n = 0; n < PD; ++n) {
        const int idx = tid + n * 256;
        *reinterpret_cast<short8*>(buf + (p * C + idx / (DP / 8)) * LDD +
                                   idx % (DP / 8) * 8) = rk[p][n];
      }
    unsigned short* vb = buf + 2 * C * LDD;
#pragma unroll
    for (int n = 0; n < PV; ++n) {
      const int idx = tid + n * 256;
      *reinterpret_cast<short8*>(vb + idx / 8 * LDV + idx % 8 * 8) = rv[n];
    }
    if (tid < DP) ((float*)(vb + C * LDV))[tid] = fast_exp2(rd);
  };

  fetch(c0);
  stage(lds_scan);
  if (c0 + 1 < c1) fetch(c0 + 1);
  for (int ch = c0; ch < c1; ++ch) {
    const unsigned short* buf = lds_scan + ((ch - c0) & 1) * BUF;
    __syncthreads();   // buf is written, the other one is read
    // registers hold the next chunk since an iteration ago
    if (ch + 1 < c1) stage(lds_scan + ((ch + 1 - c0) & 1) * BUF);
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
          sv[r] = acc[2 * g][r];
          sv[4 + r] = acc[2 * g + 1][r];
        }
        short8 sh, sl;
        split8(sv, sh, sl);
        *reinterpret_cast<short8*>(sp + g * 512) = sh;
        *reinterpret_cast<short8*>(sp + (NG + g) * 512) = sl;
      }
    }
    const unsigned short* vb = buf + 2 * C * LDD;
    const float* dt = (const float*)(vb + C * LDV);
    bf16x8 vf[NC];
#pragma unroll
    for (int k = 0; k < NC; ++k)
      vf[k] = column_frag(vb, LDV, k * 32, wave * 16 + (li & 3) * 4, li, hi);
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        const f32x4 dv = *reinterpret_cast<const f32x4*>(dt + g * 32 + hi * 8 + n * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[2 * g + n][r] *= dv[r];
#pragma unroll
        for (int k = 0; k < NC; ++k)
#pragma unroll
          for (int p = 0; p < 2; ++p)
            acc[2 * g + n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                column_frag(buf + p * C * LDD, LDD, k * 32,
                            g * 32 + (li & 3) * 8 + n * 4, li, hi),
                vf[k], acc[2 * g + n], 0, 0, 0);
      }
  }
  if (live) {
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int n = 0; n < 2; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int d = g * 32 + hi * 8 + n * 4 + r;
          if (d < a.dim) S[(long)d * a.vdim + col] = acc[2 * g + n][r];
        }
  }
}

// grid (chunks, H), eight waves; a wave owns every eighth tile of 16 value
// columns. Outputs are made transposed, o^T = S^T qd^T + v^T A^T: a lane holds
// four consecutive columns of one token. LDS: b, later v; qd; A. WRITES: beside b
// silu(q) and k, which the blocks of A read several times.
template <int DP, int C, int NCT, bool VEC, bool WRITES = false>
__global__ __launch_bounds__(512) void gla_out_kernel(GlaChunkArgs a) {
  constexpr int LDB = DP + 4, LDD = DP + 8, LDA = C + 8, NG = DP / 32;
  constexpr int NT = C / 16, NC = C / 32, NB = C / 16, VC = NCT * 128;
  constexpr int LDV = VC + 24;   // rows 12 banks apart, for column reads
  constexpr int BQK = 2 * (C + 1) * LDB + (WRITES ? 4 * C * LDB : 0);
  constexpr int FIRST = BQK > C * LDV ? BQK : C * LDV;
  constexpr int PB = C * DP / 4 / 512, PQ = C * DP / 8 / 512 > 0 ? C * DP / 8 / 512 : 1;
  constexpr int PV = C * VC / 8 / 512;
  // the states, too, are asked for ahead, where there are registers for them
  constexpr bool EARLY = VEC && NCT * NG <= 8;
  constexpr int NS = EARLY ? NCT : 1;
  constexpr float SPAN = 80.f;  // widest safe range of exponents, log2
  extern __shared__ __attribute__((aligned(16))) unsigned short lds_out[];
  __shared__ float ssum[8][C];
  float* bs = (float*)lds_out + LDB;         // (C, LDB), a zero row ahead
  unsigned short* vs = lds_out;              // (C, LDV)
  unsigned short* qs = lds_out + FIRST;      // (2, C, LDD)
  unsigned short* as = qs + 2 * C * LDD;     // (2, C, LDA)
  float* q32 = bs + C * LDB;                 // (C, LDB), WRITES
  float* k32 = q32 + C * LDB;                // (C, LDB), WRITES
  const int ch = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const long row0 = a.row0[ch], base = (long)ch * a.H + h;
  const int len = a.len[ch];

  // everything that comes from memory is asked for up front
  f32x4 rb[PB];
  float rq[PQ][8];
  short8 rv[PV];
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
  for (int n = 0; n < PB; ++n)
    rb[n] = *reinterpret_cast<const f32x4*>(a.b + base * C * DP + (tid + n * 512) * 4);
#pragma unroll
  for (int n = 0; n < PQ; ++n) {
    const int idx = min(tid + n * 512, C * DP / 8 - 1);
    const int t = idx / (DP / 8), d = idx % (DP / 8) * 8;
    if constexpr (WRITES) {
      float k[8];
      load_silu<VEC>(a, row0, len, h, t, d, rq[n]);
      load_gates<VEC>(a, row0, len, h, t, d, k, nullptr);
      stv<8>(q32 + t * LDB + d, rq[n]);
      stv<8>(k32 + t * LDB + d, k);
    } else {
      load_channels<VEC>(a, row0, len, a.q_off, h, t, d, rq[n]);
    }
  }
#pragma unroll
  for (int n = 0; n < PV; ++n) {
    const int idx = tid + n * 512;
    rv[n] = load_values<VEC>(a, row0, len, h, idx / (VC / 8), idx % (VC / 8) * 8);
  }
  if constexpr (EARLY) {
#pragma unroll
    for (int c = 0; c < NCT; ++c) load_state(c, sh[c], sl[c]);
  }
#pragma unroll
  for (int n = 0; n < PB; ++n) {
    const int idx = tid + n * 512;
    *reinterpret_cast<f32x4*>(bs + idx / (DP / 4) * LDB + idx % (DP / 4) * 4) = rb[n];
  }
  if (tid < DP) bs[tid - LDB] = 0.f;
  __syncthreads();
#pragma unroll
  for (int n = 0; n < PQ; ++n) {
    const int idx = tid + n * 512;
    if (idx >= C * DP / 8) continue;
    const int t = idx / (DP / 8), d = idx % (DP / 8) * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j)
      rq[n][j] *= a.qscale * fast_exp2(bs[t * LDB + d + j]);
    short8 vh, vl;
    split8(rq[n], vh, vl);
    *reinterpret_cast<short8*>(qs + t * LDD + d) = vh;
    *reinterpret_cast<short8*>(qs + (C + t) * LDD + d) = vl;
  }
  for (int pair = wave; pair < NB * NB; pair += 8) {
    const int I = pair / NB, J = pair % NB;
    f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
    if (J <= I && I * 16 < len) {
      const float* ref = bs + (I * 16 - 1) * LDB;  // row before block I
      bool near = true;
      if (J == I) {
        for (int d = lane; d < DP; d += WAVE)
          near = near && ref[d] - bs[(I * 16 + 15) * LDB + d] <= SPAN;
        near = __builtin_amdgcn_ballot_w64(!near) == 0;
      }
      if (near) {
        const int t = I * 16 + li, s = J * 16 + li;
        float q[NG][8], k[NG][8];
#pragma unroll
        for (int kk = 0; kk < NG; ++kk) {
          if constexpr (WRITES) {
            ldv<8>(q32 + t * LDB + kk * 32 + hi * 8, q[kk]);
            ldv<8>(k32 + s * LDB + kk * 32 + hi * 8, k[kk]);
          } else {
            load_channels<VEC>(a, row0, len, a.q_off, h, t, kk * 32 + hi * 8, q[kk]);
            load_channels<VEC>(a, row0, len, a.k_off, h, s, kk * 32 + hi * 8, k[kk]);
          }
        }
#pragma unroll
        for (int kk = 0; kk < NG; ++kk) {
          const int d = kk * 32 + hi * 8;
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const float r = ref[d + j];
            q[kk][j] *= a.qscale * fast_exp2(bs[t * LDB + d + j] - r);
            k[kk][j] *= fast_exp2(r - bs[s * LDB + d + j]);
          }
          short8 qh, ql, kh, kl;
          split8(q[kk], qh, ql);
          split8(k[kk], kh, kl);
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              as_bf16x8(qh), as_bf16x8(kh), acc, 0, 0, 0);
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              as_bf16x8(ql), as_bf16x8(kh), acc, 0, 0, 0);
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              as_bf16x8(qh), as_bf16x8(kl), acc, 0, 0, 0);
        }
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = I * 16 + hi * 4 + r, s = J * 16 + li;
          if (s > t || t >= len) continue;
          float sum = 0.f;
          if constexpr (WRITES) {
            for (int d = 0; d < a.dim; ++d)
              sum += q32[t * LDB + d] * k32[s * LDB + d] *
                     fast_exp2(bs[t * LDB + d] - bs[s * LDB + d]);
            acc[r] = sum;
            continue;
          }
          const unsigned short* qp =
              a.y + (row0 + t) * a.ldy + a.q_off + h * a.dim;
          const unsigned short* kp =
              a.y + (row0 + s) * a.ldy + a.k_off + h * a.dim;
          for (int d = 0; d < a.dim; ++d)
            sum += bf2f(qp[d]) * a.qscale * bf2f(kp[d]) *
                   fast_exp2(bs[t * LDB + d] - bs[s * LDB + d]);
          acc[r] = sum;
        }
      }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = I * 16 + hi * 4 + r, s = J * 16 + li;
      const float v = s <= t ? acc[r] : 0.f;
      const unsigned short vh = cvt_bf(v);
      as[t * LDA + s] = vh;
      as[(C + t) * LDA + s] = cvt_bf(v - bf2f(vh));
    }
  }
  __syncthreads();   // b is read
#pragma unroll
  for (int n = 0; n < PV; ++n) {
    const int idx = tid + n * 512;
    *reinterpret_cast<short8*>(vs + idx / (VC / 8) * LDV + idx % (VC / 8) * 8) = rv[n];
  }
  __syncthreads();

  // v, then the states: an operand that is read serves all of the wave's tiles
  f32x4 o[NCT][NT];
#pragma unroll
  for (int c = 0; c < NCT; ++c)
#pragma unroll
    for (int t = 0; t < NT; ++t) o[c][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
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
            as + (p * C + t * 16 + li) * LDA + k * 32 + hi * 8));
#pragma unroll
        for (int c = 0; c < NCT; ++c)
          o[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[c], af, o[c][t], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int c0 = 0; c0 < NCT; c0 += NS) {
    if constexpr (!EARLY) load_state(c0, sh[0], sl[0]);
#pragma unroll
    for (int g = 0; g < NG; ++g)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const bf16x8 qh = as_bf16x8(*reinterpret_cast<const short8*>(
            qs + (t * 16 + li) * LDD + g * 32 + hi * 8));
        const bf16x8 ql = as_bf16x8(*reinterpret_cast<const short8*>(
            qs + (C + t * 16 + li) * LDD + g * 32 + hi * 8));
#pragma unroll
        for (int c = 0; c < NS; ++c) {
          f32x4& r = o[c0 + c][t];
          r = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sh[c][g], qh, r, 0, 0, 0);
          r = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sh[c][g], ql, r, 0, 0, 0);
          r = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sl[c][g], qh, r, 0, 0, 0);
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
    float ss = 0.f;
#pragma unroll
    for (int c = 0; c < NCT; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) ss += o[c][t][r] * o[c][t][r];
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
    unsigned short* op = a.out + (row0 + tt) * a.ldo + h * a.vdim;
#pragma unroll
    for (int c = 0; c < NCT; ++c) {
      const int v0 = (c * 8 + wave) * 16 + hi * 4;
      if (v0 >= a.vdim) continue;
      if constexpr (VEC) {
        float g[4], w[4];
        if constexpr (!WRITES) ldv<4>(gp + v0, g);
        ldv<4>(a.nw + v0, w);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          w[r] *= o[c][t][r] * inv;
          if constexpr (!WRITES) w[r] *= g[r] * sigmoid_f(g[r]);
        }
        stv<4>(op + v0, w);
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (v0 + r >= a.vdim) continue;
          float w = o[c][t][r] * inv * a.nw[v0 + r];
          if constexpr (!WRITES) {
            const float g = bf2f(gp[v0 + r]);
            w *= g * sigmoid_f(g);
          }
          op[v0 + r] = cvt_bf(w);
        }
      }
    }
  }
}
