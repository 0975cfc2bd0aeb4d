// Row-wise fused steps of parallel-residual blocks over ragged batches.
//
// residual_norm_kernel — folds everything a layer left pending (split-K
//     partials of its output GEMM, routed expert rows, identity-expert
//     weights) into the 32-bit residual and emits the next layer's grouped
//     RMS norm, in one pass per row. For norms after the sum the residual is
//     scaled first and the normed row takes its place.
// proj_post_kernel — everything between the fused input GEMM and attention:
//     folds split-K partials, RMS-norms q and k over the whole projection,
//     writes K/V into the pages, hands on the output gate, applies the
//     feed-forward activation and routes the token to its experts.
// clamped_glu_kernel — bias, clamps, gate and product of a gated feed-forward.
// softcap_kernel — cap * tanh(z / cap), in place.
// router_gemm_kernel — f32 router logits where the input GEMM emits bf16.
//
// T is the activation element (unsigned short = bf16 bits, or float), TP the
// element of the GEMM output being read. All arithmetic is f32.

#pragma once
#include "common.h"

DEVINL float ldf(const unsigned short* p) { return bf2f(*p); }
DEVINL float ldf(const float* p) { return *p; }
// round to nearest even in hardware
DEVINL unsigned short cvt_bf(float v) {
  return __builtin_bit_cast(unsigned short, (__bf16)v);
}
DEVINL void stf(unsigned short* p, float v) { *p = cvt_bf(v); }
DEVINL void stf(float* p, float v) { *p = v; }

typedef __attribute__((ext_vector_type(4))) unsigned short ushort4v;

// V (1, 4 or 8) consecutive elements as f32, aligned to V elements.
template <int V>
DEVINL void ldv(const unsigned short* p, float* o) {
  if constexpr (V == 8) {
    load_bf16x8(p, o);
  } else if constexpr (V == 4) {
    const ushort4v u = *reinterpret_cast<const ushort4v*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = bf2f(u[j]);
  } else {
    o[0] = bf2f(*p);
  }
}
template <int V>
DEVINL void ldv(const float* p, float* o) {
  if constexpr (V == 8) {
    ldv<4>(p, o);
    ldv<4>(p + 4, o + 4);
  } else if constexpr (V == 4) {
    const f32x4 u = *reinterpret_cast<const f32x4*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = u[j];
  } else {
    o[0] = *p;
  }
}
template <int V>
DEVINL void stv(unsigned short* p, const float* v) {
  if constexpr (V == 8) {
    short8 u;
#pragma unroll
    for (int j = 0; j < 8; ++j) u[j] = (short)cvt_bf(v[j]);
    *reinterpret_cast<short8*>(p) = u;
  } else if constexpr (V == 4) {
    ushort4v u;
#pragma unroll
    for (int j = 0; j < 4; ++j) u[j] = cvt_bf(v[j]);
    *reinterpret_cast<ushort4v*>(p) = u;
  } else {
    *p = cvt_bf(v[0]);
  }
}
template <int V>
DEVINL void stv(float* p, const float* v) {
  if constexpr (V == 8) {
    stv<4>(p, v);
    stv<4>(p + 4, v + 4);
  } else if constexpr (V == 4) {
    f32x4 u;
#pragma unroll
    for (int j = 0; j < 4; ++j) u[j] = v[j];
    *reinterpret_cast<f32x4*>(p) = u;
  } else {
    *p = v[0];
  }
}

DEVINL float sigmoid_f(float z) {
  return __builtin_amdgcn_rcpf(1.f + fast_exp2(-z * LOG2E));
}

// e^z - 1 - z for z <= 0. Near zero the series, where the difference would
// cancel.
DEVINL float exp_minus_1_minus(float z) {
  const float far = fast_exp2(z * LOG2E) - 1.f - z;
  const float t = 1.f + z * (1.f / 6) * (1.f + z * (1.f / 7) * (1.f + z * (1.f / 8)));
  const float near = 0.5f * z * z *
      (1.f + z * (1.f / 3) * (1.f + z * (1.f / 4) * (1.f + z * (1.f / 5) * t)));
  return z > -0.5f ? near : far;
}

// ---------------------------------------------------------------------------

struct ResidualArgs {
  float* x;            // (N, W) f32 residual, updated in place
  const void* parts;   // (ks, N, ldp) pending GEMM output, or null
  long pstride;        // elements between splits
  const void* routed;  // (N, top, ldr) weighted expert outputs, or null
  const int* ids;      // (N, top): < 0 = no routed row for this choice
  const float* idw;    // (N,) weight of the layer's own input, or null
  const void* hprev;   // (N, ldhp) that input
  const float* bias;   // (W,) of the pending GEMM, or null
  const float* nw;     // (W,) norm weight; null = fold only
  void* h;             // (N, ldh) normed row, zero beyond W
  int W, ks, ldp, top, ldr, ldhp, ldh, groups;
  int post;            // the normed row becomes the residual
  float eps, alpha;    // alpha scales x before the sum
};

// LDS: W floats (the row) + groups * subs partial sums.
template <typename TP, typename T, int V, int BLOCK>
__global__ __launch_bounds__(BLOCK) void residual_norm_kernel(ResidualArgs a) {
  extern __shared__ float lds_row[];
  float* stat = lds_row + ((a.W + 3) & ~3);
  const long t = blockIdx.x;
  const int W = a.W;
  float* xr = a.x + t * W;
  const TP* pr = (const TP*)a.parts + t * a.ldp;
  const T* rr = (const T*)a.routed + t * (long)a.top * a.ldr;
  const T* hp = (const T*)a.hprev + t * (long)a.ldhp;
  const float iw = a.idw ? a.idw[t] : 0.f;

  for (int i = threadIdx.x * V; i < W; i += BLOCK * V) {
    float v[V], u[V];
    ldv<V>(xr + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] *= a.alpha;
    if (a.parts) {
      float d[V];
      ldv<V>(pr + i, d);
      for (int s = 1; s < a.ks; ++s) {
        ldv<V>(pr + s * a.pstride + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) d[j] += u[j];
      }
      if (a.routed) {
        for (int k = 0; k < a.top; ++k) {
          if (a.ids[t * a.top + k] < 0) continue;
          ldv<V>(rr + (long)k * a.ldr + i, u);
#pragma unroll
          for (int j = 0; j < V; ++j) d[j] += u[j];
        }
      }
      if (iw != 0.f) {
        ldv<V>(hp + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) d[j] += iw * u[j];
      }
      if (a.bias) {
        ldv<V>(a.bias + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) d[j] += u[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] += d[j];
      if (!a.post) stv<V>(xr + i, v);
    }
#pragma unroll
    for (int j = 0; j < V; ++j) lds_row[i + j] = v[j];
  }
  if (!a.nw) return;
  __syncthreads();

  // sums of squares: every unit (a group, or an even share of one where
  // there are fewer groups than waves) belongs to one wave
  constexpr int NWAVE = BLOCK / WAVE;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int gs = W / a.groups;
  const int subs = a.groups >= NWAVE ? 1 : NWAVE / a.groups;
  for (int un = wave; un < a.groups * subs; un += NWAVE) {
    const int g = un / subs, sb = un % subs;
    const int lo = g * gs + (int)((long)gs * sb / subs);
    const int hi = g * gs + (int)((long)gs * (sb + 1) / subs);
    float ss = 0.f;
    for (int i = lo + lane; i < hi; i += WAVE) ss += lds_row[i] * lds_row[i];
    ss = wave_reduce_sum(ss);
    if (lane == 0) stat[un] = ss;
  }
  __syncthreads();
  T* hr = (T*)a.h + t * (long)a.ldh;
  // one scale per group, in place of its first partial sum
  for (int g = threadIdx.x; g < a.groups; g += BLOCK) {
    float ss = 0.f;
    for (int k = 0; k < subs; ++k) ss += stat[g * subs + k];
    stat[g * subs] = 1.f / sqrtf(ss / (float)gs + a.eps);
  }
  __syncthreads();
  for (int i = threadIdx.x * V; i < a.ldh; i += BLOCK * V) {
    float v[V];
#pragma unroll
    for (int j = 0; j < V; ++j)
      v[j] = i + j < W ? lds_row[i + j] * stat[(i + j) / gs * subs] * a.nw[i + j]
                       : 0.f;
    stv<V>(hr + i, v);
    if (a.post && i < W) stv<V>(xr + i, v);
  }
}

struct GluArgs {
  const void* parts;  // (ks, N, ldp) [gate | up] columns
  long pstride;
  const float* gb;    // (ff,) biases, or null
  const float* ub;
  void* out;          // (N, ldo), zero beyond ff
  long N;
  int ks, ldp, g_off, u_off, ff, ldo;
  float limit, slope;
};

// g = min(gate, limit), u = clamp(up, -limit, limit):
// out = g * sigmoid(slope * g) * (u + 1). grid (chunks of 256 * V columns,
// groups of R rows): the biases of its columns stay in a thread's registers.
template <typename TP, typename T, int V, int R>
__global__ __launch_bounds__(256) void clamped_glu_kernel(GluArgs a) {
  const int i = (blockIdx.x * 256 + threadIdx.x) * V;
  if (i >= a.ldo) return;
  const bool live = i < a.ff;
  float gb[V], ub[V];
#pragma unroll
  for (int j = 0; j < V; ++j) gb[j] = ub[j] = 0.f;
  if (live && a.gb) ldv<V>(a.gb + i, gb);
  if (live && a.ub) ldv<V>(a.ub + i, ub);
#pragma unroll
  for (int n = 0; n < R; ++n) {
    const long t = blockIdx.y * R + n;
    if (R > 1 && t >= a.N) return;
    float g[V], u[V], w[V];
#pragma unroll
    for (int j = 0; j < V; ++j) g[j] = 0.f;
    if (live) {
      const TP* row = (const TP*)a.parts + t * (long)a.ldp;
      ldv<V>(row + a.g_off + i, g);
      ldv<V>(row + a.u_off + i, u);
      for (int s = 1; s < a.ks; ++s) {
        ldv<V>(row + s * a.pstride + a.g_off + i, w);
#pragma unroll
        for (int j = 0; j < V; ++j) g[j] += w[j];
        ldv<V>(row + s * a.pstride + a.u_off + i, w);
#pragma unroll
        for (int j = 0; j < V; ++j) u[j] += w[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float gj = fminf(g[j] + gb[j], a.limit);
        const float uj = fminf(fmaxf(u[j] + ub[j], -a.limit), a.limit);
        g[j] = gj * sigmoid_f(a.slope * gj) * (uj + 1.f);
      }
    }
    stv<V>((T*)a.out + t * (long)a.ldo + i, g);
  }
}

__global__ __launch_bounds__(256) void softcap_kernel(float* __restrict__ z,
                                                      long n, float cap) {
  for (long i = blockIdx.x * 256L + threadIdx.x; i < n; i += gridDim.x * 256L)
    z[i] = cap * tanhf(z[i] / cap);
}

// x[n] = table[ids[n]] (+ pos_table[pos[n]]) in f32; indices are clamped.
template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(
    const int* __restrict__ ids, const int* __restrict__ pos,
    const T* __restrict__ table, const T* __restrict__ pos_table,
    float* __restrict__ x, int W, int vocab, int max_pos) {
  const long n = blockIdx.x;
  const T* a = table + (long)min(max(ids[n], 0), vocab - 1) * W;
  if (!pos_table) {
    for (int i = threadIdx.x; i < W; i += 256) x[n * W + i] = ldf(a + i);
    return;
  }
  const T* b = pos_table + (long)min(max(pos[n], 0), max_pos - 1) * W;
  for (int i = threadIdx.x; i < W; i += 256) x[n * W + i] = ldf(a + i) + ldf(b + i);
}

// ---------------------------------------------------------------------------

struct PostArgs {
  const void* parts;    // (ks, N, ldp) input GEMM output
  long pstride;
  const float* rparts;  // (rks, N, ldr) router logits, f32
  long rstride;
  const float* qn;      // (H*dim,) q norm weight
  const float* kn;      // (G*dim,)
  const float* corr;    // (E + NI,) added to the scores for the choice only
  void* q;              // (N, H, dkp)
  void* gate;           // (N, H*vdim) or null: the reader takes it from parts
  void* a2;             // (N, lda2): [attention | activation | zeros]
  void* kp;             // (np, G, P, dkp)
  void* vp;             // (np, G, dvp, P)
  const int* table;     // (S, maxp)
  const int* tok_seq;
  const int* tok_pos;
  int* ids;             // (N, top)
  float* wts;           // (N, top)
  float* idw;           // (N,)
  int ks, ldp, rks, ldr;
  int q_off, k_off, v_off, g_off, u_off, u2_off, r_off, sg_off;
  int H, G, dim, vdim, dkp, dvp, P, maxp;
  int has_kv;
  int act;              // 0 none, 1 xIELU, 2 silu(gate) * up
  int ff, act_col, lda2;
  int E, NI, top;
  float eps, xp, xq, rscale;
};

static constexpr int POST_BLOCK = 256;
static constexpr int POST_CHUNK = 2048;  // elementwise columns per workgroup
static constexpr int MAX_ROUTED = 1024;  // router outputs

template <typename TP, int V>
DEVINL void fold(const PostArgs& a, const TP* row, int c, float* o) {
  ldv<V>(row + c, o);
  for (int s = 1; s < a.ks; ++s) {
    float u[V];
    ldv<V>(row + s * a.pstride + c, u);
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] += u[j];
  }
}

DEVINL float router_logit(const PostArgs& a, long t, int c) {
  const float* r = a.rparts + t * a.ldr + c;
  float v = r[0];
  for (int s = 1; s < a.rks; ++s) v += r[s * a.rstride];
  return v;
}

// One projection section of n columns into LDS; returns 1 / rms over all n.
template <typename TP, int V>
DEVINL float stage_section(const PostArgs& a, const TP* row, int off, int n,
                           float* lds, float* red) {
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < n; i += POST_BLOCK * V) {
    float v[V];
    fold<TP, V>(a, row, off + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      lds[i + j] = v[j];
      ss += v[j] * v[j];
    }
  }
  ss = wave_reduce_sum(ss);
  if ((threadIdx.x & (WAVE - 1)) == 0) red[threadIdx.x / WAVE] = ss;
  __syncthreads();
  float tot = 0.f;
#pragma unroll
  for (int i = 0; i < POST_BLOCK / WAVE; ++i) tot += red[i];
  return 1.f / sqrtf(tot / (float)n + a.eps);
}

// grid (N, 3 + chunks): y = 0 q, 1 k and v, 2 router, 3.. elementwise.
template <typename TP, typename T, int V>
__global__ __launch_bounds__(POST_BLOCK) void proj_post_kernel(PostArgs a) {
  extern __shared__ float lds_sec[];
  __shared__ float red[POST_BLOCK / WAVE];
  const long t = blockIdx.x;
  const int role = blockIdx.y;
  const TP* row = (const TP*)a.parts + t * (long)a.ldp;

  if (role == 0) {
    const int n = a.H * a.dim;
    const float inv = stage_section<TP, V>(a, row, a.q_off, n, lds_sec, red);
    T* q = (T*)a.q + t * (long)a.H * a.dkp;
    for (int i = threadIdx.x; i < a.H * a.dkp; i += POST_BLOCK) {
      const int h = i / a.dkp, d = i % a.dkp;
      float v = 0.f;
      if (d < a.dim) {
        const int c = h * a.dim + d;
        v = lds_sec[c] * inv * a.qn[c];
      }
      stf(q + i, v);
    }
    return;
  }
  if (role == 1) {
    const int pos = a.tok_pos[t];
    if (!a.has_kv || pos < 0) return;
    const int n = a.G * a.dim;
    const float inv = stage_section<TP, V>(a, row, a.k_off, n, lds_sec, red);
    const long page = a.table[(long)a.tok_seq[t] * a.maxp + pos / a.P];
    const int slot = pos % a.P;
    T* kp = (T*)a.kp + page * a.G * a.P * a.dkp;
    for (int i = threadIdx.x; i < a.G * a.dkp; i += POST_BLOCK) {
      const int g = i / a.dkp, d = i % a.dkp;
      float v = 0.f;
      if (d < a.dim) {
        const int c = g * a.dim + d;
        v = lds_sec[c] * inv * a.kn[c];
      }
      stf(kp + ((long)g * a.P + slot) * a.dkp + d, v);
    }
    T* vp = (T*)a.vp + page * a.G * a.dvp * a.P;
    for (int i = threadIdx.x; i < a.G * a.dvp; i += POST_BLOCK) {
      const int g = i / a.dvp, d = i % a.dvp;
      float v[1] = {0.f};
      if (d < a.vdim) fold<TP, 1>(a, row, a.v_off + g * a.vdim + d, v);
      stf(vp + (long)i * a.P + slot, v[0]);
    }
    return;
  }
  if (role == 2) {
    const int n = a.E + a.NI;
    if (n == 0 || threadIdx.x >= WAVE) return;
    float* s = lds_sec;                // scores
    float* ch = lds_sec + MAX_ROUTED;  // choice scores
    const int lane = threadIdx.x;
    float mx = NEG_BIG;
    for (int i = lane; i < n; i += WAVE) {
      const float z = router_logit(a, t, a.r_off + i);
      s[i] = z;
      mx = fmaxf(mx, z);
    }
    mx = wave_reduce_max(mx);
    float sum = 0.f;
    for (int i = lane; i < n; i += WAVE) {
      s[i] = expf(s[i] - mx);
      sum += s[i];
    }
    const float inv = 1.f / wave_reduce_sum(sum);
    for (int i = lane; i < n; i += WAVE) {
      s[i] *= inv;
      ch[i] = s[i] + a.corr[i];
    }
    // every lane reads and writes its own columns only
    float idw = 0.f;
    for (int k = 0; k < a.top; ++k) {
      float best = -__builtin_inff();
      int at = n;
      for (int i = lane; i < n; i += WAVE)
        if (ch[i] > best || at == n) { best = ch[i]; at = i; }
#pragma unroll
      for (int m = 1; m < WAVE; m <<= 1) {
        const float ob = __shfl_xor(best, m);
        const int oa = __shfl_xor(at, m);
        if (oa < n && (at == n || ob > best || (ob == best && oa < at))) {
          best = ob;
          at = oa;
        }
      }
      // the owning lane holds the score; broadcast it
      float w = 0.f;
      if ((at & (WAVE - 1)) == lane) {
        w = s[at] * a.rscale;
        ch[at] = -__builtin_inff();
      }
      w = __shfl(w, at & (WAVE - 1));
      if (at >= a.E) idw += w;
      if (lane == 0) {
        a.ids[t * a.top + k] = at < a.E ? at : -1;
        a.wts[t * a.top + k] = w;
      }
    }
    if (lane == 0) a.idw[t] = idw;
    return;
  }

  // elementwise columns: [gate copy | activation and zero columns of a2]
  const int gn = a.gate ? a.H * a.vdim : 0;
  const int z0 = a.H * a.vdim;  // first column of a2 attention leaves alone
  const int total = gn + a.lda2 - z0;
  const int base = (role - 3) * POST_CHUNK;
  const int end = min(base + POST_CHUNK, total);
  float sg = 1.f;
  if (a.act == 2) sg = sigmoid_f(router_logit(a, t, a.sg_off));
  for (int i = base + threadIdx.x * V; i < end; i += POST_BLOCK * V) {
    float v[V];
    if (i < gn) {
      fold<TP, V>(a, row, a.g_off + i, v);
      stv<V>((T*)a.gate + t * (long)z0 + i, v);
      continue;
    }
    const int c = z0 + i - gn;
    const int f = c - a.act_col;
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (a.act && f >= 0 && f < a.ff) {
      fold<TP, V>(a, row, a.u_off + f, v);
      if (a.act == 1) {
#pragma unroll
        for (int j = 0; j < V; ++j) {
          const float z = v[j];
          v[j] = (z > 0.f ? a.xp * z * z : a.xq * exp_minus_1_minus(z)) + 0.5f * z;
        }
      } else {
        float u[V];
        fold<TP, V>(a, row, a.u2_off + f, u);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] = v[j] * sigmoid_f(v[j]) * u[j] * sg;
      }
    }
    stv<V>((T*)a.a2 + t * (long)a.lda2 + c, v);
  }
}

// ---------------------------------------------------------------------------
// C (M, N) f32 = A (M, K) bf16 @ W (N, K)^T, N small. One workgroup per
// 32 x 64 tile; its four waves split K and fold through LDS.
// ---------------------------------------------------------------------------

__global__ __launch_bounds__(256) void router_gemm_kernel(
    const unsigned short* __restrict__ A, const unsigned short* __restrict__ W,
    float* __restrict__ C, int M, int N, int K) {
  __shared__ float acc_lds[4][32 * 64];
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int m0 = blockIdx.y * 32, n0 = blockIdx.x * 64;
  const int steps = K / 32, per = (steps + 3) / 4;
  const int k0 = wave * per * 32, k1 = min(K, k0 + per * 32);
  const unsigned short* ar[2];
  const unsigned short* wr[4];
#pragma unroll
  for (int m = 0; m < 2; ++m)
    ar[m] = A + (long)min(m0 + m * 16 + li, M - 1) * K + hi * 8;
#pragma unroll
  for (int n = 0; n < 4; ++n)
    wr[n] = W + (long)min(n0 + n * 16 + li, N - 1) * K + hi * 8;
  f32x4 acc[2][4];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int n = 0; n < 4; ++n) acc[m][n] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int k = k0; k < k1; k += 32) {
    bf16x8 af[2], wf[4];
#pragma unroll
    for (int m = 0; m < 2; ++m)
      af[m] = as_bf16x8(*reinterpret_cast<const short8*>(ar[m] + k));
#pragma unroll
    for (int n = 0; n < 4; ++n)
      wf[n] = as_bf16x8(*reinterpret_cast<const short8*>(wr[n] + k));
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int n = 0; n < 4; ++n)
        acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af[m], wf[n],
                                                            acc[m][n], 0, 0, 0);
  }
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int n = 0; n < 4; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        acc_lds[wave][(m * 16 + hi * 4 + r) * 64 + n * 16 + li] = acc[m][n][r];
  __syncthreads();
  for (int i = threadIdx.x; i < 32 * 64; i += 256) {
    const int m = m0 + i / 64, n = n0 + i % 64;
    if (m < M && n < N)
      C[(long)m * N + n] =
          acc_lds[0][i] + acc_lds[1][i] + acc_lds[2][i] + acc_lds[3][i];
  }
}
