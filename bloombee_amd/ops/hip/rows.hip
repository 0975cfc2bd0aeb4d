// Row-wise fused steps of parallel-residual blocks over ragged batches.
//
// residual_norm_kernel — folds everything a layer left pending (split-K
//     partials of its output GEMM, routed expert rows, identity-expert
//     weights) into the 32-bit residual and emits the next layer's grouped
//     RMS norm, in one pass per row. For norms after the sum the residual is
//     scaled first and the normed row takes its place; for norms around a
//     sublayer what is pending is normed before it is added. Without a norm it
//     can hand on the sum as it is, beside the row of another matrix.
// proj_post_kernel — everything between the fused input GEMM and attention:
//     folds split-K partials, RMS-norms q and k over the whole projection,
//     writes K/V into the pages, hands on the output gate, applies the
//     feed-forward activation and routes the token to its experts.
// head_post_kernel — the same step for projections with biases, a norm per head
//     and a query temperature, without feed-forward.
// rope_post_kernel — the same step for projections with rotary positions and one
//     or several queries and keys per head.
// ff_post_kernel — feed-forward activation and routing of layers whose
//     feed-forward has an input of its own.
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

// 16 B a lane from memory to LDS without registers; l is the wave's, lane i's piece
// lands i * 16 behind it.
typedef const __attribute__((address_space(1))) void* gptr_t;
typedef __attribute__((address_space(3))) void* lptr_t;

DEVINL void copy16_to_lds(const unsigned short* g, unsigned char* l) {
  __builtin_amdgcn_global_load_lds((gptr_t)g, (lptr_t)l, 16, 0, 0);
}

// A GEMM's output as ks partial sums (N, ld).
struct Parts {
  const void* p;  // (ks, N, ld)
  long stride;    // elements between splits
  int ks, ld;
};

template <typename TP, int V>
DEVINL void fold_parts(const Parts& a, long t, int c, float* o) {
  const TP* row = (const TP*)a.p + t * (long)a.ld + c;
  ldv<V>(row, o);
  for (int s = 1; s < a.ks; ++s) {
    float u[V];
    ldv<V>(row + s * a.stride, u);
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] += u[j];
  }
}

// turns: frequency / 2 pi
DEVINL void rotation(int pos, double turns, float& c, float& s) {
  double r = (double)pos * turns;
  r -= rint(r);
  sincospif(2.f * (float)r, &s, &c);
}

// V consecutive elements d.. of a vector of `size` elements at column col of row
// t, those from r0 on to r0 + rdims turned, element r0 + k with r0 + rdims / 2 + k;
// zero from size on. cs: cosines of the pairs, then sines.
template <typename TP, int V>
DEVINL void turned_piece(const Parts& y, long t, int col, int d, int size, int r0,
                         int rdims, const float* cs, float* v) {
  const int half = rdims / 2, e0 = d - r0;
  if (d + V <= size && (e0 + V <= 0 || e0 >= rdims)) {
    fold_parts<TP, V>(y, t, col + d, v);
    return;
  }
  if (e0 >= 0 && e0 + V <= rdims && half % V == 0) {
    // a piece inside one half: its partners are a piece, too
    const bool first = e0 < half;
    float w[V];
    fold_parts<TP, V>(y, t, col + d, v);
    fold_parts<TP, V>(y, t, col + d + (first ? half : -half), w);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const int k = e0 + j - (first ? 0 : half);
      const float c = cs[k], s = cs[half + k];
      v[j] = first ? v[j] * c - w[j] * s : v[j] * c + w[j] * s;
    }
    return;
  }
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const int e = e0 + j;  // may straddle the border
    v[j] = 0.f;
    if (d + j >= size) continue;
    float x[1], w[1];
    fold_parts<TP, 1>(y, t, col + d + j, x);
    v[j] = x[0];
    if (e < 0 || e >= rdims) continue;
    const int k = e % half;
    fold_parts<TP, 1>(y, t, col + r0 + (e < half ? e + half : k), w);
    const float c = cs[k], s = cs[half + k];
    v[j] = e < half ? x[0] * c - w[0] * s : x[0] * c + w[0] * s;
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
  float* x;            // (N, W) f32 residual, row stride ldx, updated in place
  const void* parts;   // (ks, N, ldp) pending GEMM output, or null
  long pstride;        // elements between splits
  const void* routed;  // (N, top, ldr) weighted expert outputs, or null
  const int* ids;      // (N, top): < 0 = no routed row for this choice
  const float* idw;    // (N,) weight of the layer's own input, or null
  const void* hprev;   // (N, ldhp) that input
  const float* bias;   // (W,) of the pending GEMM, or null
  const float* bw;     // (W,) norm weight of what is pending; null = no norm
  const float* nw;     // (W,) norm weight; null = fold only
  const float* other;  // (N, W) f32, row stride ldx2: without nw, h is [x | other]
  void* h;             // (N, ldh) normed row, zero beyond W
  long ldx, ldx2;
  int W, ks, ldp, top, ldr, ldhp, ldh, groups;
  int post;            // the normed row becomes the residual
  float eps, alpha;    // alpha scales x before the sum
};

// LDS: W floats (the row) + at least 32 and groups * subs partial sums.
template <typename TP, typename T, int V, int BLOCK>
__global__ __launch_bounds__(BLOCK) void residual_norm_kernel(ResidualArgs a) {
  extern __shared__ float lds_row[];
  float* stat = lds_row + ((a.W + 3) & ~3);
  const long t = blockIdx.x;
  const int W = a.W;
  float* xr = a.x + t * a.ldx;
  const TP* pr = (const TP*)a.parts + t * a.ldp;
  const T* rr = (const T*)a.routed + t * (long)a.top * a.ldr;
  const T* hp = (const T*)a.hprev + t * (long)a.ldhp;
  const float iw = a.idw ? a.idw[t] : 0.f;

  // what is pending at columns i..
  auto owed = [&](int i, float* d) {
    float u[V];
    if (a.parts) {
      ldv<V>(pr + i, d);
      for (int s = 1; s < a.ks; ++s) {
        ldv<V>(pr + s * a.pstride + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) d[j] += u[j];
      }
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) d[j] = 0.f;
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
  };
  constexpr int NWAVE = BLOCK / WAVE;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const bool some = a.parts || a.routed;
  if (a.bw && some) {
    float ss = 0.f;
    for (int i = threadIdx.x * V; i < W; i += BLOCK * V) {
      float d[V];
      owed(i, d);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        lds_row[i + j] = d[j];
        ss += d[j] * d[j];
      }
    }
    ss = wave_reduce_sum(ss);
    if (lane == 0) stat[wave] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int k = 0; k < NWAVE; ++k) ss += stat[k];
    const float inv = 1.f / sqrtf(ss / (float)W + a.eps);
    __syncthreads();   // stat is written again below
    // a thread reads back what it wrote
    for (int i = threadIdx.x * V; i < W; i += BLOCK * V) {
      float v[V], w[V];
      ldv<V>(xr + i, v);
      ldv<V>(a.bw + i, w);
#pragma unroll
      for (int j = 0; j < V; ++j) {
        v[j] = v[j] * a.alpha + lds_row[i + j] * inv * w[j];
        lds_row[i + j] = v[j];
      }
      if (!a.post) stv<V>(xr + i, v);
    }
  } else {
    for (int i = threadIdx.x * V; i < W; i += BLOCK * V) {
      float v[V];
      ldv<V>(xr + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] *= a.alpha;
      if (some) {
        float d[V];
        owed(i, d);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] += d[j];
        if (!a.post) stv<V>(xr + i, v);
      }
#pragma unroll
      for (int j = 0; j < V; ++j) lds_row[i + j] = v[j];
    }
  }
  if (!a.nw) {
    if (!a.other) return;
    T* hr = (T*)a.h + t * (long)a.ldh;
    const float* xo = a.other + t * a.ldx2;
    // a thread reads back what it wrote
    for (int i = threadIdx.x * V; i < a.ldh; i += BLOCK * V) {
      float v[V];
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
      if (i < W) {
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] = lds_row[i + j];
      } else if (i < 2 * W) {
        ldv<V>(xo + i - W, v);
      }
      stv<V>(hr + i, v);
    }
    return;
  }
  __syncthreads();

  // sums of squares: every unit (a group, or an even share of one where
  // there are fewer groups than waves) belongs to one wave
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

struct EmbedArgs {
  const int* ids;
  const int* pos;
  const int* prev;      // token before each, < 0 = none; with pair_table only
  const void* table;    // (vocab, W)
  const void* pos_table;   // (max_pos, W) or null: learned positions
  const void* pair_table;  // (buckets + 1, W) or null: rows of token pairs
  const double* turns;     // ((W + 1) / 2,) or null: sines and cosines
  float* x;                // (N, copies * W)
  long buckets, mul_prev, mul_cur;
  int W, vocab, max_pos, copies;
  float scale;
};

// x[n] = scale * table[ids[n]] (+ pos_table[pos[n]]) (+ pair_table[row of the pair])
// (+ sin at 2i, cos at 2i + 1 of pos[n] * frequency i) in f32; indices are
// clamped. A token without a predecessor takes the pair table's last row.
template <typename T>
__global__ __launch_bounds__(256) void embed_rows_kernel(EmbedArgs a) {
  const long n = blockIdx.x;
  const int W = a.W, id = min(max(a.ids[n], 0), a.vocab - 1);
  const T* e = (const T*)a.table + (long)id * W;
  const T *p = nullptr, *q = nullptr;
  if (a.pos_table)
    p = (const T*)a.pos_table + (long)min(max(a.pos[n], 0), a.max_pos - 1) * W;
  if (a.pair_table) {
    const int b = a.prev[n];
    const long r = b < 0 ? a.buckets
                         : (min(b, a.vocab - 1) * a.mul_prev + id * a.mul_cur) %
                               a.buckets;
    q = (const T*)a.pair_table + r * W;
  }
  for (int i = threadIdx.x; i < W; i += 256) {
    float v = ldf(e + i) * a.scale;
    if (p) v += ldf(p + i);
    if (q) v += ldf(q + i);
    if (a.turns) {
      float c, s;
      rotation(max(a.pos[n], 0), a.turns[i / 2], c, s);
      v += i & 1 ? c : s;
    }
    for (int c = 0; c < a.copies; ++c) a.x[(n * a.copies + c) * W + i] = v;
  }
}

// ---------------------------------------------------------------------------

static constexpr int MAX_ROUTED = 1024;  // router outputs

struct RouteArgs {
  const float* parts;   // (ks, N, ld) router logits, f32
  long stride;
  const float* corr;    // (E + NI,) added to the scores for the choice only,
                        // or null
  int* ids;             // (N, top)
  float* wts;           // (N, top)
  float* idw;           // (N,) or null
  int ks, ld, off, E, NI, top;
  int sigmoid;          // scores: sigmoid of each logit, else softmax
  int renorm;           // the chosen scores are divided by their sum
  float scale;
};

DEVINL float router_logit(const RouteArgs& a, long t, int c) {
  const float* r = a.parts + t * a.ld + c;
  float v = r[0];
  for (int s = 1; s < a.ks; ++s) v += r[s * a.stride];
  return v;
}

// Chooses token t's experts; one wave. LDS: s and ch, MAX_ROUTED each.
DEVINL void route_row(const RouteArgs& a, long t, float* s, float* ch) {
  const int n = a.E + a.NI, lane = threadIdx.x & (WAVE - 1);
  float inv = 1.f;
  if (a.sigmoid) {
    for (int i = lane; i < n; i += WAVE)
      s[i] = 1.f / (1.f + expf(-router_logit(a, t, a.off + i)));
  } else {
    float mx = NEG_BIG;
    for (int i = lane; i < n; i += WAVE) {
      const float z = router_logit(a, t, a.off + i);
      s[i] = z;
      mx = fmaxf(mx, z);
    }
    mx = wave_reduce_max(mx);
    float sum = 0.f;
    for (int i = lane; i < n; i += WAVE) {
      s[i] = expf(s[i] - mx);
      sum += s[i];
    }
    inv = 1.f / wave_reduce_sum(sum);
  }
  for (int i = lane; i < n; i += WAVE) {
    s[i] *= inv;
    ch[i] = s[i] + (a.corr ? a.corr[i] : 0.f);
  }
  // every lane reads and writes its own columns only
  float idw = 0.f, total = 0.f, mine = 0.f;
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
      w = s[at] * a.scale;
      ch[at] = -__builtin_inff();
    }
    w = __shfl(w, at & (WAVE - 1));
    if (at >= a.E) idw += w;
    total += w;
    if (lane == k) mine = w;
    if (lane == 0) {
      a.ids[t * a.top + k] = at < a.E ? at : -1;
      if (!a.renorm || k >= WAVE) a.wts[t * a.top + k] = w;
    }
  }
  if (a.renorm) {
    const float f = a.scale / total;
    idw *= f;
    if (lane < a.top) a.wts[t * a.top + lane] = mine * f;
    if (lane == 0)
      for (int k = WAVE; k < a.top; ++k) a.wts[t * a.top + k] *= f;
  }
  if (lane == 0 && a.idw) a.idw[t] = idw;
}

struct PostArgs {
  const void* parts;    // (ks, N, ldp) input GEMM output
  long pstride;
  RouteArgs rt;         // router, and the shared expert's gate at rt column sg_off
  const float* qn;      // (H*dim,) q norm weight
  const float* kn;      // (G*dim,)
  void* q;              // (N, H, dkp)
  void* gate;           // (N, H*vdim) or null: the reader takes it from parts
  void* a2;             // (N, lda2): [attention | activation | zeros]
  void* kp;             // (np, G, P, dkp)
  void* vp;             // (np, G, dvp, P)
  const int* table;     // (S, maxp)
  const int* tok_seq;
  const int* tok_pos;
  int ks, ldp;
  int q_off, k_off, v_off, g_off, u_off, u2_off, sg_off;
  int H, G, dim, vdim, dkp, dvp, P, maxp;
  int has_kv;
  int act;              // 0 none, 1 xIELU, 2 silu(gate) * up
  int ff, act_col, lda2;
  float eps, xp, xq;
};

static constexpr int POST_BLOCK = 256;
static constexpr int POST_CHUNK = 2048;  // elementwise columns per workgroup
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
    if (a.rt.E + a.rt.NI > 0 && threadIdx.x < WAVE)
      route_row(a.rt, t, lds_sec, lds_sec + MAX_ROUTED);
    return;
  }

  // elementwise columns: [gate copy | activation and zero columns of a2]
  const int gn = a.gate ? a.H * a.vdim : 0;
  const int z0 = a.H * a.vdim;  // first column of a2 attention leaves alone
  const int total = gn + a.lda2 - z0;
  const int base = (role - 3) * POST_CHUNK;
  const int end = min(base + POST_CHUNK, total);
  float sg = 1.f;
  if (a.act == 2) sg = sigmoid_f(router_logit(a.rt, t, a.sg_off));
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

struct HeadPostArgs {
  Parts y;              // q, k, v columns
  const float* qb;      // biases (H*dim,), (G*dim,), (G*vdim,), or null
  const float* kb;
  const float* vb;
  const float* qn;      // (dim,) norm weights, shared by the heads
  const float* kn;
  void* q;              // (N, H, dkp)
  void* kp;             // (np, G, P, dkp)
  void* vp;             // (np, G, dvp, P)
  const int* table;     // (S, maxp)
  const int* tok_seq;
  const int* tok_pos;
  int q_off, k_off, v_off, H, G, dim, vdim, dkp, dvp, P, maxp;
  float eps;
  float temp_coef;      // query temperature 1 + coef ln(floor((pos+1)/every)+1)
  double temp_every;
};

// grid (N, (H + 2 G) / 4), a wave a head: q heads, k heads, v heads. LDS: four
// heads of dim.
template <typename TP, typename T, int V>
__global__ __launch_bounds__(256) void head_post_kernel(HeadPostArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds_head[];
  const long t = blockIdx.x;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int unit = blockIdx.y * 4 + wave;
  if (unit >= a.H + 2 * a.G) return;
  const int pos = a.tok_pos[t];
  const bool is_q = unit < a.H;
  if (!is_q && pos < 0) return;   // an empty slot writes no K/V
  long page = 0;
  int slot = 0;
  if (!is_q) {
    page = a.table[(long)a.tok_seq[t] * a.maxp + pos / a.P];
    slot = pos % a.P;
  }
  if (unit >= a.H + a.G) {
    const int g = unit - a.H - a.G;
    T* vp = (T*)a.vp + ((page * a.G + g) * a.dvp) * (long)a.P + slot;
    for (int d = lane; d < a.dvp; d += WAVE) {
      float v[1] = {0.f};
      if (d < a.vdim) {
        fold_parts<TP, 1>(a.y, t, a.v_off + g * a.vdim + d, v);
        if (a.vb) v[0] += a.vb[g * a.vdim + d];
      }
      stf(vp + (long)d * a.P, v[0]);
    }
    return;
  }
  const int h = is_q ? unit : unit - a.H;
  const float* bias = is_q ? a.qb : a.kb;
  const float* nw = is_q ? a.qn : a.kn;
  float* row = lds_head + wave * ((a.dim + 7) & ~7);
  float ss = 0.f;
  for (int i = lane * V; i < a.dim; i += WAVE * V) {
    float v[V], b[V];
    fold_parts<TP, V>(a.y, t, (is_q ? a.q_off : a.k_off) + h * a.dim + i, v);
    if (bias) {
      ldv<V>(bias + h * a.dim + i, b);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] += b[j];
    }
#pragma unroll
    for (int j = 0; j < V; ++j) {
      row[i + j] = v[j];
      ss += v[j] * v[j];
    }
  }
  float f = 1.f / sqrtf(wave_reduce_sum(ss) / (float)a.dim + a.eps);
  if (is_q && a.temp_coef != 0.f)
    f *= 1.f + a.temp_coef *
                   logf((float)(floor((double)(max(pos, 0) + 1) / a.temp_every) + 1.0));
  T* o = is_q ? (T*)a.q + (t * a.H + h) * (long)a.dkp
              : (T*)a.kp + ((page * a.G + h) * a.P + slot) * (long)a.dkp;
  // a lane reads back what it wrote
  for (int i = lane * V; i < a.dkp; i += WAVE * V) {
    float v[V], w[V];
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (i < a.dim) {
      ldv<V>(nw + i, w);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = row[i + j] * f * w[j];
    }
    stv<V>(o + i, v);
  }
}

struct RopePostArgs {
  Parts y;              // q, k, v columns
  const double* turns;  // (rdims / 2,)
  void* q;              // (N, H, M, dk)
  void* kp;             // (np, G, P, M * dk)
  void* vp;             // (np, G, dvp, P)
  const int* table;     // (S, maxp)
  const int* tok_seq;
  const int* tok_pos;
  int q_off, k_off, v_off, H, G, M, dim, vdim, rdims, dk, dvp, P, maxp;
  int per;              // units of a workgroup
  float amp;            // factor of cosine and sine
};

// grid (N, units / per); units are the H M queries, G M keys and G values of a
// row. LDS: cosine and sine of every pair.
template <typename TP, typename T, int V>
__global__ __launch_bounds__(256) void rope_post_kernel(RopePostArgs a) {
  extern __shared__ float lds_cs[];
  const long t = blockIdx.x;
  const int tid = threadIdx.x, half = a.rdims / 2, pos = a.tok_pos[t];
  for (int k = tid; k < half; k += 256) {
    float c, s;
    rotation(max(pos, 0), a.turns[k], c, s);
    lds_cs[k] = c * a.amp;
    lds_cs[half + k] = s * a.amp;
  }
  __syncthreads();
  const int nq = a.H * a.M, nk = a.G * a.M;
  const int u0 = blockIdx.y * a.per, u1 = min(u0 + a.per, nq + nk + a.G);
  long page = 0;
  int slot = 0;
  if (pos >= 0) {
    page = a.table[(long)a.tok_seq[t] * a.maxp + pos / a.P];
    slot = pos % a.P;
  }
  const int pieces = max(a.dk, a.dvp) / V;
  for (int idx = tid; idx < (u1 - u0) * pieces; idx += 256) {
    const int u = u0 + idx / pieces, d = idx % pieces * V;
    if (u >= nq && pos < 0) break;   // an empty slot writes no K/V
    float v[V];
    if (u >= nq + nk) {
      if (d >= a.dvp) continue;
      const int g = u - nq - nk;
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
      if (d + V <= a.vdim) {
        fold_parts<TP, V>(a.y, t, a.v_off + g * a.vdim + d, v);
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j)
          if (d + j < a.vdim)
            fold_parts<TP, 1>(a.y, t, a.v_off + g * a.vdim + d + j, v + j);
      }
      T* vp = (T*)a.vp + ((page * a.G + g) * a.dvp + d) * (long)a.P + slot;
#pragma unroll
      for (int j = 0; j < V; ++j) stf(vp + j * a.P, v[j]);
      continue;
    }
    if (d >= a.dk) continue;
    const bool is_q = u < nq;
    const int i = is_q ? u : u - nq;
    turned_piece<TP, V>(a.y, t, (is_q ? a.q_off : a.k_off) + i * a.dim, d, a.dim, 0,
                        a.rdims, lds_cs, v);
    T* o = is_q ? (T*)a.q + (t * nq + i) * a.dk
                : (T*)a.kp + ((page * a.G + i / a.M) * a.P + slot) * (long)(a.M * a.dk) +
                      i % a.M * a.dk;
    stv<V>(o + d, v);
  }
}

struct FfPostArgs {
  Parts y;              // feed-forward columns, or null
  RouteArgs rt;         // E = 0: no router
  void* out;            // (N, ldo), zero beyond ff
  int act;              // 1 silu(gate) * up, 2 relu(up)^2
  int u_off, u2_off, ff, ldo;  // act 1: gate, up; act 2: up
};

// grid (N, 1 + chunks): y = 0 router, 1.. elementwise.
template <typename TP, typename T, int V>
__global__ __launch_bounds__(POST_BLOCK) void ff_post_kernel(FfPostArgs a) {
  __shared__ float lds_rt[2 * MAX_ROUTED];
  const long t = blockIdx.x;
  if (blockIdx.y == 0) {
    if (a.rt.E + a.rt.NI > 0 && threadIdx.x < WAVE)
      route_row(a.rt, t, lds_rt, lds_rt + MAX_ROUTED);
    return;
  }
  const int base = (blockIdx.y - 1) * POST_CHUNK;
  const int end = min(base + POST_CHUNK, a.ldo);
  for (int i = base + threadIdx.x * V; i < end; i += POST_BLOCK * V) {
    float v[V], u[V];
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (i < a.ff) {
      fold_parts<TP, V>(a.y, t, a.u_off + i, v);
      if (a.act == 1) {
        fold_parts<TP, V>(a.y, t, a.u2_off + i, u);
#pragma unroll
        for (int j = 0; j < V; ++j) v[j] = v[j] * sigmoid_f(v[j]) * u[j];
      } else {
#pragma unroll
        for (int j = 0; j < V; ++j) {
          const float r = fmaxf(v[j], 0.f);
          v[j] = r * r;
        }
      }
    }
    stv<V>((T*)a.out + t * (long)a.ldo + i, v);
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
