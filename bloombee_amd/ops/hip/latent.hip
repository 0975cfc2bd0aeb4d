// Latent attention over ragged batches: what a token leaves in the cache is one
// normed latent c and one rotated key part shared by all heads, [c | r] in one
// key page plane. Per-head keys and values are linear in c.
//
//  latent_post_kernel    norms the query latent, norms c, rotates r, writes
//                        the page slot.
//  latent_rope_kernel    queries of prompt rows: [unrotated | rotated].
//  latent_scatter_kernel keys and values of a context, made from its latents by
//                        one GEMM, into pages of the prompt attention kernel.
//  latent_absorb_kernel  queries of decoded rows, taken into the latent space:
//                        q_lat = W_uk^T q, beside the rotated part. One head's
//                        query then meets [c | r] itself.
//  attn_latent_decode_kernel  decoded rows: every key tile is read once for up
//                        to 32 heads, for the scores by rows and for the values
//                        by columns (transposing LDS reads).
//  latent_combine_kernel folds the splits and the sink.
//  latent_output_kernel  applies W_uv and the sigmoid output gate.
//
// Rotary pairs are (i, i + dims/2). Angles are reduced in double, in turns.

#pragma once
#include "common.h"
#include "rows.hip"

struct LatentPostArgs {
  Parts y;              // [query latent | c | r | gate] columns
  const float* qn;      // (q_rank,)
  const float* cn;      // (rank,)
  const double* turns;  // (rdims / 2,)
  void* cq;             // (N, ldq), zero beyond q_rank
  void* gate;           // (N, gn) or null
  void* kp;             // (np, 1, P, ck)
  const int* table;
  const int* tok_seq;
  const int* tok_pos;
  int q_off, c_off, g_off, q_rank, rank, rot, rdims, rp, ck, ldq, gn, P, maxp;
  int has_kv;
  float eps, amp;       // amp: factor of cosine and sine
};

// Section of n columns into LDS; returns 1 / rms.
template <typename TP, int V>
DEVINL float stage_norm(const Parts& y, long t, int off, int n, float eps,
                        float* lds, float* red) {
  float ss = 0.f;
  for (int i = threadIdx.x * V; i < n; i += 256 * V) {
    float v[V];
    fold_parts<TP, V>(y, t, off + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) {
      lds[i + j] = v[j];
      ss += v[j] * v[j];
    }
  }
  ss = wave_reduce_sum(ss);
  if ((threadIdx.x & (WAVE - 1)) == 0) red[threadIdx.x / WAVE] = ss;
  __syncthreads();
  return 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)n + eps);
}

// o[0..cols) = x * inv * w, zero from n on; n and cols are multiples of V.
template <typename T, int V>
DEVINL void scale_row(T* o, const float* x, const float* w, float inv, int n,
                      int cols) {
  for (int i = threadIdx.x * V; i < cols; i += 256 * V) {
    float v[V];
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (i < n) {
      ldv<V>(w + i, v);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] *= x[i + j] * inv;
    }
    stv<V>(o + i, v);
  }
}

// grid (N, 2 + gate chunks of 2048): y = 0 query latent, 1 page slot, 2.. gate
template <typename TP, typename T, int V>
__global__ __launch_bounds__(256) void latent_post_kernel(LatentPostArgs a) {
  extern __shared__ float lds_sec[];
  __shared__ float red[4];
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  if (blockIdx.y == 0) {
    const float inv = stage_norm<TP, V>(a.y, t, a.q_off, a.q_rank, a.eps,
                                        lds_sec, red);
    scale_row<T, V>((T*)a.cq + t * (long)a.ldq, lds_sec, a.qn, inv, a.q_rank,
                    a.ldq);
    return;
  }
  if (blockIdx.y == 1) {
    const int pos = a.tok_pos[t];
    if (!a.has_kv || pos < 0) return;
    const float inv = stage_norm<TP, V>(a.y, t, a.c_off, a.rank, a.eps,
                                        lds_sec, red);
    const long page = a.table[(long)a.tok_seq[t] * a.maxp + pos / a.P];
    T* o = (T*)a.kp + (page * a.P + pos % a.P) * a.ck;
    scale_row<T, V>(o, lds_sec, a.cn, inv, a.rank, a.rp);
    const int half = a.rdims / 2;
    for (int i = tid; i < a.ck - a.rp; i += 256) {
      float v[1] = {0.f};
      if (i < a.rot) fold_parts<TP, 1>(a.y, t, a.c_off + a.rank + i, v);
      if (i < a.rdims) {
        const int k = i % half;
        float w[1], c, s;
        fold_parts<TP, 1>(a.y, t, a.c_off + a.rank + (i < half ? i + half : k), w);
        rotation(pos, a.turns[k], c, s);
        c *= a.amp;
        s *= a.amp;
        v[0] = i < half ? v[0] * c - w[0] * s : v[0] * c + w[0] * s;
      }
      stf(o + a.rp + i, v[0]);
    }
    return;
  }
  const int base = (blockIdx.y - 2) * 2048;
  const int end = min(base + 2048, a.gn);
  for (int i = base + tid * V; i < end; i += 256 * V) {
    float v[V];
    fold_parts<TP, V>(a.y, t, a.g_off + i, v);
    stv<V>((T*)a.gate + t * (long)a.gn + i, v);
  }
}

struct LatentQueryArgs {
  Parts y;              // (N, H * (dim + rot))
  const double* turns;
  const int* tok_pos;
  const int* cu;        // decoded rows: row = cu[list[i]]
  const int* list;
  const void* wk;       // (H, rp, dimp): W_uk^T, zero padded
  void* q;              // rope: (N, H, ldq); absorb: (n_list, H, ck)
  int n_list, H, dim, rot, rdims, rp, ck, dimp, ldq;
  float amp;            // factor of cosine and sine
};

// grid N: a row's queries, [dim unrotated | rot rotated | zeros] per head
template <typename TP, typename T, int V>
__global__ __launch_bounds__(256) void latent_rope_kernel(LatentQueryArgs a) {
  extern __shared__ float lds_cs[];  // cos, sin of every pair
  const long t = blockIdx.x;
  const int tid = threadIdx.x, half = a.rdims / 2;
  const int pos = max(a.tok_pos[t], 0);
  for (int k = tid; k < half; k += 256) {
    float c, s;
    rotation(pos, a.turns[k], c, s);
    lds_cs[k] = c * a.amp;
    lds_cs[half + k] = s * a.amp;
  }
  __syncthreads();
  T* q = (T*)a.q + t * (long)a.H * a.ldq;
  const int per = a.ldq / V;
  for (int idx = tid; idx < a.H * per; idx += 256) {
    const int h = idx / per, d = (idx % per) * V;
    float v[V];
    turned_piece<TP, V>(a.y, t, h * (a.dim + a.rot), d, a.dim + a.rot, a.dim,
                        a.rdims, lds_cs, v);
    stv<V>(q + (long)h * a.ldq + d, v);
  }
}

// grid (rp / 128 + 1, H, rows / 32): 32 listed rows of one head times W_uk^T;
// the last x block writes the rotated part and the zero columns.
template <typename TP, int V>
__global__ __launch_bounds__(256) void latent_absorb_kernel(LatentQueryArgs a) {
  extern __shared__ __attribute__((aligned(16))) unsigned short lds_q[];
  const int tid = threadIdx.x, h = blockIdx.y, m0 = blockIdx.z * 32;
  const int M = min(32, a.n_list - m0);
  const int col = h * (a.dim + a.rot);
  unsigned short* out = (unsigned short*)a.q;
  if (blockIdx.x == gridDim.x - 1) {
    // a pair a thread, then what does not turn
    const int half = a.rdims / 2, rest = a.ck - a.rp - a.rdims;
    for (int idx = tid; idx < M * half; idx += 256) {
      const int m = idx / half, k = idx % half;
      const long row = a.cu[a.list[m0 + m]];
      float u[1], v[1], c, s;
      fold_parts<TP, 1>(a.y, row, col + a.dim + k, u);
      fold_parts<TP, 1>(a.y, row, col + a.dim + half + k, v);
      rotation(max(a.tok_pos[row], 0), a.turns[k], c, s);
      c *= a.amp;
      s *= a.amp;
      unsigned short* o = out + ((long)(m0 + m) * a.H + h) * a.ck + a.rp + k;
      o[0] = cvt_bf(u[0] * c - v[0] * s);
      o[half] = cvt_bf(v[0] * c + u[0] * s);
    }
    for (int idx = tid; idx < M * rest; idx += 256) {
      const int m = idx / rest, e = a.rdims + idx % rest;
      float v[1] = {0.f};
      if (e < a.rot)
        fold_parts<TP, 1>(a.y, a.cu[a.list[m0 + m]], col + a.dim + e, v);
      out[((long)(m0 + m) * a.H + h) * a.ck + a.rp + e] = cvt_bf(v[0]);
    }
    return;
  }
  const int ldr = a.dimp + 8, pieces = a.dimp / V;
  for (int idx = tid; idx < 32 * pieces; idx += 256) {
    const int m = idx / pieces, d = idx % pieces * V;
    float v[V];
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (m < M && d < a.dim)
      fold_parts<TP, V>(a.y, a.cu[a.list[m0 + m]], col + d, v);
    stv<V>(lds_q + m * ldr + d, v);
  }
  __syncthreads();
  const int wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
#pragma unroll
  for (int nt = 0; nt < 2; ++nt) {
    const int n0 = blockIdx.x * 128 + nt * 64 + wave * 16;
    if (n0 >= a.rp) return;
    const unsigned short* w = (const unsigned short*)a.wk +
                              ((long)h * a.rp + n0 + li) * a.dimp + hi * 8;
    f32x4 acc[2];
    acc[0] = acc[1] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < a.dimp; k0 += 128) {
      short8 wf[4];
#pragma unroll
      for (int u = 0; u < 4; ++u)
        wf[u] = k0 + u * 32 < a.dimp
                    ? *reinterpret_cast<const short8*>(w + k0 + u * 32) : short8{};
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int k = min(k0 + u * 32, a.dimp - 32);
#pragma unroll
        for (int m = 0; m < 2; ++m) {
          const bf16x8 qf = as_bf16x8(*reinterpret_cast<const short8*>(
              lds_q + (m * 16 + li) * ldr + k + hi * 8));
          acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              qf, as_bf16x8(wf[u]), acc[m], 0, 0, 0);
        }
      }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = m * 16 + hi * 4 + r;
        if (row < M)
          out[((long)(m0 + row) * a.H + h) * a.ck + n0 + li] = cvt_bf(acc[m][r]);
      }
  }
}

struct LatentScatterArgs {
  const unsigned short* y;    // (npg * P, ldy): [H x dim keys | H x vdim values]
  const unsigned short* ctx;  // (npg, P, ck) page copies, for the rotated part
  const int* valid;           // (npg,) tokens in use of every page
  unsigned short* k;          // (npg, H, P, dkp)
  unsigned short* v;          // (npg, H, dvp, P)
  int ldy, H, dim, rot, vdim, rp, ck, dkp, dvp, P;
};

// grid (npg, H). V = 8: sizes are multiples of it.
template <int V>
__global__ __launch_bounds__(256) void latent_scatter_kernel(LatentScatterArgs a) {
  const long pg = blockIdx.x;
  const int h = blockIdx.y, tid = threadIdx.x;
  const int n = a.valid[pg];
  const unsigned short* y = a.y + pg * a.P * a.ldy;
  unsigned short* k = a.k + (pg * a.H + h) * (long)a.P * a.dkp;
  const int per = a.dkp / V;
  for (int idx = tid; idx < a.P * per; idx += 256) {
    const int r = idx / per, d = (idx % per) * V;
    float v[V];
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = 0.f;
    if (d + V <= a.dim) {
      ldv<V>(y + (long)r * a.ldy + h * a.dim + d, v);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const int e = d + j - a.dim;
        if (e < 0) v[j] = bf2f(y[(long)r * a.ldy + h * a.dim + d + j]);
        else if (e < a.rot) v[j] = bf2f(a.ctx[(pg * a.P + r) * a.ck + a.rp + e]);
      }
    }
    stv<V>(k + (long)r * a.dkp + d, v);
  }
  unsigned short* vo = a.v + (pg * a.H + h) * (long)a.dvp * a.P;
  const unsigned short* vy = y + a.H * a.dim + h * a.vdim;
  if constexpr (V == 8) {
    // 8 x 8 blocks, turned in a lane's registers
    for (int idx = tid; idx < a.dvp / 8 * (a.P / 8); idx += 256) {
      const int d = idx % (a.dvp / 8) * 8, r0 = idx / (a.dvp / 8) * 8;
      short8 in[8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        in[j] = r0 + j < n && d < a.vdim
                    ? *reinterpret_cast<const short8*>(vy + (long)(r0 + j) * a.ldy + d)
                    : short8{};
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        short8 o;
#pragma unroll
        for (int j = 0; j < 8; ++j) o[j] = in[j][e];
        *reinterpret_cast<short8*>(vo + (long)(d + e) * a.P + r0) = o;
      }
    }
  } else {
    for (int idx = tid; idx < a.dvp * (a.P / 8); idx += 256) {
      const int d = idx % a.dvp, r0 = idx / a.dvp * 8;
      short8 o = short8{};
      if (d < a.vdim)
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (r0 + j < n) o[j] = (short)vy[(long)(r0 + j) * a.ldy + d];
      *reinterpret_cast<short8*>(vo + (long)d * a.P + r0) = o;
    }
  }
}

struct LatentDecodeArgs {
  const unsigned short* q;   // (n_list, H, ck)
  const unsigned short* kp;  // (np, 1, P, ck)
  const int* table;
  const int* q_start;        // (S,) position of a listed sequence's one token
  const int* list;
  float* pml;   // (n_list, H, n_split, 2): max (log2 units) and sum
  float* pacc;  // (n_list, H, n_split, rp)
  int H, p_log2, maxp, window, n_split;
  float scale;
};

typedef __attribute__((address_space(3))) short4v lds_short4;

// 4 rows of 16-bit elements by columns: lane i of 16 gets column i of the rows
// whose pieces of four the lanes point at (lane j*4 + c: row j, columns c*4..).
DEVINL short4v read_columns(const unsigned short* p) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4*)p);
}

// Fragment of 8 rows x 16 columns, rows r0.. of a tile with row stride ld:
// lane (li, hi) gets column perm-of-li, rows r0 + hi*8 .. +7. col points this
// lane's group of four columns at its place in the row.
DEVINL bf16x8 column_frag(const unsigned short* tile, int ld, int r0, int col,
                          int li, int hi) {
  const unsigned short* p = tile + (r0 + hi * 8 + li / 4) * ld + col;
  const short4v a = read_columns(p), b = read_columns(p + 4 * ld);
  short8 v;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    v[j] = a[j];
    v[j + 4] = b[j];
  }
  return as_bf16x8(v);
}

// Row stride of a key tile, in elements: rows and columns are read without
// bank conflicts.
constexpr int latent_tile_ld(int ck) { return ck + (ck / 2 % 64 < 32 ? 24 : 8); }

// grid (n_list * chunks of 16 * HG heads, n_split), four waves for each of HG
// groups of 16 heads. ck = ND * 64 + NR * 32; a wave owns every fourth
// 16-column tile of the values.
template <int ND, int NR, int HG>
__global__ __launch_bounds__(256 * HG, 3 - HG) void attn_latent_decode_kernel(
    LatentDecodeArgs a) {
  constexpr int KT = 64, RP = ND * 64, CK = RP + NR * 32, NKK = CK / 32;
  constexpr int LDK = latent_tile_ld(CK), LDS_S = KT + 4;
  constexpr int LANES = 256 * HG / KT;   // threads that stage one row
  constexpr int NP = (CK / 8 + LANES - 1) / LANES;  // 16 B pieces each
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_dec[];
  unsigned short* kt = (unsigned short*)lds_dec;
  const int tid = threadIdx.x;
  const int wv = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int wave = wv & 3, grp = wv >> 2;
  float* sc = (float*)(lds_dec + KT * LDK * 2) + grp * 16 * LDS_S;

  const int nch = (a.H + 16 * HG - 1) / (16 * HG);
  const int unit = blockIdx.x, i = unit / nch;
  const int h0 = unit % nch * 16 * HG + grp * 16;
  const int s = a.list[i];
  const int pos = a.q_start[s];
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int* table = a.table + (long)s * a.maxp;

  const int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  const int t_beg = lo / KT;
  const int t_all = pos < 0 ? 0 : pos / KT + 1 - t_beg;
  const int t_lo = t_beg + t_all * blockIdx.y / a.n_split;
  const int t_hi = t_beg + t_all * (blockIdx.y + 1) / a.n_split;

  // a thread stages pieces piece, piece + LANES, .. of one row of the tile; the
  // row's page is looked up a tile ahead
  const int srow = tid / LANES, piece = tid % LANES;
  short8 reg[NP];
  auto page_of = [&](int t) {
    return table[min(t * KT + srow, max(pos, 0)) >> a.p_log2];
  };
  auto fetch = [&](int t, int page) {
    const int key = min(t * KT + srow, pos);
    const unsigned short* kp =
        a.kp + (((long)page << a.p_log2) + (key & ((1 << a.p_log2) - 1))) * CK;
#pragma unroll
    for (int n = 0; n < NP; ++n) {
      const int pc = piece + n * LANES;
      if ((CK / 8) % LANES == 0 || pc < CK / 8)
        reg[n] = *reinterpret_cast<const short8*>(kp + pc * 8);
    }
  };
  int page = page_of(t_lo);
  if (t_lo < t_hi) {
    fetch(t_lo, page);
    page = page_of(t_lo + 1);
  }

  bf16x8 qf[NKK];
  const unsigned short* qp =
      a.q + ((long)i * a.H + min(h0 + li, a.H - 1)) * CK + hi * 8;
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk)
    qf[kk] = as_bf16x8(*reinterpret_cast<const short8*>(qp + kk * 32));
  // the queries arrive here: else the waits for them sit in the loop and take
  // the next tile's loads along
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk) asm volatile("" : "+v"(qf[kk]));

  float m2 = NEG_BIG, l = 0.f;
  f32x4 acc[ND];
#pragma unroll
  for (int n = 0; n < ND; ++n) acc[n] = (f32x4){0.f, 0.f, 0.f, 0.f};
  const float sc2 = a.scale * LOG2E;

  for (int t = t_lo; t < t_hi; ++t) {
    __syncthreads();  // the last tile is read
#pragma unroll
    for (int n = 0; n < NP; ++n) {
      const int pc = piece + n * LANES;
      if ((CK / 8) % LANES == 0 || pc < CK / 8)
        *reinterpret_cast<short8*>(kt + srow * LDK + pc * 8) = reg[n];
    }
    __syncthreads();
    if (t + 1 < t_hi) {
      fetch(t + 1, page);
      page = page_of(t + 2);
    }
    f32x4 st[2];  // two chains
    st[0] = st[1] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk) {
      const bf16x8 kf = as_bf16x8(*reinterpret_cast<const short8*>(
          kt + (wave * 16 + li) * LDK + kk * 32 + hi * 8));
      st[kk & 1] =
          __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[kk], st[kk & 1], 0, 0, 0);
    }
    *reinterpret_cast<f32x4*>(sc + li * LDS_S + wave * 16 + hi * 4) =
        st[0] + st[1];
    __syncthreads();
    // every wave takes the softmax of the whole tile
    float p[2][8];
    float rm = NEG_BIG;
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(
          sc + li * LDS_S + (q >> 1) * 32 + hi * 8 + (q & 1) * 4);
#pragma unroll
      for (int r = 0; r < 4; ++r) p[q >> 1][(q & 1) * 4 + r] = v[r] * sc2;
    }
    if (t * KT < lo || t * KT + KT - 1 > pos) {
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int key = t * KT + hf * 32 + hi * 8 + j;
          if (key < lo || key > pos) p[hf][j] = NEG_BIG;
        }
    }
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int j = 0; j < 8; ++j) rm = fmaxf(rm, p[hf][j]);
    rm = fmaxf(rm, __shfl_xor(rm, 16));
    rm = fmaxf(rm, __shfl_xor(rm, 32));
    const float mn = fmaxf(m2, rm);  // every tile has a visible key
    const float corr = fast_exp2(m2 - mn);
    float ps = 0.f;
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        p[hf][j] = fast_exp2(p[hf][j] - mn);
        ps += p[hf][j];
      }
    ps += __shfl_xor(ps, 16);
    ps += __shfl_xor(ps, 32);
    l = l * corr + ps;
    m2 = mn;
#pragma unroll
    for (int n = 0; n < ND; ++n)
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[n][r] *= corr;
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      // weights as two bf16, so that their rounding does not show
      bf16x8 ph, pl;
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        ph[j] = (__bf16)p[hf][j];
        pl[j] = (__bf16)(p[hf][j] - (float)ph[j]);
      }
#pragma unroll
      for (int n = 0; n < ND; ++n) {
        const bf16x8 vf = column_frag(kt, LDK, hf * 32,
                                      (n * 4 + wave) * 16 + (li & 3) * 4, li, hi);
        acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph, acc[n], 0, 0, 0);
        acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, acc[n], 0, 0, 0);
      }
    }
  }
  const int h = h0 + li;
  if (h >= a.H) return;
  const long u = ((long)i * a.H + h) * a.n_split + blockIdx.y;
  if (wave == 0 && hi == 0) {
    a.pml[u * 2] = m2;
    a.pml[u * 2 + 1] = l;
  }
#pragma unroll
  for (int n = 0; n < ND; ++n)
    *reinterpret_cast<f32x4*>(a.pacc + u * RP + (n * 4 + wave) * 16 + hi * 4) =
        acc[n];
}

// grid n_list * H: one row's head, folded over the splits, to bf16 (H, n, rp).
template <int NS>  // splits at most
__global__ __launch_bounds__(128) void latent_combine_kernel(
    const float* __restrict__ pml, const float* __restrict__ pacc,
    const float* __restrict__ sinks, unsigned short* __restrict__ o, int n,
    int H, int rp, int n_split) {
  const long u = blockIdx.x, u0 = u * n_split;
  float w[NS];
  float mx = sinks ? sinks[u % H] * LOG2E : NEG_BIG;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    w[i] = i < n_split ? pml[(u0 + i) * 2] : NEG_BIG;
    mx = fmaxf(mx, w[i]);
  }
  float l = sinks ? fast_exp2(sinks[u % H] * LOG2E - mx) : 0.f;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    w[i] = i < n_split ? fast_exp2(w[i] - mx) : 0.f;
    if (i < n_split) l += pml[(u0 + i) * 2 + 1] * w[i];
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
  for (int d = threadIdx.x * 4; d < rp; d += 512) {
    f32x4 v[NS];
#pragma unroll
    for (int i = 0; i < NS; ++i)
      v[i] = i < n_split ? *reinterpret_cast<const f32x4*>(pacc + (u0 + i) * rp + d)
                         : (f32x4){0.f, 0.f, 0.f, 0.f};
    float s[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NS; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) s[r] += v[i][r] * w[i];
#pragma unroll
    for (int r = 0; r < 4; ++r) s[r] *= inv;
    stv<4>(o + (u % H * n + u / H) * rp + d, s);
  }
}

struct LatentOutputArgs {
  const unsigned short* o;     // (H, n_list, rp)
  const unsigned short* wv;    // (H, vp, rp): W_uv, zero padded
  const unsigned short* gate;  // row stride ldg, or null
  unsigned short* out;         // row stride ldo
  const int* cu;
  const int* list;
  long ldg, ldo;
  int n_list, H, rp, vdim, vp;
};

// grid (vp / 64, H, rows / 16)
__global__ __launch_bounds__(256) void latent_output_kernel(LatentOutputArgs a) {
  const int tid = threadIdx.x, h = blockIdx.y, m0 = blockIdx.z * 16;
  const int M = min(16, a.n_list - m0);
  const int wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int n0 = blockIdx.x * 64 + wave * 16, d = n0 + li;
  // what the epilogue needs is looked up while the product runs
  long row[4];
  float g[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    row[r] = a.cu[a.list[m0 + min(hi * 4 + r, M - 1)]];
    g[r] = a.gate && d < a.vdim ? bf2f(a.gate[row[r] * a.ldg + h * a.vdim + d])
                                : 0.f;
  }
  const unsigned short* w = a.wv + ((long)h * a.vp + n0 + li) * a.rp + hi * 8;
  const unsigned short* op =
      a.o + ((long)h * a.n_list + m0 + min(li, M - 1)) * a.rp + hi * 8;
  f32x4 acc = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < a.rp; k0 += 256) {
    short8 wf[8], of[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) {
      const int k = k0 + u * 32;
      const bool in = k < a.rp;
      wf[u] = in ? *reinterpret_cast<const short8*>(w + k) : short8{};
      of[u] = in ? *reinterpret_cast<const short8*>(op + k) : short8{};
    }
#pragma unroll
    for (int u = 0; u < 8; ++u)
      acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(as_bf16x8(of[u]),
                                                    as_bf16x8(wf[u]), acc, 0, 0, 0);
  }
  if (d >= a.vdim) return;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    if (hi * 4 + r >= M) continue;
    const float v = a.gate ? acc[r] * sigmoid_f(g[r]) : acc[r];
    a.out[row[r] * a.ldo + h * a.vdim + d] = cvt_bf(v);
  }
}
