// Paged attention over ragged batches: rows of many sequences, each with its
// own position, with a sliding window, chunks (a row sees its own stretch of
// positions, counted from the sequence's start), a linear distance bias
// (score - slope_h * (i - j)), separate key and value sizes, grouped key/value
// heads, a sink (one more score per head, unscaled and without a value) and a
// sigmoid output gate in the epilogue. Every one of these is a parameter;
// window 0, chunk 0, null slopes, null sinks and a null gate switch them off.
//
// Two MFMA kernels and one plain kernel:
//  * attn_ragged_prefill_kernel: sequences that bring two tokens or more. The
//    rows of a tile are (token, head of the group) pairs, so a K/V tile in LDS
//    serves all heads of its group.
//  * attn_ragged_decode_kernel: sequences that bring one. Columns are the
//    heads of the group; only the visible range [i - window + 1, i] is walked
//    and split over waves and workgroups.
//  * attn_ragged_simple_kernel: one wave per (row, head), f32 arithmetic on
//    any element type and any head size. Without value pages the values are
//    the first vdim elements of the keys. Keys may hold several maps side by
//    side, of which query heads take turns.
//
// Both MFMA kernels compute S^T = K Q^T and O^T = V^T P^T. The rows of a
// 32-key tile are handed to the two score MFMAs in the order
//     MFMA n, row a*4+b  <->  key a*8 + n*4 + b        (a, b < 4)
// so that the score registers of a lane (MFMA n, rows hi*4..hi*4+3) are the
// eight consecutive keys hi*8..hi*8+7: exactly the B fragment of O^T. P never
// leaves the lane's registers.
//
// The weights are f32. The P.V product takes them as a sum of two bf16 (the
// value and what its rounding lost), so their rounding does not show.

#pragma once
#include "common.h"
#include "rows.hip"

struct AttnArgs {
  const void* q;        // (N, H, dkp)
  const void* kp;       // (np, G, P, dkp)
  const void* vp;       // (np, G, dvp, P) or null: values are key prefixes
  const int* table;     // (S, maxp)
  const int* tok_seq;   // (N,)
  const int* tok_pos;   // (N,) -1 = empty slot
  const int* cu;        // (S + 1,)
  const int* q_start;   // (S,)
  const int* list;      // sequences of this launch
  const float* slopes;  // (H,) or null
  const float* sinks;   // (H,) or null
  const void* gate;     // row stride ldg, (H*vdim) columns; or null
  void* out;            // row stride ldo, (H*vdim) columns
  float* pml;           // decode splits: (units, 16, 2) max and sum
  float* pacc;          // (units, 16, dvp)
  long ldg, ldo;
  int H, G, dim, vdim, dkp, dvp, P, maxp, window, chunk, n_split;
  int maps;             // of a key (plain kernel): its rows are maps * dkp long
  float scale;
};

// First position that a row sees.
DEVINL int first_key(const AttnArgs& a, int pos) {
  int lo = a.window > 0 ? max(0, pos - a.window + 1) : 0;
  if (a.chunk > 0) lo = max(lo, pos - max(pos, 0) % a.chunk);
  return lo;
}

// Takes a sink (log2 units) into a row's softmax: returns the factor of its
// accumulated values.
DEVINL float add_sink(float sink2, float m2, float& l) {
  const float mn = fmaxf(m2, sink2);
  const float c = fast_exp2(m2 - mn);
  l = l * c + fast_exp2(sink2 - mn);
  return c;
}

// Four consecutive output columns of one row, gated.
DEVINL void store_out4(const AttnArgs& a, long row, int h, int d, const float* o) {
  unsigned short* op = (unsigned short*)a.out + row * a.ldo + h * a.vdim + d;
  const unsigned short* gp =
      (const unsigned short*)a.gate + row * a.ldg + h * a.vdim + d;
  const bool vec = ((a.vdim | (int)a.ldo | (int)a.ldg) & 3) == 0;
  if (vec && d + 4 <= a.vdim) {
    float v[4];
    if (a.gate) {
      float g[4];
      ldv<4>(gp, g);
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = o[j] * sigmoid_f(g[j]);
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j) v[j] = o[j];
    }
    stv<4>(op, v);
    return;
  }
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (d + j < a.vdim)
      op[j] = f2bf(a.gate ? o[j] * sigmoid_f(bf2f(gp[j])) : o[j]);
}

// p[0..7] -> two bf16 fragments whose sum is p.
DEVINL void split_bf16(const float* p, bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    hi[j] = (__bf16)p[j];
    lo[j] = (__bf16)(p[j] - (float)hi[j]);
  }
}

// ---------------------------------------------------------------------------
// prefill: grid (row tiles of the longest portion, G, sequences)
// ---------------------------------------------------------------------------

template <int DK, int DV, int QC>  // QC: 16-row column tiles per wave
__global__ __launch_bounds__(256, DK + DV > 256 ? 1 : 2) void attn_ragged_prefill_kernel(AttnArgs a) {
  constexpr int KT = 64;                 // keys per tile
  constexpr int KROW = DK * 2 + 16;      // bytes
  constexpr int VROW = KT * 2 + 16;
  constexpr int NKK = DK / 32, ND = DV / 16;
  constexpr int KCH = KT * (DK / 8) / 256;  // 16 B pieces per thread
  constexpr int VCH = DV * (KT / 8) / 256;
  static_assert(KCH >= 1 && VCH >= 1, "tile smaller than the workgroup");
  __shared__ __attribute__((aligned(16))) unsigned char
      lds[KT * KROW + DV * VROW];
  unsigned char* k_lds = lds;
  unsigned char* v_lds = lds + KT * KROW;

  const int s = a.list[blockIdx.z];
  const int g = blockIdx.y;
  const int Hg = a.H / a.G;
  const int t0 = a.cu[s], T = a.cu[s + 1] - t0, qs = a.q_start[s];
  const int R = T * Hg;
  const int base = blockIdx.x * (64 * QC);
  if (base >= R) return;
  const int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int* table = a.table + (long)s * a.maxp;
  const unsigned short* kpool = (const unsigned short*)a.kp;
  const unsigned short* vpool = (const unsigned short*)a.vp;

  // this lane's rows (columns of S^T): token, head, position
  int tok[QC], head[QC], qpos[QC], sees[QC];
  float sl2[QC];
  bf16x8 qf[QC][NKK];
#pragma unroll
  for (int c = 0; c < QC; ++c) {
    const int r = min(base + (wave * QC + c) * 16 + li, R - 1);
    tok[c] = r / Hg;
    head[c] = g * Hg + r % Hg;
    qpos[c] = qs + tok[c];
    sees[c] = qpos[c] - first_key(a, qpos[c]) + 1;
    sl2[c] = a.slopes ? a.slopes[head[c]] * LOG2E : 0.f;
    const unsigned short* qp = (const unsigned short*)a.q +
        ((long)(t0 + tok[c]) * a.H + head[c]) * DK + hi * 8;
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk)
      qf[c][kk] = as_bf16x8(*reinterpret_cast<const short8*>(qp + kk * 32));
  }
  const float sc2 = a.scale * LOG2E;

  // visible keys of the workgroup and of this wave
  const int last = min(base + 64 * QC, R) - 1;
  const int kend = qs + last / Hg + 1;
  const int kbeg = first_key(a, qs + base / Hg) & ~31;
  const int wr0 = min(base + wave * QC * 16, R - 1);
  const int wr1 = min(base + (wave + 1) * QC * 16, R) - 1;
  const int wlo = first_key(a, qs + wr0 / Hg);   // any row sees >= wlo
  const int whi = qs + max(wr0, wr1) / Hg;              // any row sees <= whi
  const int flo = first_key(a, qs + max(wr0, wr1) / Hg);  // all rows do
  const int fhi = qs + wr0 / Hg;

  float m2[QC], l[QC];
  f32x4 acc[QC][ND];
#pragma unroll
  for (int c = 0; c < QC; ++c) {
    m2[c] = NEG_BIG;
    l[c] = 0.f;
#pragma unroll
    for (int n = 0; n < ND; ++n) acc[c][n] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }

  short8 kreg[KCH], vreg[VCH];
  auto fetch = [&](int kb) {
#pragma unroll
    for (int i = 0; i < KCH; ++i) {
      const int idx = tid + i * 256;
      const int pos = kb + idx / (DK / 8), d8 = (idx % (DK / 8)) * 8;
      kreg[i] = short8{};
      if (pos < kend)
        kreg[i] = *reinterpret_cast<const short8*>(
            kpool + (((long)table[pos / a.P] * a.G + g) * a.P + pos % a.P) * DK + d8);
    }
#pragma unroll
    for (int i = 0; i < VCH; ++i) {
      const int idx = tid + i * 256;
      const int d = idx / (KT / 8), pos = kb + (idx % (KT / 8)) * 8;
      vreg[i] = short8{};
      if (pos < kend)
        vreg[i] = *reinterpret_cast<const short8*>(
            vpool + (((long)table[pos / a.P] * a.G + g) * DV + d) * a.P + pos % a.P);
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int i = 0; i < KCH; ++i) {
      const int idx = tid + i * 256;
      const int key = idx / (DK / 8), c8 = idx % (DK / 8);
      const int k = key & 31;  // LDS row = MFMA n * 16 + row
      const int r = (key & 32) + ((k >> 2) & 1) * 16 + (k >> 3) * 4 + (k & 3);
      *reinterpret_cast<short8*>(k_lds + r * KROW + c8 * 16) = kreg[i];
    }
#pragma unroll
    for (int i = 0; i < VCH; ++i) {
      const int idx = tid + i * 256;
      *reinterpret_cast<short8*>(v_lds + (idx / (KT / 8)) * VROW +
                                 (idx % (KT / 8)) * 16) = vreg[i];
    }
  };

  fetch(kbeg);
  for (int kb = kbeg; kb < kend; kb += KT) {
    __syncthreads();
    stage();
    __syncthreads();
    if (kb + KT < kend) fetch(kb + KT);
    if (kb > whi || kb + KT <= wlo) continue;  // nothing here for this wave
    const bool inside = kb >= flo && kb + KT - 1 <= fhi;

    int d0[QC];
    float b0[QC];
#pragma unroll
    for (int c = 0; c < QC; ++c) {
      d0[c] = qpos[c] - kb - hi * 8;
      b0[c] = sl2[c] * (float)d0[c];
    }
    float p[QC][2][8];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        f32x4 st[QC];
#pragma unroll
        for (int c = 0; c < QC; ++c) st[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < NKK; ++kk) {
          const bf16x8 kf = as_bf16x8(*reinterpret_cast<const short8*>(
              k_lds + (hf * 32 + n * 16 + li) * KROW + hi * 16 + kk * 64));
#pragma unroll
          for (int c = 0; c < QC; ++c)
            st[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[c][kk],
                                                            st[c], 0, 0, 0);
        }
        // bias: -slope * (distance to the lane's first key - key offset)
#pragma unroll
        for (int c = 0; c < QC; ++c)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            p[c][hf][n * 4 + r] = fmaf(
                st[c][r], sc2, fmaf(sl2[c], (float)(hf * 32 + n * 4 + r), -b0[c]));
      }
    if (!inside) {
      // a row that has seen nothing yet piles up weights of one here; its
      // first visible key scales them by exp2(-1e30) = 0
#pragma unroll
      for (int c = 0; c < QC; ++c)
#pragma unroll
        for (int hf = 0; hf < 2; ++hf)
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const int dist = d0[c] - (hf * 32 + j);
            if (dist < 0 || dist >= sees[c]) p[c][hf][j] = NEG_BIG;
          }
    }
#pragma unroll
    for (int c = 0; c < QC; ++c) {
      float rm = NEG_BIG;
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int j = 0; j < 8; ++j) rm = fmaxf(rm, p[c][hf][j]);
      rm = fmaxf(rm, __shfl_xor(rm, 16));
      rm = fmaxf(rm, __shfl_xor(rm, 32));
      const float mn = fmaxf(m2[c], rm);
      const float corr = fast_exp2(m2[c] - mn);
      float ps = 0.f;
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          p[c][hf][j] = fast_exp2(p[c][hf][j] - mn);
          ps += p[c][hf][j];
        }
      ps += __shfl_xor(ps, 16);
      ps += __shfl_xor(ps, 32);
      l[c] = l[c] * corr + ps;
      m2[c] = mn;
      if (__builtin_amdgcn_ballot_w64(corr != 1.f)) {
#pragma unroll
        for (int n = 0; n < ND; ++n)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[c][n][r] *= corr;
      }
    }
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      bf16x8 ph[QC], pl[QC];
#pragma unroll
      for (int c = 0; c < QC; ++c) split_bf16(p[c][hf], ph[c], pl[c]);
#pragma unroll
      for (int n = 0; n < ND; ++n) {
        const bf16x8 vf = as_bf16x8(*reinterpret_cast<const short8*>(
            v_lds + (n * 16 + li) * VROW + hf * 64 + hi * 16));
#pragma unroll
        for (int c = 0; c < QC; ++c) {
          acc[c][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[c],
                                                              acc[c][n], 0, 0, 0);
          acc[c][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[c],
                                                              acc[c][n], 0, 0, 0);
        }
      }
    }
  }

#pragma unroll
  for (int c = 0; c < QC; ++c) {
    if (base + (wave * QC + c) * 16 + li >= R) continue;
    const float sc = a.sinks ? add_sink(a.sinks[head[c]] * LOG2E, m2[c], l[c]) : 1.f;
    const float inv = l[c] > 0.f ? sc / l[c] : 0.f;
#pragma unroll
    for (int n = 0; n < ND; ++n) {
      float o[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = acc[c][n][r] * inv;
      if (n * 16 + hi * 4 < a.vdim)
        store_out4(a, t0 + tok[c], head[c], n * 16 + hi * 4, o);
    }
  }
}

// ---------------------------------------------------------------------------
// decode: grid (sequences * G * chunks of 16 heads, n_split)
// ---------------------------------------------------------------------------

template <int DK, int DV>
__global__ __launch_bounds__(256, DK + DV > 256 ? 1 : 2) void attn_ragged_decode_kernel(AttnArgs a) {
  constexpr int NKK = DK / 32, ND = DV / 16;
  constexpr int MROW = DV + 4;  // f32 per column of the merge buffer
  __shared__ __attribute__((aligned(16))) float merge[3][16 * MROW];

  const int Hg = a.H / a.G;
  const int nch = (Hg + 15) / 16;
  const int unit = blockIdx.x;
  const int s = a.list[unit / (a.G * nch)];
  const int g = (unit / nch) % a.G;
  const int h0 = (unit % nch) * 16;
  const int Hl = min(16, Hg - h0);
  const int row = a.cu[s];
  const int pos = a.tok_pos[row];
  const int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int* table = a.table + (long)s * a.maxp;
  const unsigned short* kpool = (const unsigned short*)a.kp;
  const unsigned short* vpool = (const unsigned short*)a.vp;

  const int h = g * Hg + h0 + min(li, Hl - 1);
  const float sl2 = a.slopes ? a.slopes[h] * LOG2E : 0.f;
  const float sc2 = a.scale * LOG2E;
  bf16x8 qf[NKK];
  const unsigned short* qp =
      (const unsigned short*)a.q + ((long)row * a.H + h) * DK + hi * 8;
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk)
    qf[kk] = as_bf16x8(*reinterpret_cast<const short8*>(qp + kk * 32));

  // tiles of the visible range, this split's share, this wave's every fourth
  const int lo = first_key(a, pos);
  const int t_beg = lo / 32;
  const int t_all = pos < 0 ? 0 : pos / 32 + 1 - t_beg;
  const int per = (t_all + a.n_split - 1) / a.n_split;
  const int t_lo = t_beg + blockIdx.y * per;
  const int t_hi = min(t_beg + t_all, t_lo + per);

  float m2 = NEG_BIG, l = 0.f;
  f32x4 acc[ND];
#pragma unroll
  for (int n = 0; n < ND; ++n) acc[n] = (f32x4){0.f, 0.f, 0.f, 0.f};

  bf16x8 k0[2][NKK], v0[ND];
  auto load = [&](bf16x8 (&kf)[2][NKK], bf16x8 (&vf)[ND], int tile) {
    const int vpos = tile * 32 + hi * 8;
    const bool live = vpos <= pos;
    const long vrow = live ? ((long)table[vpos / a.P] * a.G + g) * DV : 0;
#pragma unroll
    for (int n = 0; n < ND; ++n) {
      vf[n] = as_bf16x8(short8{});
      if (live)
        vf[n] = as_bf16x8(__builtin_nontemporal_load(
            reinterpret_cast<const short8*>(
                vpool + (vrow + n * 16 + li) * a.P + vpos % a.P)));
    }
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int key = min(tile * 32 + (li >> 2) * 8 + n * 4 + (li & 3), pos);
      const unsigned short* kr = kpool +
          (((long)table[key / a.P] * a.G + g) * a.P + key % a.P) * DK + hi * 8;
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk)
        kf[n][kk] = as_bf16x8(__builtin_nontemporal_load(
            reinterpret_cast<const short8*>(kr + kk * 32)));
    }
  };
  auto compute = [&](const bf16x8 (&kf)[2][NKK], const bf16x8 (&vf)[ND],
                     int tile) {
    float p[8];
    float rm = NEG_BIG;
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      f32x4 st = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk)
        st = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[n][kk], qf[kk], st,
                                                     0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int key = tile * 32 + hi * 8 + n * 4 + r;
        const float v = st[r] * sc2 - sl2 * (float)(pos - key);
        p[n * 4 + r] = (key < lo || key > pos) ? NEG_BIG : v;
        rm = fmaxf(rm, p[n * 4 + r]);
      }
    }
    rm = fmaxf(rm, __shfl_xor(rm, 16));
    rm = fmaxf(rm, __shfl_xor(rm, 32));
    const float mn = fmaxf(m2, rm);
    const float corr = fast_exp2(m2 - mn);
    float ps = 0.f;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      p[j] = fast_exp2(p[j] - mn);  // every tile has a visible key
      ps += p[j];
    }
    ps += __shfl_xor(ps, 16);
    ps += __shfl_xor(ps, 32);
    l = l * corr + ps;
    m2 = mn;
    if (__builtin_amdgcn_ballot_w64(corr != 1.f)) {
#pragma unroll
      for (int n = 0; n < ND; ++n)
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[n][r] *= corr;
    }
    bf16x8 ph, pl;
    split_bf16(p, ph, pl);
#pragma unroll
    for (int n = 0; n < ND; ++n) {
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[n], ph, acc[n], 0, 0, 0);
      acc[n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[n], pl, acc[n], 0, 0, 0);
    }
  };

  int t = t_lo + wave;
  if constexpr (DK + DV > 256) {   // no registers for a second buffer
    for (; t < t_hi; t += 4) {
      load(k0, v0, t);
      compute(k0, v0, t);
    }
  } else {
    // two named buffers: the next tile's loads fly behind this one's compute
    bf16x8 k1[2][NKK], v1[ND];
    if (t < t_hi) load(k0, v0, t);
    for (; t < t_hi; t += 8) {
      if (t + 4 < t_hi) load(k1, v1, t + 4);
      __builtin_amdgcn_sched_barrier(0);
      compute(k0, v0, t);
      if (t + 4 >= t_hi) break;
      if (t + 8 < t_hi) load(k0, v0, t + 8);
      __builtin_amdgcn_sched_barrier(0);
      compute(k1, v1, t + 4);
    }
  }

  // fold waves 1..3 into wave 0
  if (wave > 0) {
    float* mr = merge[wave - 1] + li * MROW;
    if (hi == 0) {
      mr[0] = m2;
      mr[1] = l;
    }
#pragma unroll
    for (int n = 0; n < ND; ++n)
      *reinterpret_cast<f32x4*>(mr + 4 + n * 16 + hi * 4) = acc[n];
  }
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int w = 0; w < 3; ++w) {
    const float* mr = merge[w] + li * MROW;
    const float om = mr[0], ol = mr[1];
    const float mn = fmaxf(m2, om);
    const float c0 = fast_exp2(m2 - mn), c1 = fast_exp2(om - mn);
    l = l * c0 + ol * c1;
    m2 = mn;
#pragma unroll
    for (int n = 0; n < ND; ++n) {
      const f32x4 oa = *reinterpret_cast<const f32x4*>(mr + 4 + n * 16 + hi * 4);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[n][r] = acc[n][r] * c0 + oa[r] * c1;
    }
  }
  if (li >= Hl) return;
  if (a.n_split > 1) {
    const long u = (long)unit * a.n_split + blockIdx.y;
    if (hi == 0) {
      a.pml[(u * 16 + li) * 2] = m2;
      a.pml[(u * 16 + li) * 2 + 1] = l;
    }
#pragma unroll
    for (int n = 0; n < ND; ++n)
      *reinterpret_cast<f32x4*>(a.pacc + (u * 16 + li) * DV + n * 16 + hi * 4) =
          acc[n];
    return;
  }
  const float sc = a.sinks ? add_sink(a.sinks[h] * LOG2E, m2, l) : 1.f;
  const float inv = l > 0.f ? sc / l : 0.f;
#pragma unroll
  for (int n = 0; n < ND; ++n) {
    float o[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = acc[n][r] * inv;
    if (n * 16 + hi * 4 < a.vdim) store_out4(a, row, h, n * 16 + hi * 4, o);
  }
}

// Fold the splits of one unit; grid = units, one column of 16 per 16 threads.
__global__ __launch_bounds__(256) void attn_ragged_combine_kernel(AttnArgs a) {
  const int Hg = a.H / a.G;
  const int nch = (Hg + 15) / 16;
  const int unit = blockIdx.x;
  const int g = (unit / nch) % a.G;
  const int h0 = (unit % nch) * 16;
  const int col = threadIdx.x / 16;
  if (h0 + col >= Hg) return;
  const int row = a.cu[a.list[unit / (a.G * nch)]];
  const long u0 = (long)unit * a.n_split;
  float m = NEG_BIG;
  for (int i = 0; i < a.n_split; ++i)
    m = fmaxf(m, a.pml[((u0 + i) * 16 + col) * 2]);
  float l = 0.f;
  for (int i = 0; i < a.n_split; ++i)
    l += a.pml[((u0 + i) * 16 + col) * 2 + 1] *
         fast_exp2(a.pml[((u0 + i) * 16 + col) * 2] - m);
  const float sc =
      a.sinks ? add_sink(a.sinks[g * Hg + h0 + col] * LOG2E, m, l) : 1.f;
  const float inv = l > 0.f ? sc / l : 0.f;
  for (int d = (threadIdx.x % 16) * 4; d < a.vdim; d += 64) {
    float o[4] = {0.f, 0.f, 0.f, 0.f};
    for (int i = 0; i < a.n_split; ++i) {
      const float c = fast_exp2(a.pml[((u0 + i) * 16 + col) * 2] - m);
      const f32x4 v = *reinterpret_cast<const f32x4*>(
          a.pacc + ((u0 + i) * 16 + col) * a.dvp + d);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] += v[r] * c;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] *= inv;
    store_out4(a, row, g * Hg + h0 + col, d, o);
  }
}

// ---------------------------------------------------------------------------
// plain: grid (N, H), one wave
// ---------------------------------------------------------------------------

static constexpr int SIMPLE_MAXD = 1024;

template <typename T, typename TO>
__global__ __launch_bounds__(64) void attn_ragged_simple_kernel(AttnArgs a) {
  __shared__ float q_lds[SIMPLE_MAXD];
  __shared__ float p_lds[64];
  __shared__ long v_lds[64];
  const int row = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int g = h / (a.H / a.G);
  const int pos = a.tok_pos[row];
  const int* table = a.table + (long)a.tok_seq[row] * a.maxp;
  const T* kpool = (const T*)a.kp;
  const T* vpool = a.vp ? (const T*)a.vp : kpool;
  const long vstep = a.vp ? a.P : 1;  // between a value's elements
  const long ldk = (long)a.maps * a.dkp, map0 = h % a.maps * a.dkp;
  for (int d = lane; d < a.dim; d += 64)
    q_lds[d] = ldf((const T*)a.q + ((long)row * a.H + h) * a.dkp + d);
  __syncthreads();
  const float slope = a.slopes ? a.slopes[h] : 0.f;
  float m = NEG_BIG, l = 0.f;
  float acc[SIMPLE_MAXD / 64];
#pragma unroll
  for (int i = 0; i < SIMPLE_MAXD / 64; ++i) acc[i] = 0.f;
  for (int kb = first_key(a, pos); kb <= pos; kb += 64) {
    const int key = kb + lane;
    float sc = NEG_BIG;
    if (key <= pos) {
      const long pg = (long)table[key / a.P] * a.G + g;
      const T* kr = kpool + (pg * a.P + key % a.P) * ldk + map0;
      float dot = 0.f;
      for (int d = 0; d < a.dim; ++d) dot += q_lds[d] * ldf(kr + d);
      sc = dot * a.scale - slope * (float)(pos - key);
      v_lds[lane] = a.vp ? pg * a.dvp * a.P + key % a.P
                         : (pg * a.P + key % a.P) * ldk;
    }
    const float mn = fmaxf(m, wave_reduce_max(sc));
    const float corr = expf(m - mn);
    const float p = key <= pos ? expf(sc - mn) : 0.f;
    p_lds[lane] = p;
    l = l * corr + wave_reduce_sum(p);
    m = mn;
    __syncthreads();
    const int n = min(64, pos - kb + 1);
#pragma unroll
    for (int i = 0; i < SIMPLE_MAXD / 64; ++i) {
      const int d = lane + i * 64;
      if (d >= a.vdim) break;
      float s = 0.f;
      for (int j = 0; j < n; ++j) s += p_lds[j] * ldf(vpool + v_lds[j] + d * vstep);
      acc[i] = acc[i] * corr + s;
    }
    __syncthreads();
  }
  float sc = 1.f;
  if (a.sinks) {
    const float mn = fmaxf(m, a.sinks[h]);
    sc = expf(m - mn);
    l = l * sc + expf(a.sinks[h] - mn);
  }
  const float inv = l > 0.f ? sc / l : 0.f;
#pragma unroll
  for (int i = 0; i < SIMPLE_MAXD / 64; ++i) {
    const int d = lane + i * 64;
    if (d >= a.vdim) break;
    float o = acc[i] * inv;
    if (a.gate)
      o *= sigmoid_f(ldf((const T*)a.gate + row * a.ldg + h * a.vdim + d));
    stf((TO*)a.out + row * a.ldo + h * a.vdim + d, o);
  }
}
