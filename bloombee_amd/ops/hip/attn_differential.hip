// Differential attention over ragged batches: every head has two queries (maps),
// every key/value head two keys and one value. With a1 and a2 the attentions of
// the two maps over the same values,
//     o = (a1 - lam a2) / sqrt(mean((a1 - lam a2)^2) + eps) * factor
// per head. A key's maps lie side by side in its page slot, so a K/V tile is read
// once for both.
//
//  attn_diff_prefill_kernel  rows of a tile are (token, head of the group) pairs;
//                            a wave keeps the softmax of both maps for its rows,
//                            so they combine in its registers.
//  attn_diff_decode_kernel   columns are (map, head of the group), eight heads a
//                            unit; the queries are zero where the other map's
//                            key lies.
//  attn_diff_combine_kernel  folds the splits of a unit, then the maps.
//  attn_diff_join_kernel     combines maps that the plain kernel made apart.
//
// Order of keys, weights as two bf16, visible ranges: as in attn_ragged.hip.

#pragma once
#include "common.h"
#include "rows.hip"
#include "attn_ragged.hip"

struct DiffArgs : AttnArgs {
  float lam, factor, eps;
  int p_log2;           // of the page size
};

// Four consecutive output columns of one row.
DEVINL void store_diff4(const DiffArgs& a, long row, int h, int d, const float* o) {
  unsigned short* op = (unsigned short*)a.out + row * a.ldo + h * a.vdim + d;
  if (((a.vdim | (int)a.ldo) & 3) == 0 && d + 4 <= a.vdim) {
    stv<4>(op, o);
    return;
  }
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (d + j < a.vdim) op[j] = cvt_bf(o[j]);
}

// ---------------------------------------------------------------------------
// prefill: grid (row tiles of the longest portion, G, sequences)
// ---------------------------------------------------------------------------

// A K/V tile of 64 keys in LDS, filled by loads that bypass the registers: 16 B
// pieces, piece c of row r at c ^ swizzle(r), so that eight rows read at one piece
// lie in different banks.
template <int DK, int DV>
struct DiffTile {
  static constexpr int KT = 64, RC = DK / 4;      // pieces of a key row, two maps
  static constexpr int KB = KT * RC * 16;         // bytes
  static constexpr int VB = DV * KT * 2;
  static constexpr int BYTES = KB + VB;
  static constexpr int KSW = RC >= 16 ? 15 : 7;
};

// NW waves of 16 rows; tiles are double-buffered.
template <int DK, int DV, int NW>  // DK: one map
__global__ __launch_bounds__(NW * 64, NW / 4) void attn_diff_prefill_kernel(
    DiffArgs a) {
  using Tile = DiffTile<DK, DV>;
  constexpr int KT = Tile::KT, RC = Tile::RC, KB = Tile::KB;
  constexpr int NKK = DK / 32, ND = DV / 16;
  constexpr int KI = KB / 1024, VI = Tile::VB / 1024;  // loads of a wave's width
  constexpr int KN = (KI + NW - 1) / NW, VN = (VI + NW - 1) / NW;
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_tiles[];

  const int s = a.list[blockIdx.z];
  const int g = blockIdx.y;
  const int Hg = a.H / a.G;
  const int t0 = a.cu[s], T = a.cu[s + 1] - t0, qs = a.q_start[s];
  const int R = T * Hg;
  // late rows see the most keys: they go first
  const int base = (int)(gridDim.x - 1 - blockIdx.x) * (16 * NW);
  if (base >= R) return;
  const int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int* table = a.table + (long)s * a.maxp;
  const unsigned short* kpool = (const unsigned short*)a.kp;
  const unsigned short* vpool = (const unsigned short*)a.vp;
  const int plog = a.p_log2, pmask = (1 << plog) - 1;

  // this lane's row (column of S^T): token, head, position
  const int r = min(base + wave * 16 + li, R - 1);
  const int tok = r / Hg, head = g * Hg + r % Hg, qpos = qs + tok;
  const int sees = qpos - first_key(a, qpos) + 1;
  bf16x8 qf[2][NKK];
  const unsigned short* qp = (const unsigned short*)a.q +
                             ((long)(t0 + tok) * a.H + head) * (2 * DK) + hi * 8;
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int kk = 0; kk < NKK; ++kk)
      qf[m][kk] =
          as_bf16x8(*reinterpret_cast<const short8*>(qp + m * DK + kk * 32));
  const float sc2 = a.scale * LOG2E;

  // visible keys of the workgroup and of this wave
  const int last = min(base + 16 * NW, R) - 1;
  const int kend = qs + last / Hg + 1;
  const int kbeg = first_key(a, qs + base / Hg) & ~31;
  const int wr0 = min(base + wave * 16, R - 1);
  const int wr1 = max(wr0, min(base + (wave + 1) * 16, R) - 1);
  const int wlo = first_key(a, qs + wr0 / Hg);   // any row sees >= wlo
  const int whi = qs + wr1 / Hg;                 // any row sees <= whi
  const int flo = first_key(a, qs + wr1 / Hg);   // all rows do
  const int fhi = qs + wr0 / Hg;

  // where this lane's pieces come from: LDS row r of the keys is MFMA row order,
  // n * 16 + x * 4 + y  <->  key x * 8 + n * 4 + y  (of 32)
  int kkey[KN], kcol[KN], vblk[VN], vrow[VN];
#pragma unroll
  for (int i = 0; i < KN; ++i) {
    const int at = min(wave + i * NW, KI - 1) * 64 + lane;
    const int row = at / RC, q = row & 31;
    kcol[i] = ((at % RC) ^ (row & Tile::KSW)) * 8;
    kkey[i] = (row & 32) + ((q >> 2) & 3) * 8 + (q >> 4) * 4 + (q & 3);
  }
#pragma unroll
  for (int i = 0; i < VN; ++i) {
    const int at = min(wave + i * NW, VI - 1) * 64 + lane;
    vrow[i] = at / 8;
    vblk[i] = (at % 8) ^ (vrow[i] & 7);
  }
  // lanes 0..7: the pages of a tile's eight blocks of eight keys
  auto pages_of = [&](int kb) {
    return table[min(kb + (lane & 7) * 8, kend - 1) >> plog];
  };
  auto issue = [&](int kb, int pages, unsigned char* buf) {
#pragma unroll
    for (int i = 0; i < KN; ++i) {
      if (KI % NW && wave + i * NW >= KI) break;
      const int pos = min(kb + kkey[i], kend - 1);
      const long page = __shfl(pages, kkey[i] >> 3);
      copy16_to_lds(kpool + (((page * a.G + g) << plog) + (pos & pmask)) * (2 * DK) +
                        kcol[i],
                    buf + (wave + i * NW) * 1024);
    }
#pragma unroll
    for (int i = 0; i < VN; ++i) {
      if (VI % NW && wave + i * NW >= VI) break;
      const int pos = min(kb + vblk[i] * 8, (kend - 1) & ~7);
      const long page = __shfl(pages, vblk[i]);
      copy16_to_lds(vpool + (((page * a.G + g) * DV + vrow[i]) << plog) +
                        (pos & pmask),
                    buf + KB + (wave + i * NW) * 1024);
    }
  };

  float m2[2], l[2];
  f32x4 acc[2][ND];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    m2[m] = NEG_BIG;
    l[m] = 0.f;
#pragma unroll
    for (int n = 0; n < ND; ++n) acc[m][n] = (f32x4){0.f, 0.f, 0.f, 0.f};
  }

  auto compute = [&](int kb, const unsigned char* kt) {
    const unsigned char* vt = kt + KB;
    const bool inside = kb >= flo && kb + KT - 1 <= fhi;
    const int d0 = qpos - kb - hi * 8;
    float p[2][2][8];
#pragma unroll
    for (int hf = 0; hf < 2; ++hf)
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        f32x4 st[2];
        st[0] = st[1] = (f32x4){0.f, 0.f, 0.f, 0.f};
        const unsigned char* row = kt + (hf * 32 + n * 16 + li) * RC * 16;
#pragma unroll
        for (int kk = 0; kk < NKK; ++kk)
#pragma unroll
          for (int m = 0; m < 2; ++m) {
            const int c = m * (DK / 8) + kk * 4 + hi;
            const bf16x8 kf = as_bf16x8(*reinterpret_cast<const short8*>(
                row + (c ^ (li & Tile::KSW)) * 16));
            st[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[m][kk], st[m],
                                                            0, 0, 0);
          }
#pragma unroll
        for (int m = 0; m < 2; ++m)
#pragma unroll
          for (int q = 0; q < 4; ++q) p[m][hf][n * 4 + q] = st[m][q] * sc2;
      }
    if (!inside) {
      // a row that has seen nothing yet piles up weights of one here; its
      // first visible key scales them by exp2(-1e30) = 0
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const int dist = d0 - (hf * 32 + j);
          if (dist < 0 || dist >= sees) p[0][hf][j] = p[1][hf][j] = NEG_BIG;
        }
    }
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float rm = NEG_BIG;
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int j = 0; j < 8; ++j) rm = fmaxf(rm, p[m][hf][j]);
      rm = fmaxf(rm, __shfl_xor(rm, 16));
      rm = fmaxf(rm, __shfl_xor(rm, 32));
      const float mn = fmaxf(m2[m], rm);
      const float corr = fast_exp2(m2[m] - mn);
      float ps = 0.f;
#pragma unroll
      for (int hf = 0; hf < 2; ++hf)
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          p[m][hf][j] = fast_exp2(p[m][hf][j] - mn);
          ps += p[m][hf][j];
        }
      ps += __shfl_xor(ps, 16);
      ps += __shfl_xor(ps, 32);
      l[m] = l[m] * corr + ps;
      m2[m] = mn;
      if (__builtin_amdgcn_ballot_w64(corr != 1.f)) {
#pragma unroll
        for (int n = 0; n < ND; ++n)
#pragma unroll
          for (int q = 0; q < 4; ++q) acc[m][n][q] *= corr;
      }
    }
#pragma unroll
    for (int hf = 0; hf < 2; ++hf) {
      bf16x8 ph[2], pl[2];
#pragma unroll
      for (int m = 0; m < 2; ++m) split_bf16(p[m][hf], ph[m], pl[m]);
#pragma unroll
      for (int n = 0; n < ND; ++n) {
        const bf16x8 vf = as_bf16x8(*reinterpret_cast<const short8*>(
            vt + (n * 16 + li) * 128 + ((hf * 4 + hi) ^ (li & 7)) * 16));
#pragma unroll
        for (int m = 0; m < 2; ++m)
          acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[m],
                                                              acc[m][n], 0, 0, 0);
#pragma unroll
        for (int m = 0; m < 2; ++m)
          acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[m],
                                                              acc[m][n], 0, 0, 0);
      }
    }
  };

  // page numbers are looked up a tile ahead of the loads that need them
  int pages = pages_of(kbeg);
  issue(kbeg, pages, lds_tiles);
  pages = pages_of(kbeg + KT);
  __syncthreads();
  int buf = 0;
  for (int kb = kbeg; kb < kend; kb += KT) {
    if (kb + KT < kend) {
      issue(kb + KT, pages, lds_tiles + (buf ^ 1) * Tile::BYTES);
      pages = pages_of(kb + 2 * KT);
    }
    if (kb <= whi && kb + KT > wlo) compute(kb, lds_tiles + buf * Tile::BYTES);
    __syncthreads();
    buf ^= 1;
  }

  // a row's values are spread over the four lanes of its column; those beyond
  // vdim are zero
  const float i0 = l[0] > 0.f ? 1.f / l[0] : 0.f;
  const float i1 = l[1] > 0.f ? a.lam / l[1] : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const float o = acc[0][n][q] * i0 - acc[1][n][q] * i1;
      acc[0][n][q] = n * 16 + hi * 4 + q < a.vdim ? o : 0.f;
      ss += acc[0][n][q] * acc[0][n][q];
    }
  ss += __shfl_xor(ss, 16);
  ss += __shfl_xor(ss, 32);
  if (base + wave * 16 + li >= R) return;
  const float f = a.factor / sqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
  for (int n = 0; n < ND; ++n) {
    float o[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) o[q] = acc[0][n][q] * f;
    if (n * 16 + hi * 4 < a.vdim)
      store_diff4(a, t0 + tok, head, n * 16 + hi * 4, o);
  }
}

// ---------------------------------------------------------------------------
// decode: grid (sequences * G * chunks of 8 heads, n_split)
// ---------------------------------------------------------------------------

template <int DK, int DV>  // DK: both maps
__global__ __launch_bounds__(256, DK + DV > 256 ? 1 : 2) void attn_diff_decode_kernel(
    DiffArgs a) {
  constexpr int NKK = DK / 32, ND = DV / 16;
  constexpr int MROW = DV + 4;  // f32 per column of the merge buffer
  __shared__ __attribute__((aligned(16))) float merge[3][16 * MROW];

  const int Hg = a.H / a.G;
  const int nch = (Hg + 7) / 8;
  const int unit = blockIdx.x;
  const int s = a.list[unit / (a.G * nch)];
  const int g = (unit / nch) % a.G;
  const int h0 = (unit % nch) * 8;
  const int Hl = min(8, Hg - h0);
  const int row = a.cu[s];
  const int pos = a.tok_pos[row];
  const int tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid / WAVE);
  const int lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int* table = a.table + (long)s * a.maxp;
  const unsigned short* kpool = (const unsigned short*)a.kp;
  const unsigned short* vpool = (const unsigned short*)a.vp;

  const int map = li >> 3;
  const int h = g * Hg + h0 + min(li & 7, Hl - 1);
  const float sc2 = a.scale * LOG2E;
  bf16x8 qf[NKK];
  const unsigned short* qp =
      (const unsigned short*)a.q + ((long)row * a.H + h) * DK + hi * 8;
#pragma unroll
  for (int kk = 0; kk < NKK; ++kk) {
    const short8 v = *reinterpret_cast<const short8*>(qp + kk * 32);
    qf[kk] = as_bf16x8(kk / (NKK / 2) == map ? v : short8{});
  }

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

  // page numbers of a tile: this lane's block of eight keys, then of values
  const int plog = a.p_log2, pmask = (1 << plog) - 1;
  auto pages_of = [&](int tile, int (&pg)[2]) {
    pg[0] = table[min(tile * 32 + (li >> 2) * 8, max(pos, 0)) >> plog];
    pg[1] = table[min(tile * 32 + hi * 8, max(pos, 0)) >> plog];
  };
  auto load = [&](bf16x8 (&kf)[2][NKK], bf16x8 (&vf)[ND], int tile,
                  const int (&pg)[2]) {
    const unsigned short* kr = kpool + (((long)pg[0] * a.G + g) << plog) * DK + hi * 8;
#pragma unroll
    for (int n = 0; n < 2; ++n) {
      const int key = min(tile * 32 + (li >> 2) * 8 + n * 4 + (li & 3), pos);
#pragma unroll
      for (int kk = 0; kk < NKK; ++kk)
        kf[n][kk] = as_bf16x8(__builtin_nontemporal_load(
            reinterpret_cast<const short8*>(kr + (key & pmask) * DK + kk * 32)));
    }
    // values beyond the last key weigh nothing
    const int vpos = min(tile * 32 + hi * 8, pos & ~7);
    const unsigned short* vr = vpool +
        ((((long)pg[1] * a.G + g) * DV + li) << plog) + (vpos & pmask);
#pragma unroll
    for (int n = 0; n < ND; ++n)
      vf[n] = as_bf16x8(__builtin_nontemporal_load(
          reinterpret_cast<const short8*>(vr + ((long)n << (plog + 4)))));
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
        p[n * 4 + r] = (key < lo || key > pos) ? NEG_BIG : st[r] * sc2;
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

  // two named buffers: the next tile's loads fly behind this one's compute, and
  // page numbers are looked up a tile ahead of them
  bf16x8 k0[2][NKK], v0[ND], k1[2][NKK], v1[ND];
  int pg[2];
  int t = t_lo + wave;
  pages_of(t, pg);
  if (t < t_hi) load(k0, v0, t, pg);
  pages_of(t + 4, pg);
  for (; t < t_hi; t += 8) {
    if (t + 4 < t_hi) load(k1, v1, t + 4, pg);
    pages_of(t + 8, pg);
    __builtin_amdgcn_sched_barrier(0);
    compute(k0, v0, t);
    if (t + 4 >= t_hi) break;
    if (t + 8 < t_hi) load(k0, v0, t + 8, pg);
    pages_of(t + 12, pg);
    __builtin_amdgcn_sched_barrier(0);
    compute(k1, v1, t + 4);
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
  if (a.n_split > 1) {
    const long u = ((long)unit * a.n_split + blockIdx.y) * 16 + li;
    if (hi == 0) {
      a.pml[u * 2] = m2;
      a.pml[u * 2 + 1] = l;
    }
#pragma unroll
    for (int n = 0; n < ND; ++n)
      *reinterpret_cast<f32x4*>(a.pacc + u * DV + n * 16 + hi * 4) = acc[n];
    return;
  }
  // the other map of the head is eight columns on
  const float inv = l > 0.f ? 1.f / l : 0.f;
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < ND; ++n)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float v = acc[n][r] * inv;
      const float o = v - a.lam * __shfl_xor(v, 8);
      acc[n][r] = n * 16 + hi * 4 + r < a.vdim ? o : 0.f;
      ss += acc[n][r] * acc[n][r];
    }
  ss += __shfl_xor(ss, 16);
  ss += __shfl_xor(ss, 32);
  if (li >= Hl) return;
  const float f = a.factor / sqrtf(ss / (float)a.vdim + a.eps);
#pragma unroll
  for (int n = 0; n < ND; ++n) {
    float o[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] = acc[n][r] * f;
    if (n * 16 + hi * 4 < a.vdim) store_diff4(a, row, h, n * 16 + hi * 4, o);
  }
}

// grid = units; 32 threads a head, of which each looks after one split at first
__global__ __launch_bounds__(256) void attn_diff_combine_kernel(DiffArgs a) {
  constexpr int NP = 2;  // pieces of four columns a thread, dvp <= 256
  const int Hg = a.H / a.G;
  const int nch = (Hg + 7) / 8;
  const int unit = blockIdx.x;
  const int h0 = (unit % nch) * 8;
  const int col = threadIdx.x / 32, part = threadIdx.x % 32, d0 = part * 4;
  if (h0 + col >= Hg) return;   // whole groups of 32 lanes
  const int row = a.cu[a.list[unit / (a.G * nch)]];
  const long u0 = (long)unit * a.n_split * 16 + col;
  float w[2];   // weight of this thread's split
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    const long u = u0 + m * 8 + min(part, a.n_split - 1) * 16;
    const float mi = part < a.n_split ? a.pml[u * 2] : NEG_BIG;
    float mx = mi;
#pragma unroll
    for (int k = 1; k < 32; k <<= 1) mx = fmaxf(mx, __shfl_xor(mx, k));
    w[m] = part < a.n_split ? fast_exp2(mi - mx) : 0.f;
    float l = part < a.n_split ? a.pml[u * 2 + 1] * w[m] : 0.f;
#pragma unroll
    for (int k = 1; k < 32; k <<= 1) l += __shfl_xor(l, k);
    w[m] = l > 0.f ? w[m] / l : 0.f;
  }
  float o[2][NP][4];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int p = 0; p < NP; ++p)
#pragma unroll
      for (int r = 0; r < 4; ++r) o[m][p][r] = 0.f;
#pragma unroll 4
  for (int i = 0; i < a.n_split; ++i)
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const float c = __shfl(w[m], i, 32);
#pragma unroll
      for (int p = 0; p < NP; ++p) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(
            a.pacc + (u0 + m * 8 + i * 16) * a.dvp + min(d0 + p * 128, a.dvp - 4));
#pragma unroll
        for (int r = 0; r < 4; ++r) o[m][p][r] += v[r] * c;
      }
    }
  float ss = 0.f;
#pragma unroll
  for (int p = 0; p < NP; ++p)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float v = o[0][p][r] - a.lam * o[1][p][r];
      o[0][p][r] = d0 + p * 128 + r < a.vdim ? v : 0.f;
      ss += o[0][p][r] * o[0][p][r];
    }
#pragma unroll
  for (int m = 1; m < 32; m <<= 1) ss += __shfl_xor(ss, m);
  const float f = a.factor / sqrtf(ss / (float)a.vdim + a.eps);
  const int h = (unit / nch) % a.G * Hg + h0 + col;
#pragma unroll
  for (int p = 0; p < NP; ++p) {
    const int d = d0 + p * 128;
    if (d >= a.vdim) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[0][p][r] *= f;
    store_diff4(a, row, h, d, o[0][p]);
  }
}

// grid (N, H), one wave: y (N, H, 2, vdim) f32 -> out
template <typename T>
__global__ __launch_bounds__(64) void attn_diff_join_kernel(
    const float* __restrict__ y, T* __restrict__ out, long ldo, int H, int vdim,
    float lam, float factor, float eps) {
  const long row = blockIdx.x;
  const int h = blockIdx.y;
  const float* a1 = y + (row * H + h) * 2 * vdim;
  float ss = 0.f;
  for (int d = threadIdx.x; d < vdim; d += WAVE) {
    const float v = a1[d] - lam * a1[vdim + d];
    ss += v * v;
  }
  const float f = factor / sqrtf(wave_reduce_sum(ss) / (float)vdim + eps);
  for (int d = threadIdx.x; d < vdim; d += WAVE)
    stf(out + row * ldo + h * vdim + d, (a1[d] - lam * a1[vdim + d]) * f);
}
