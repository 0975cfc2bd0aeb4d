// Routed experts over (token, choice) slots: slot = token * top + choice.
//
//   act[.]  = glu(W_gate[e] h, W_up[e] h)              one fused launch
//   y[slot] = wts[slot] * (W_down[e] act)              one launch
//
// with glu(g, u) = g sigmoid(slope g) (u + shift) after g = min(g, limit) and
// u = clamp(u, -limit, limit): silu(g) * u for an infinite limit, slope 1 and
// shift 0; or act = relu(W_up[e] h)^2, and the weight may multiply h instead: by then
// it has passed through the linear map, so the first launch's epilogue applies
// it ahead of the activation.
//
// ids[slot] < 0 marks a choice without weights (an identity expert, which the
// residual fold adds by itself): it is skipped everywhere.
//
// First weights (E, planes, F, K): of two planes, row f of plane 0 is the gate of
// activation f, of plane 1 its up projection; a single plane is the up projection
// of relu^2. down (E, N, F). K, F and N are padded to 64.
//
// Kernels take UP, the planes of the first product, 0 for the second, and wts,
// the weights to apply or null.
//
//  * moe_skinny_kernel — up to 32 tokens: streams each chosen expert's weights
//    once; a workgroup finds its expert's slots by scanning the ids itself, so
//    a decode step needs no sort.
//  * moe_sort_kernel + moe_tile_kernel — longer batches: expert-sorted slots,
//    MFMA tiles of 64 or 128 rows staged through LDS.
//  * moe_simple_kernel — f32 arithmetic on f32 data.

#pragma once
#include "common.h"
#include "rows.hip"

static constexpr int MOE_MAX_E = 1024;

struct GluConst {
  float limit, slope, shift;
};

DEVINL float gated(const GluConst& c, float g, float u) {
  g = fminf(g, c.limit);
  u = fminf(fmaxf(u, -c.limit), c.limit) + c.shift;
  return g * sigmoid_f(c.slope * g) * u;
}

// XCD-aware order: consecutive tiles, which share operand rows, on one XCD.
DEVINL int xcd_order(int id, int n) {
  const int q = n / 8, r = n % 8, x = id % 8, o = id / 8;
  return (x < r ? x * (q + 1) : r * (q + 1) + (x - r) * q) + o;
}

// ---------------------------------------------------------------------------
// sort: one workgroup of 1024
// ---------------------------------------------------------------------------

// off (E+1), sorted (S) slots, tiles (max_tiles + 1, 2): expert (-1 = unused)
// and first sorted position of every BM-row tile; then the number of tiles.
__global__ __launch_bounds__(1024) void moe_sort_kernel(
    const int* __restrict__ ids, int* __restrict__ off,
    int* __restrict__ sorted, int* __restrict__ tiles, int S, int E, int BM,
    int max_tiles) {
  __shared__ int cnt[MOE_MAX_E], scan[MOE_MAX_E], tscan[MOE_MAX_E];
  const int tid = threadIdx.x;
  cnt[tid] = 0;
  __syncthreads();
  for (int i = tid; i < S; i += 1024) {
    const int e = ids[i];
    if (e >= 0 && e < E) atomicAdd(&cnt[e], 1);
  }
  __syncthreads();
  const int c = cnt[tid], nt = (c + BM - 1) / BM;
  scan[tid] = c;
  tscan[tid] = nt;
  __syncthreads();
  for (int d = 1; d < MOE_MAX_E; d <<= 1) {
    const int a = tid >= d ? scan[tid - d] : 0;
    const int b = tid >= d ? tscan[tid - d] : 0;
    __syncthreads();
    scan[tid] += a;
    tscan[tid] += b;
    __syncthreads();
  }
  const int first = scan[tid] - c;
  if (tid < E) {
    off[tid] = first;
    for (int k = 0; k < nt; ++k) {
      const int at = tscan[tid] - nt + k;
      if (at < max_tiles) {
        tiles[2 * at] = tid;
        tiles[2 * at + 1] = first + k * BM;
      }
    }
  }
  if (tid == E - 1) off[E] = scan[tid];
  if (tid == 0) tiles[2 * max_tiles] = min(tscan[MOE_MAX_E - 1], max_tiles);
  for (int i = tscan[MOE_MAX_E - 1] + tid; i < max_tiles; i += 1024)
    tiles[2 * i] = -1;
  cnt[tid] = first;
  __syncthreads();
  for (int i = tid; i < S; i += 1024) {
    const int e = ids[i];
    if (e >= 0 && e < E) sorted[atomicAdd(&cnt[e], 1)] = i;
  }
}

// ---------------------------------------------------------------------------
// skinny: grid (N / 64, E), at most 32 tokens
// ---------------------------------------------------------------------------

DEVINL float relu_sq(float z) {
  const float r = fmaxf(z, 0.f);
  return r * r;
}

// UP: A row = slot / top (the token), out row = slot, activation.
// else: A row = slot, out row = slot.
template <int UP, bool FULL>  // FULL: K % 256 == 0
__global__ __launch_bounds__(256) void moe_skinny_kernel(
    const unsigned short* __restrict__ A, const unsigned short* __restrict__ W,
    const int* __restrict__ ids, const float* __restrict__ wts,
    unsigned short* __restrict__ C, int S, int top, int N, int K, int lda,
    int ldc, GluConst glu) {
  constexpr int NW = UP ? UP : 1, U = 4, KSTEP = 256, RS = KSTEP + 8;
  __shared__ __attribute__((aligned(16))) unsigned short at[32 * RS];
  __shared__ int slots[32];
  __shared__ int n_slots;
  const int e = blockIdx.y;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  if (wave == 0) {
    int n = 0;
    for (int b = 0; b < S; b += WAVE) {
      const bool mine = b + lane < S && ids[b + lane] == e;
      const unsigned long long m = __builtin_amdgcn_ballot_w64(mine);
      const int at_ = n + __popcll(m & ((1ull << lane) - 1));
      if (mine && at_ < 32) slots[at_] = b + lane;
      n += __popcll(m);
    }
    if (lane == 0) n_slots = min(n, 32);  // choices of a token are distinct
  }
  __syncthreads();
  const int cnt = n_slots;
  if (cnt == 0) return;
  const int mt = cnt > 16 ? 2 : 1;
  const int n0 = xcd_order(blockIdx.x, gridDim.x) * 64 + wave * 16;
  const unsigned short* wr[NW];
#pragma unroll
  for (int w = 0; w < NW; ++w)
    wr[w] = W + (((long)e * NW + w) * N + n0 + li) * K + hi * 8;

  f32x4 acc[NW][2];
#pragma unroll
  for (int w = 0; w < NW; ++w)
#pragma unroll
    for (int t = 0; t < 2; ++t) acc[w][t] = (f32x4){0.f, 0.f, 0.f, 0.f};

  const unsigned short* arow[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int flat = threadIdx.x + j * 256;
    const int sl = slots[min(flat / 32, cnt - 1)];
    arow[j] = A + (long)(UP ? sl / top : sl) * lda + (flat % 32) * 8;
  }
  short8 areg[4];
  auto load_a = [&](int k) {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j >= 2 * mt) break;
      areg[j] = short8{};
      if (FULL || k + (int)(threadIdx.x % 32) * 8 < K)
        areg[j] = *reinterpret_cast<const short8*>(arow[j] + k);
    }
  };
  auto store_a = [&]() {
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j >= 2 * mt) break;
      const int flat = threadIdx.x + j * 256;
      *reinterpret_cast<short8*>(at + (flat / 32) * RS + (flat % 32) * 8) = areg[j];
    }
  };
  bf16x8 b0[NW][U], b1[NW][U];
  auto load_w = [&](bf16x8 (&b)[NW][U], int k) {
#pragma unroll
    for (int w = 0; w < NW; ++w)
#pragma unroll
      for (int u = 0; u < U; ++u) {
        if constexpr (FULL) {
          b[w][u] = as_bf16x8(
              *reinterpret_cast<const short8*>(wr[w] + k + u * 32));
        } else {
          b[w][u] = as_bf16x8(short8{});
          if (k + u * 32 < K)
            b[w][u] = as_bf16x8(
                *reinterpret_cast<const short8*>(wr[w] + k + u * 32));
        }
      }
  };
  auto mma = [&](const bf16x8 (&b)[NW][U], int half) {
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        if (t >= mt) break;
        const bf16x8 af = as_bf16x8(*reinterpret_cast<const short8*>(
            at + (t * 16 + li) * RS + half * 128 + u * 32 + hi * 8));
#pragma unroll
        for (int w = 0; w < NW; ++w)
          acc[w][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af, b[w][u],
                                                              acc[w][t], 0, 0, 0);
      }
  };

  load_a(0);
  load_w(b0, 0);
  store_a();
  __syncthreads();
  for (int k = 0; k < K; k += KSTEP) {
    const bool more = k + KSTEP < K;
    if (more) load_a(k + KSTEP);
    load_w(b1, k + 128);
    __builtin_amdgcn_sched_barrier(0);
    mma(b0, 0);
    if (more) load_w(b0, k + KSTEP);
    __builtin_amdgcn_sched_barrier(0);
    mma(b1, 1);
    if (more) {
      __syncthreads();
      store_a();
      __syncthreads();
    }
  }
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int m = t * 16 + hi * 4 + r;
      if (m >= cnt) continue;
      const int sl = slots[m];
      const float w = wts ? wts[sl] : 1.f;
      float v = acc[0][t][r] * w;
      if constexpr (UP == 2) v = gated(glu, v, acc[NW - 1][t][r] * w);
      if constexpr (UP == 1) v = relu_sq(v);
      C[(long)sl * ldc + n0 + li] = f2bf(v);
    }
}

// ---------------------------------------------------------------------------
// tile: grid of column tiles * row tiles; K % 64 == 0
// ---------------------------------------------------------------------------

// UP: A row = sorted slot / top, out row = sorted position, N = activations
//     (two planes: 128 per tile, 128 gate rows and 128 up rows of W; one: 256).
// else: A row = sorted position, out row = slot, 256 columns per tile.
//
// A BM x 256 tile per workgroup; each of the four waves holds all BM rows of
// 64 columns, so a W fragment read from LDS feeds BM / 16 MFMAs. LDS rows are
// 64 B (32 of K) in four 16 B pieces, piece c of row r at c ^ (r / 4 % 4).
template <int BM, int UP>
__global__ __launch_bounds__(256, BM > 64 ? 2 : 3) void moe_tile_kernel(
    const unsigned short* __restrict__ A, const unsigned short* __restrict__ W,
    const int* __restrict__ off, const int* __restrict__ sorted,
    const int* __restrict__ tiles, const float* __restrict__ wts,
    unsigned short* __restrict__ C, int max_tiles, int ntn, int top, int N,
    int K, int lda, int ldc, GluConst glu) {
  constexpr int BK = 32, RB = BK * 2, BN = 256, HN = BN / 2;
  constexpr int AI = BM * 4 / 256, BI = BN * 4 / 256;  // 16 B pieces per thread
  constexpr int MT = BM / 16, NT = 4;
  __shared__ __attribute__((aligned(16))) unsigned char lds[2][(BM + BN) * RB];

  // eight row tiles by all column tiles at a time: the workgroups that run
  // together share both operands
  const int nrt = tiles[2 * max_tiles];
  const int total = nrt * ntn;
  if ((int)blockIdx.x >= total) return;
  const int id = xcd_order(blockIdx.x, total);
  const int grp = id / (8 * ntn), in_grp = id % (8 * ntn);
  const int gsz = min(8, nrt - grp * 8);
  const int rt = grp * 8 + in_grp % gsz, nt = in_grp / gsz;
  const int e = tiles[2 * rt];
  const int p0 = tiles[2 * rt + 1];
  const int cnt = min(BM, off[e + 1] - p0);
  const int n0 = nt * (UP == 2 ? HN : BN);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
  const int lane = threadIdx.x & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;

  const unsigned short* ap[AI];
  const unsigned short* bp[BI];
#pragma unroll
  for (int i = 0; i < AI; ++i) {
    const int ch = (i * 4 + wave) * 64 + lane;
    const int r = ch / 4, c = (ch % 4) ^ ((r >> 2) & 3);
    const int p = p0 + min(r, cnt - 1);
    ap[i] = A + (long)(UP ? sorted[p] / top : p) * lda + c * 8;
  }
#pragma unroll
  for (int i = 0; i < BI; ++i) {
    const int ch = (i * 4 + wave) * 64 + lane;
    const int r = ch / 4, c = (ch % 4) ^ ((r >> 2) & 3);
    const long wrow =
        UP == 2 ? ((long)e * 2 + r / HN) * N + min(n0 + r % HN, N - 1)
                : (long)e * N + min(n0 + r, N - 1);
    bp[i] = W + wrow * K + c * 8;
  }
  auto issue = [&](int k, int buf) {
#pragma unroll
    for (int i = 0; i < AI; ++i)
      copy16_to_lds(ap[i] + k, lds[buf] + (i * 4 + wave) * 1024);
#pragma unroll
    for (int i = 0; i < BI; ++i)
      copy16_to_lds(bp[i] + k, lds[buf] + BM * RB + (i * 4 + wave) * 1024);
  };
  // W rows of this wave's four column tiles: two planes pair gate and up columns
  int brow[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
    brow[n] = (UP == 2 ? (n >> 1) * HN + wave * 32 + (n & 1) * 16
                  : wave * 64 + n * 16) + li;

  f32x4 acc[MT][NT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[m][n] = (f32x4){0.f, 0.f, 0.f, 0.f};

  issue(0, 0);
  __syncthreads();
  int buf = 0;
  for (int k = 0; k < K; k += BK) {
    if (k + BK < K) issue(k + BK, buf ^ 1);
    bf16x8 wf[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n)
      wf[n] = as_bf16x8(*reinterpret_cast<const short8*>(
          lds[buf] + (BM + brow[n]) * RB + ((hi ^ ((brow[n] >> 2) & 3)) * 16)));
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const int r = m * 16 + li;
      const bf16x8 af = as_bf16x8(*reinterpret_cast<const short8*>(
          lds[buf] + r * RB + ((hi ^ ((r >> 2) & 3)) * 16)));
#pragma unroll
      for (int n = 0; n < NT; ++n)
        acc[m][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[n], af,
                                                            acc[m][n], 0, 0, 0);
    }
    __syncthreads();
    buf ^= 1;
  }

  // a lane holds columns hi*4..hi*4+3 of row li in every tile
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int r = m * 16 + li;
    if (r >= cnt) continue;
    const int sl = sorted[p0 + r];
    const float w = wts ? wts[sl] : 1.f;
    if constexpr (UP == 2) {
#pragma unroll
      for (int n = 0; n < 2; ++n) {
        const int col = n0 + wave * 32 + n * 16 + hi * 4;
        if (col >= N) continue;
        float v[4];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          v[j] = gated(glu, acc[m][n][j] * w, acc[m][n + 2][j] * w);
        stv<4>(C + (long)(p0 + r) * ldc + col, v);
      }
    } else {
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const int col = n0 + wave * 64 + n * 16 + hi * 4;
        if (col >= N) continue;
        float v[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          v[j] = acc[m][n][j] * w;
          if constexpr (UP == 1) v[j] = relu_sq(v[j]);
        }
        stv<4>(C + (long)(UP ? p0 + r : sl) * ldc + col, v);
      }
    }
  }
}

// ---------------------------------------------------------------------------
// plain f32: 64 x 64 tiles, same row tiles (BM = 64)
// ---------------------------------------------------------------------------

template <int UP>
__global__ __launch_bounds__(256) void moe_simple_kernel(
    const float* __restrict__ A, const float* __restrict__ W,
    const int* __restrict__ off, const int* __restrict__ sorted,
    const int* __restrict__ tiles, const float* __restrict__ wts,
    float* __restrict__ C, int top, int N, int K, int lda, int ldc,
    GluConst glu) {
  constexpr int NW = UP ? UP : 1, BK = 16;
  __shared__ float al[BK][64 + 4], wl[NW][BK][64 + 4];
  const int e = tiles[2 * blockIdx.y];
  if (e < 0) return;
  const int p0 = tiles[2 * blockIdx.y + 1];
  const int cnt = min(64, off[e + 1] - p0);
  const int n0 = blockIdx.x * 64;
  const int tx = threadIdx.x % 16, ty = threadIdx.x / 16;
  float acc[NW][4][4] = {};
  for (int k = 0; k < K; k += BK) {
    for (int i = threadIdx.x; i < 64 * BK; i += 256) {
      const int r = i / BK, c = i % BK;
      const int p = p0 + min(r, cnt - 1);
      al[c][r] = A[(long)(UP ? sorted[p] / top : p) * lda + k + c];
      for (int w = 0; w < NW; ++w)
        wl[w][c][r] = W[(((long)e * NW + w) * N + n0 + r) * K + k + c];
    }
    __syncthreads();
    for (int c = 0; c < BK; ++c)
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int w = 0; w < NW; ++w)
#pragma unroll
          for (int j = 0; j < 4; ++j)
            acc[w][i][j] += al[c][ty * 4 + i] * wl[w][c][tx * 4 + j];
    __syncthreads();
  }
  for (int i = 0; i < 4; ++i) {
    const int r = ty * 4 + i;
    if (r >= cnt) continue;
    const int sl = sorted[p0 + r];
    const float w = wts ? wts[sl] : 1.f;
    for (int j = 0; j < 4; ++j) {
      float v = acc[0][i][j] * w;
      if constexpr (UP == 2) v = gated(glu, v, acc[NW - 1][i][j] * w);
      if constexpr (UP == 1) v = relu_sq(v);
      C[(long)(UP ? p0 + r : sl) * ldc + n0 + tx * 4 + j] = v;
    }
  }
}
