// Gated linear recurrent unit (RG-LRU) with its short convolution and output
// branch over ragged batches. Per channel, with x and y columns of the input
// projection,
//     u = causal convolution of x + x bias,
//     r, i = sigmoid(block-diagonal matrix of u + bias),
//     log a = decay * r,  S <- a S + sqrt(1 - a^2) i u,   out = S gelu(y + y bias)
// with a negative decay per channel. State: S and the convolution's last
// taps - 1 inputs, 32-bit. A sequence whose portion starts at position 0 starts
// from zero, whatever its slot holds.
//
//  rglru_conv_kernel   u of all rows; the inputs' state of single tokens moves on
//                      here, that of portions with the kernel that ends them.
//  rglru_step_kernel   single tokens: both gates as one MFMA product per block of
//                      channels, the recurrence and the output.
//  rglru_gates_kernel  portions in chunks of 64 tokens: both gates, and the
//                      chunk's own recurrence from zero: h and the product F
//                      of the factors a since the chunk's start, 32-bit.
//  rglru_carry_kernel  S from chunk to chunk, and the states.
//  rglru_out_kernel    (h + F S) gelu(y), all rows side by side.
//  rglru_seq_kernel    token by token from finished gate products: 32-bit runs.

#pragma once
#include "common.h"
#include "rows.hip"

static constexpr int LRU_C = 64;      // tokens of a chunk
static constexpr int LRU_KC = 256;    // inner step of the gate product

struct LruArgs {
  Parts y;             // columns y_off.., x_off..
  const float* yb;     // (W,) biases
  const float* xb;
  const float* taps;   // (K, W), the last row is the current token's
  const float* cb;     // (W,)
  const void* gw;      // (B, 2, Cp, Cp) bf16: [out, in] of r and of i, padded
  const float* gb;     // (2, W)
  const float* decay;  // (W,) < 0
  float* S;            // (slots, W)
  float* conv;         // (slots, K - 1, W), oldest first
  void* u;             // (N, B * Cp): block b's channels from b * Cp on
  const float* z;      // seq: (B, N, 2 * Cb) gate products
  float* h;            // (N, W) chunk form
  float* F;            // (N, W)
  float* S0;           // (chunks, W): S before each chunk
  void* out;           // (N, ldo), W columns
  const int* slots;
  const int* tok_seq;
  const int* tok_pos;
  const int* q_start;
  const int* cu;
  const int* list;
  const int* row0;     // (chunks,)
  const int* len;
  const int* ccu;      // (listed + 1,)
  long ldo;
  int N, y_off, x_off, W, K, B, Cb, Cp, n_list;
};

// x + bias of V channels
template <typename TP, int V>
DEVINL void lru_input(const LruArgs& a, long t, int c, float* o) {
  float b[V];
  fold_parts<TP, V>(a.y, t, a.x_off + c, o);
  ldv<V>(a.xb + c, b);
#pragma unroll
  for (int j = 0; j < V; ++j) o[j] += b[j];
}

DEVINL float gelu_tanh_f(float z) {
  // 0.5 (1 + tanh v) = sigmoid(2 v)
  return z * sigmoid_f(1.5957691216057308f * (z + 0.044715f * z * z * z));
}

// The gate of channel c's output, gelu(y + bias).
template <typename TP>
DEVINL float lru_branch(const LruArgs& a, long t, int c) {
  float v[1];
  fold_parts<TP, 1>(a.y, t, a.y_off + c, v);
  return gelu_tanh_f(v[0] + a.yb[c]);
}

// 1 - e^z for z <= 0. Near zero the series, where the difference would cancel.
DEVINL float one_minus_exp(float z) {
  const float far = 1.f - fast_expf(z);
  const float t = 1.f + z * (1.f / 5) * (1.f + z * (1.f / 6) * (1.f + z * (1.f / 7)));
  const float near =
      -z * (1.f + z * (1.f / 2) * (1.f + z * (1.f / 3) * (1.f + z * (1.f / 4) * t)));
  return z > -0.5f ? near : far;
}

// Gate logits -> the state's factor and what enters it. FAST: the hardware's
// exponential and reciprocal, an ulp or two each.
template <bool FAST>
DEVINL void lru_step(float zr, float zi, float u, float decay, float& f, float& x) {
  if constexpr (FAST) {
    const float la = decay * sigmoid_f(zr);
    f = fast_expf(la);
    x = __builtin_amdgcn_sqrtf(one_minus_exp(2.f * la)) * sigmoid_f(zi) * u;
  } else {
    const float la = decay / (1.f + expf(-zr));
    f = expf(la);
    x = sqrtf(-expm1f(2.f * la)) / (1.f + expf(-zi)) * u;
  }
}

// Channel c's last K - 1 inputs after the n tokens of sequence s, unless the
// convolution kernel kept them (n = 1); one thread a channel, ascending, so that
// an entry is read before it is overwritten.
template <typename TP>
DEVINL void lru_keep_inputs(const LruArgs& a, int s, int n, int c) {
  if (n == 1) return;
  const int start = a.q_start[s];
  const long t0 = a.cu[s];
  float* st = a.conv + (long)a.slots[s] * (a.K - 1) * a.W + c;
  for (int e = 0; e < a.K - 1; ++e) {
    const int at = n - (a.K - 1) + e;   // place in the portion
    float v[1] = {0.f};
    if (at >= 0) lru_input<TP, 1>(a, t0 + at, c, v);
    else if (start + at >= 0) v[0] = st[(long)(n + e) * a.W];
    st[(long)e * a.W] = v[0];
  }
}

// grid (channels / (256 V), N). Where the row is all that its sequence brings,
// the thread is also the only reader of the kept inputs and moves them on.
template <typename TP, typename T, int V>
__global__ __launch_bounds__(256) void rglru_conv_kernel(LruArgs a) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * V;
  if (c >= a.W) return;
  const long t = blockIdx.y;
  const int pos = a.tok_pos[t];
  if (pos < 0) return;
  const int s = a.tok_seq[t], start = a.q_start[s];
  const bool one = a.cu[s + 1] - a.cu[s] == 1;
  float* st = a.conv + (long)a.slots[s] * (a.K - 1) * a.W + c;
  float o[V], x[V], w[V], held[V];
  ldv<V>(a.cb + c, o);
  int j = 0;
  for (; j < a.K && j <= pos; ++j) {
    const long e = a.K - 1 + pos - j - start;   // the input's entry, if kept
    if (pos - j >= start) lru_input<TP, V>(a, t - j, c, x);
    else ldv<V>(st + e * a.W, x);
    if (one && j > 0) stv<V>(st + e * a.W, held);
    ldv<V>(a.taps + (long)(a.K - 1 - j) * a.W + c, w);
#pragma unroll
    for (int k = 0; k < V; ++k) {
      o[k] += w[k] * x[k];
      held[k] = x[k];
    }
  }
  if (one && j < a.K) stv<V>(st + (long)(a.K - 1 - j) * a.W, held);
  T* u = (T*)a.u + t * a.B * a.Cp;
  stv<V>(u + c / a.Cb * a.Cp + c % a.Cb, o);
}

// Single tokens: gates, recurrence and output. grid (B * Cp / 16, rows / 16), a
// wave: both gates of 16 channels and up to 16 listed rows.
template <typename TP>
__global__ __launch_bounds__(64) void rglru_step_kernel(LruArgs a) {
  const int lane = threadIdx.x, li = lane & 15, hi = lane >> 4;
  const int tiles = a.Cp / 16, b = blockIdx.x / tiles;
  const int n0 = blockIdx.x % tiles * 16;
  const int m0 = blockIdx.y * 16, cnt = min(16, a.n_list - m0);
  const long ldu = (long)a.B * a.Cp;
  const unsigned short* u = (const unsigned short*)a.u + (long)b * a.Cp;
  const unsigned short* xr =
      u + (long)a.cu[a.list[m0 + min(li, cnt - 1)]] * ldu + hi * 8;
  const unsigned short* wr[2];
#pragma unroll
  for (int g = 0; g < 2; ++g)
    wr[g] = (const unsigned short*)a.gw +
            (((long)b * 2 + g) * a.Cp + n0 + li) * a.Cp + hi * 8;

  // what the epilogue needs is asked for ahead of the product
  const int cl = n0 + li, c = b * a.Cb + min(cl, a.Cb - 1);
  const float br = a.gb[c], bi = a.gb[a.W + c], dec = a.decay[c], yb = a.yb[c];
  long t[4];
  int pos[4];
  float S[4], uv[4], y[4];
  float* sp[4];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int s = a.list[m0 + min(hi * 4 + r, cnt - 1)];
    t[r] = a.cu[s];
    sp[r] = a.S + (long)a.slots[s] * a.W + c;
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    pos[r] = a.tok_pos[t[r]];
    S[r] = *sp[r];
    uv[r] = bf2f(u[t[r] * ldu + min(cl, a.Cb - 1)]);
    fold_parts<TP, 1>(a.y, t[r], a.y_off + c, y + r);
  }

  f32x4 acc[2];
  acc[0] = acc[1] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
  for (int k = 0; k < a.Cp; k += 32) {
    const bf16x8 x = as_bf16x8(*reinterpret_cast<const short8*>(xr + k));
#pragma unroll
    for (int g = 0; g < 2; ++g)
      acc[g] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
          x, as_bf16x8(*reinterpret_cast<const short8*>(wr[g] + k)), acc[g], 0, 0, 0);
  }
  if (cl >= a.Cb) return;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    if (hi * 4 + r >= cnt || pos[r] < 0) continue;   // none, or an empty slot
    float f, x;
    lru_step<true>(acc[0][r] + br, acc[1][r] + bi, uv[r], dec, f, x);
    x += pos[r] > 0 ? S[r] * f : 0.f;
    *sp[r] = x;
    ((unsigned short*)a.out)[t[r] * a.ldo + c] = cvt_bf(x * gelu_tanh_f(y[r] + yb));
  }
}

// grid (B * Cp / 64, chunks): a wave holds both gates of 16 channels.
__global__ __launch_bounds__(256) void rglru_gates_kernel(LruArgs a) {
  constexpr int LDU = LRU_KC + 8, LDC = 65;
  __shared__ __attribute__((aligned(16))) unsigned char
      lds[64 * LDU * 2 > 2 * 64 * LDC * 4 ? 64 * LDU * 2 : 2 * 64 * LDC * 4];
  unsigned short* us = (unsigned short*)lds;
  const int tid = threadIdx.x, wave = tid / WAVE, lane = tid & (WAVE - 1);
  const int li = lane & 15, hi = lane >> 4;
  const int tiles = a.Cp / 64, b = blockIdx.x / tiles;
  const int n0 = blockIdx.x % tiles * 64;     // first channel in the block
  const int cnt = a.len[blockIdx.y];
  const long row0 = a.row0[blockIdx.y];
  const int mt = (cnt + 15) / 16;
  const unsigned short* gw = (const unsigned short*)a.gw;
  const unsigned short* wr[2];
#pragma unroll
  for (int g = 0; g < 2; ++g)
    wr[g] = gw + (((long)b * 2 + g) * a.Cp + n0 + wave * 16 + li) * a.Cp + hi * 8;
  const long ldu = (long)a.B * a.Cp;
  const unsigned short* u = (const unsigned short*)a.u + (long)b * a.Cp;

  f32x4 acc[2][4];
#pragma unroll
  for (int g = 0; g < 2; ++g)
#pragma unroll
    for (int m = 0; m < 4; ++m) acc[g][m] = (f32x4){0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < a.Cp; k0 += LRU_KC) {
    const int kn = min(LRU_KC, a.Cp - k0);   // a multiple of 64
    const int pc = kn / 8;
    for (int i = tid; i < mt * 16 * pc; i += 256) {
      const int r = i / pc, c = i % pc * 8;
      *reinterpret_cast<short8*>(us + r * LDU + c) =
          *reinterpret_cast<const short8*>(u + (row0 + min(r, cnt - 1)) * ldu + k0 + c);
    }
    __syncthreads();
#pragma unroll 4
    for (int k = 0; k < kn; k += 32) {
      bf16x8 w[2];
#pragma unroll
      for (int g = 0; g < 2; ++g)
        w[g] = as_bf16x8(*reinterpret_cast<const short8*>(wr[g] + k0 + k));
#pragma unroll
      for (int m = 0; m < 4; ++m) {
        if (m >= mt) break;
        const bf16x8 x = as_bf16x8(*reinterpret_cast<const short8*>(
            us + (m * 16 + li) * LDU + k + hi * 8));
#pragma unroll
        for (int g = 0; g < 2; ++g)
          acc[g][m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x, w[g], acc[g][m],
                                                              0, 0, 0);
      }
    }
    __syncthreads();
  }

  const int cl = n0 + wave * 16 + li;           // channel in the block
  const int c = b * a.Cb + min(cl, a.Cb - 1);
  const float br = a.gb[c], bi = a.gb[a.W + c], dec = a.decay[c];
  float* hs = (float*)lds;          // (64, LDC): state from zero
  float* fs = hs + 64 * LDC;        // factors, then their products
#pragma unroll
  for (int m = 0; m < 4; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int at = m * 16 + hi * 4 + r;
      float f = 1.f, x = 0.f;
      if (at < cnt)
        lru_step<true>(acc[0][m][r] + br, acc[1][m][r] + bi,
                       bf2f(u[(row0 + at) * ldu + cl]), dec, f, x);
      hs[at * LDC + wave * 16 + li] = x;
      fs[at * LDC + wave * 16 + li] = f;
    }
  __syncthreads();
  // a thread takes 16 tokens of a channel, then adds what came before them
  const int cc = tid & 63, t0 = tid / 64 * 16;
  float S[16], F[16];
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    S[t] = hs[(t0 + t) * LDC + cc];
    F[t] = fs[(t0 + t) * LDC + cc];
  }
#pragma unroll
  for (int t = 1; t < 16; ++t) {
    S[t] += S[t - 1] * F[t];
    F[t] *= F[t - 1];
  }
  hs[(t0 + 15) * LDC + cc] = S[15];
  fs[(t0 + 15) * LDC + cc] = F[15];
  __syncthreads();
  float S0 = 0.f, F0 = 1.f;
  for (int t = 15; t < t0; t += 16) {
    const float f = fs[t * LDC + cc];
    S0 = S0 * f + hs[t * LDC + cc];
    F0 *= f;
  }
  if (n0 + cc >= a.Cb) return;
  const long o = row0 * a.W + b * a.Cb + n0 + cc;
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    if (t0 + t >= cnt) break;
    a.h[o + (long)(t0 + t) * a.W] = S[t] + S0 * F[t];
    a.F[o + (long)(t0 + t) * a.W] = F[t] * F0;
  }
}

// grid (channels / 64, listed sequences)
template <typename TP>
__global__ __launch_bounds__(64) void rglru_carry_kernel(LruArgs a) {
  const int c = blockIdx.x * 64 + threadIdx.x;
  if (c >= a.W) return;
  const int s = a.list[blockIdx.y];
  float* sp = a.S + (long)a.slots[s] * a.W + c;
  float S = a.q_start[s] != 0 ? *sp : 0.f;
  const int c0 = a.ccu[blockIdx.y], c1 = a.ccu[blockIdx.y + 1];
  constexpr int U = 8;   // chunks whose loads are in flight together
  for (int k = c0; k < c1; k += U) {
    float h[U], f[U];
#pragma unroll
    for (int j = 0; j < U; ++j) {
      const int ch = min(k + j, c1 - 1);
      const long at = ((long)a.row0[ch] + a.len[ch] - 1) * a.W + c;
      h[j] = a.h[at];
      f[j] = a.F[at];
    }
#pragma unroll
    for (int j = 0; j < U; ++j) {
      if (k + j >= c1) break;
      a.S0[(long)(k + j) * a.W + c] = S;
      S = h[j] + S * f[j];
    }
  }
  *sp = S;
  lru_keep_inputs<TP>(a, s, a.cu[s + 1] - a.cu[s], c);
}

// grid (channels / (256 V), 4, chunks): 16 rows a workgroup
template <typename TP, typename T, int V>
__global__ __launch_bounds__(256) void rglru_out_kernel(LruArgs a) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * V;
  if (c >= a.W) return;
  const int ch = blockIdx.z, end = min(a.len[ch], (int)blockIdx.y * 16 + 16);
  float S[V], yb[V];
  ldv<V>(a.S0 + (long)ch * a.W + c, S);
  ldv<V>(a.yb + c, yb);
#pragma unroll 4
  for (int i = blockIdx.y * 16; i < end; ++i) {
    const long t = a.row0[ch] + i;
    float h[V], f[V], y[V];
    ldv<V>(a.h + t * a.W + c, h);
    ldv<V>(a.F + t * a.W + c, f);
    fold_parts<TP, V>(a.y, t, a.y_off + c, y);
#pragma unroll
    for (int j = 0; j < V; ++j)
      h[j] = (h[j] + f[j] * S[j]) * gelu_tanh_f(y[j] + yb[j]);
    stv<V>((T*)a.out + t * a.ldo + c, h);
  }
}

// grid (channels / 64, listed sequences)
template <typename TP, typename T>
__global__ __launch_bounds__(64) void rglru_seq_kernel(LruArgs a) {
  const int c = blockIdx.x * 64 + threadIdx.x;
  if (c >= a.W) return;
  const int s = a.list[blockIdx.y];
  const int b = c / a.Cb, cl = c % a.Cb;
  float* sp = a.S + (long)a.slots[s] * a.W + c;
  const int t0 = a.cu[s], t1 = a.cu[s + 1];
  if (a.tok_pos[t0] < 0) return;   // empty slot
  float S = a.q_start[s] != 0 ? *sp : 0.f;
  const float br = a.gb[c], bi = a.gb[a.W + c], dec = a.decay[c];
  for (long t = t0; t < t1; ++t) {
    const float* z = a.z + ((long)b * a.N + t) * 2 * a.Cb + cl;
    float f, x;
    lru_step<false>(z[0] + br, z[a.Cb] + bi,
                    ldf((const T*)a.u + t * a.B * a.Cp + (long)b * a.Cp + cl), dec,
                    f, x);
    S = S * f + x;
    stf((T*)a.out + t * a.ldo + c, S * lru_branch<TP>(a, t, c));
  }
  *sp = S;
  lru_keep_inputs<TP>(a, s, t1 - t0, c);
}
