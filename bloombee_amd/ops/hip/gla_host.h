// Launches of the chunked recurrences of gla.hip.
#pragma once

#include "host.h"
#include "gla.hip"

static int pad_dim(long dim) {
  return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 256;
}
static int chunk_of(long dim) { return dim <= 128 ? 64 : 32; }


static size_t prep_lds(int dp, int C, long r) {
  return 4 * ((size_t)C * (dp + 4) + (C + dp) * r);
}

// All chunks: decays and keys, the state from chunk to chunk, outputs.
template <bool WRITES>
static void launch_chunks(const GlaChunkArgs& a, long chunks, long seqs, bool vec) {
  auto go = [&](auto dp, auto c) {
    constexpr int D = decltype(dp)::value, CC = decltype(c)::value;
    by_bool(vec, [&](auto v) {
      constexpr bool VEC = decltype(v)::value;
      auto prep = [] {
        if constexpr (WRITES) return hgrn_prep_kernel<D, CC, VEC>;
        else return gla_prep_kernel<D, CC, VEC>;
      }();
      const size_t l1 = prep_lds(D, CC, WRITES ? 0 : a.r);
      allow_lds(prep, l1);
      prep<<<dim3(chunks, a.H), 256, l1, cur_stream()>>>(a);
      check_launch();
      auto scan = gla_scan_kernel<D, CC, VEC>;
      const size_t l2 =
          4 * (2 * CC * (D == 32 ? 96 : D + 32) + CC * 72 + 2 * D);
      allow_lds(scan, l2);
      scan<<<dim3((a.vdim + 63) / 64, a.H, seqs), 256, l2, cur_stream()>>>(a);
      check_launch();
      auto fin = [&](auto nct) {
        constexpr int N = decltype(nct)::value;
        auto k = gla_out_kernel<D, CC, N, VEC, WRITES>;
        const size_t first =
            std::max(2 * (CC + 1) * (D + 4) + (WRITES ? 4 * CC * (D + 4) : 0),
                     CC * (N * 128 + 24));
        const size_t l3 = 2 * (first + 2 * CC * (D + 8) + 2 * CC * (CC + 8));
        allow_lds(k, l3);
        k<<<dim3(chunks, a.H), 512, l3, cur_stream()>>>(a);
        check_launch();
      };
      if (a.vdim <= 128) fin(std::integral_constant<int, 1>{});
      else if (a.vdim <= 256) fin(std::integral_constant<int, 2>{});
      else fin(std::integral_constant<int, 4>{});
    });
  };
  using I32 = std::integral_constant<int, 32>;
  using I64 = std::integral_constant<int, 64>;
  const int DP = pad_dim(a.dim);
  if (DP == 32) go(I32{}, I64{});
  else if (DP == 64) go(I64{}, I64{});
  else if (DP == 128) go(std::integral_constant<int, 128>{}, I64{});
  else go(std::integral_constant<int, 256>{}, I32{});
}
