// Torch bindings of differential attention over ragged batches (module
// _hip_differential).
//
// Host side: shape checks, template dispatch, launch shapes.

#include "host.h"
#include "common.h"
#include "rows.hip"
#include "attn_differential.hip"

template <int DK, int DV>
static void launch_tiled(DiffArgs& a, const Tensor& pre, const Tensor& dec,
                         long max_new, long max_ctx, const Tensor& like) {
  const int Hg = a.H / a.G;
  if (pre.numel() > 0) {
    a.list = pre.data_ptr<int>();
    // half as many rows a workgroup where there are not enough of them
    const long rows = max_new * Hg;
    by_bool((rows + 127) / 128 * a.G * pre.numel() >= 256, [&](auto many) {
      constexpr int NW = decltype(many)::value ? 8 : 4;
      constexpr size_t lds = 2 * DiffTile<DK, DV>::BYTES;
      auto k = attn_diff_prefill_kernel<DK, DV, NW>;
      allow_lds(k, lds);
      k<<<dim3((rows + 16 * NW - 1) / (16 * NW), a.G, pre.numel()), NW * 64, lds,
          cur_stream()>>>(a);
    });
    check_launch();
  }
  if (dec.numel() == 0) return;
  a.list = dec.data_ptr<int>();
  const long units = dec.numel() * a.G * ((Hg + 7) / 8);
  // enough workgroups to fill the chip with at least two tiles for each wave, one
  // where there are few
  const long tiles = (seen_keys(a, max_ctx) + 31) / 32 + 1;
  a.n_split = (int)std::max<long>(
      1, std::min<long>({32, 512 / std::max<long>(1, units),
                         tiles / (units < 32 ? 4 : 8)}));
  Tensor pml, pacc;
  if (a.n_split > 1) {
    auto o = like.options().dtype(at::kFloat);
    pml = torch::empty({units * a.n_split, 16, 2}, o);
    pacc = torch::empty({units * a.n_split, 16, DV}, o);
    a.pml = pml.data_ptr<float>();
    a.pacc = pacc.data_ptr<float>();
  }
  attn_diff_decode_kernel<2 * DK, DV>
      <<<dim3(units, a.n_split), 256, 0, cur_stream()>>>(a);
  check_launch();
  if (a.n_split > 1) {
    attn_diff_combine_kernel<<<units, 256, 0, cur_stream()>>>(a);
    check_launch();
  }
}

// q (N, H, 2, dk), kp (np, G, P, 2 * dk), vp (np, G, dvp, P) -> out (N, >= H *
// vdim)
void attn_differential(Tensor q, Tensor kp, Tensor vp, Tensor table,
                       Tensor tok_seq, Tensor tok_pos, Tensor cu, Tensor q_start,
                       Tensor pre, Tensor dec, long max_new, long max_ctx,
                       long dim, long vdim, double scale, long window, long chunk,
                       double lam, double factor, double eps, Tensor out) {
  check_act(q);
  const auto ta = q.scalar_type();
  TORCH_CHECK(q.dim() == 4 && q.is_contiguous() && q.size(2) == 2);
  DiffArgs a{};
  const long N = q.size(0);
  a.H = q.size(1);
  a.dkp = q.size(3);
  for (const Tensor& t : {kp, vp})
    TORCH_CHECK(t.is_cuda() && t.dim() == 4 && t.is_contiguous() &&
                    t.scalar_type() == ta,
                "pages must have the element type of q");
  a.G = kp.size(1);
  a.P = kp.size(2);
  a.dvp = vp.size(2);
  a.dim = (int)dim;
  a.vdim = (int)vdim;
  TORCH_CHECK(a.H % a.G == 0 && kp.size(3) == 2 * a.dkp && vp.size(1) == a.G &&
              vp.size(3) == a.P && vp.size(0) == kp.size(0) && dim >= 1 &&
              vdim >= 1 && dim <= a.dkp && vdim <= a.dvp);
  for (const Tensor& t : {table, tok_seq, tok_pos, cu, q_start, pre, dec})
    CHECK_I32(t);
  TORCH_CHECK(table.dim() == 2 && tok_seq.numel() == N && tok_pos.numel() == N &&
              cu.numel() == table.size(0) + 1 &&
              q_start.numel() == table.size(0));
  TORCH_CHECK(out.is_cuda() && out.dim() == 2 && out.size(0) == N &&
              out.stride(1) == 1 && out.scalar_type() == ta &&
              out.size(1) >= a.H * vdim);
  if (N == 0) return;
  a.q = q.data_ptr();
  a.kp = kp.data_ptr();
  a.vp = vp.data_ptr();
  a.table = table.data_ptr<int>();
  a.maxp = table.size(1);
  a.tok_seq = tok_seq.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  a.cu = cu.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.out = out.data_ptr();
  a.ldo = out.stride(0);
  a.window = (int)window;
  a.chunk = (int)chunk;
  a.scale = (float)scale;
  a.n_split = 1;
  a.lam = (float)lam;
  a.factor = (float)factor;
  a.eps = (float)eps;

  while (1 << a.p_log2 < a.P) ++a.p_log2;
  auto size_ok = [](int d, int most) {
    return d <= most && (d == 32 || d == 64 || d == 128 || d == 256);
  };
  if (ta == at::kBFloat16 && size_ok(a.dkp, 128) && size_ok(a.dvp, 256) &&
      a.P % 8 == 0 && 32 % a.P == 0) {
    auto by_value = [&](auto dk) {
      constexpr int DK = decltype(dk)::value;
      auto go = [&](auto dv) {
        launch_tiled<DK, decltype(dv)::value>(a, pre, dec, max_new, max_ctx, q);
      };
      if (a.dvp == 32) go(std::integral_constant<int, 32>{});
      else if (a.dvp == 64) go(std::integral_constant<int, 64>{});
      else if (a.dvp == 128) go(std::integral_constant<int, 128>{});
      else go(std::integral_constant<int, 256>{});
    };
    if (a.dkp == 32) by_value(std::integral_constant<int, 32>{});
    else if (a.dkp == 64) by_value(std::integral_constant<int, 64>{});
    else by_value(std::integral_constant<int, 128>{});
    return;
  }
  // every map as a head of its own on the plain kernel, in 32 bits
  TORCH_CHECK(dim <= SIMPLE_MAXD && vdim <= SIMPLE_MAXD,
              "head size above ", SIMPLE_MAXD);
  const int H = a.H;
  auto y = torch::empty({N, 2 * H * vdim}, q.options().dtype(at::kFloat));
  AttnArgs s = a;
  s.H = 2 * H;
  s.maps = 2;
  s.out = y.data_ptr();
  s.ldo = 2 * H * vdim;
  by_type(ta, [&](auto t) {
    using T = decltype(t);
    attn_ragged_simple_kernel<T, float>
        <<<dim3(N, 2 * H), 64, 0, cur_stream()>>>(s);
    check_launch();
    attn_diff_join_kernel<T><<<dim3(N, H), 64, 0, cur_stream()>>>(
        y.data_ptr<float>(), (T*)out.data_ptr(), a.ldo, H, (int)vdim, a.lam,
        a.factor, a.eps);
  });
  check_launch();
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("attn_differential", &attn_differential);
}
