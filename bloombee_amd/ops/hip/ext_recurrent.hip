// Torch bindings of the matrix memory and the gated linear recurrent unit over
// ragged batches (module _hip_recurrent).
//
// Host side: shape checks, template dispatch, launch shapes.

#include "host.h"
#include "common.h"
#include "rows.hip"
#include "mlstm.hip"
#include "rglru.hip"

// ---------------------------------------------------------------------------
// matrix memory
// ---------------------------------------------------------------------------

static void check_memory(const Tensor& gb, const Tensor& nw, const Tensor& S,
                         const Tensor& n, const Tensor& m, const Tensor& slots,
                         long H, long dim, long vdim) {
  for (const Tensor& t : {gb, nw, S, n, m}) CHECK_F32(t);
  CHECK_I32(slots);
  TORCH_CHECK(H >= 1 && dim >= 1 && vdim >= 1 && gb.numel() == 2 * H &&
              nw.numel() == H * vdim && S.dim() == 4 && S.size(1) == H &&
              S.size(2) == dim && S.size(3) == vdim);
  const long slots_n = S.size(0);
  TORCH_CHECK(n.numel() == slots_n * H * dim && m.numel() == slots_n * H);
}

// dims: [q_off, k_off, v_off, g_off, i_off, H, dim, vdim];
// consts: [query scale, cap, eps]
void mlstm_step(Tensor y, Tensor g, std::vector<long> dims,
                std::vector<double> consts, Tensor gb, Tensor nw, Tensor S,
                Tensor n, Tensor m, Tensor slots, Tensor tok_pos, Tensor cu,
                Tensor list, Tensor out) {
  TORCH_CHECK(dims.size() == 8 && consts.size() == 3);
  MlstmArgs a{};
  a.y = as_parts(y);
  CHECK_F32(g);
  a.g = as_parts(g);
  int* f[8] = {&a.q_off, &a.k_off, &a.v_off, &a.g_off, &a.i_off,
               &a.H, &a.dim, &a.vdim};
  for (int i = 0; i < 8; ++i) *f[i] = (int)dims[i];
  check_memory(gb, nw, S, n, m, slots, a.H, a.dim, a.vdim);
  for (const Tensor& t : {tok_pos, cu, list}) CHECK_I32(t);
  const long N = y.size(1);
  auto inside = [&](int off, long n) { return off >= 0 && off + n <= a.y.ld; };
  TORCH_CHECK(g.size(1) == N && a.i_off >= 0 && a.i_off + 2 * a.H <= a.g.ld &&
              inside(a.q_off, a.H * a.dim) && inside(a.k_off, a.H * a.dim) &&
              inside(a.v_off, a.H * a.vdim) && inside(a.g_off, a.H * a.vdim));
  TORCH_CHECK(tok_pos.numel() == N && cu.numel() == slots.numel() + 1);
  check_act(out);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == N && out.stride(1) == 1 &&
              out.size(1) >= a.H * a.vdim);
  a.qscale = (float)consts[0];
  a.cap = (float)consts[1];
  a.eps = (float)consts[2];
  a.gb = gb.data_ptr<float>();
  a.nw = nw.data_ptr<float>();
  a.S = S.data_ptr<float>();
  a.n = n.data_ptr<float>();
  a.m = m.data_ptr<float>();
  a.slots = slots.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  a.cu = cu.data_ptr<int>();
  a.list = list.data_ptr<int>();
  a.out = out.data_ptr();
  a.ldo = out.stride(0);
  if (list.numel() == 0) return;
  // few workgroups: more waves on each state
  const bool wide = a.H * list.numel() < 256;
  by_type(y.scalar_type(), [&](auto p) {
    by_type(out.scalar_type(), [&](auto t) {
      by_bool(a.vdim % 4 == 0, [&](auto v) {
        by_bool(wide, [&](auto w) {
          constexpr int V = decltype(v)::value ? 4 : 1;
          constexpr int B = decltype(w)::value ? 1024 : 256;
          const size_t lds = 4 * (((2 * a.dim + 3) & ~3) + (size_t)B * V +
                                  2 * ((a.vdim + 3) & ~3));
          auto k = mlstm_step_kernel<decltype(p), decltype(t), V, B>;
          allow_lds(k, lds);
          k<<<dim3(a.H, list.numel()), B, lds, cur_stream()>>>(a);
        });
      });
    });
  });
  check_launch();
}

static int pad_dim(long dim) {
  return dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 256;
}

// Tokens of a chunk, 0 where the chunk form does not take these sizes.
long mlstm_chunk(long dim, long vdim) {
  return dim <= 256 && vdim >= 1 && vdim <= 512 ? MLSTM_C : 0;
}

// Listed sequences in chunks; y (N, ldy) bf16, g (N, ldg) f32; dims, consts as
// mlstm_step. mprev (S, H): m of every sequence of the step; row0, len (chunks,);
// ccu (listed + 1,).
void mlstm_chunks(Tensor y, Tensor g, std::vector<long> dims,
                  std::vector<double> consts, Tensor gb, Tensor nw, Tensor S,
                  Tensor n, Tensor m, Tensor mprev, Tensor slots,
                  Tensor q_start, Tensor list, Tensor row0, Tensor len,
                  Tensor ccu, Tensor out) {
  TORCH_CHECK(dims.size() == 8 && consts.size() == 3);
  CHECK_T(y, at::kBFloat16);
  CHECK_F32(g);
  CHECK_F32(mprev);
  TORCH_CHECK(y.dim() == 2 && g.dim() == 2 && g.size(0) == y.size(0));
  MlstmChunkArgs a{};
  int* f[8] = {&a.q_off, &a.k_off, &a.v_off, &a.g_off, &a.i_off,
               &a.H, &a.dim, &a.vdim};
  for (int i = 0; i < 8; ++i) *f[i] = (int)dims[i];
  check_memory(gb, nw, S, n, m, slots, a.H, a.dim, a.vdim);
  for (const Tensor& t : {q_start, list, row0, len, ccu}) CHECK_I32(t);
  TORCH_CHECK(mlstm_chunk(a.dim, a.vdim) > 0, "sizes beyond the chunk kernels");
  const int DP = pad_dim(a.dim);
  const long N = y.size(0), chunks = row0.numel();
  a.ldy = y.size(1);
  a.ldg = g.size(1);
  auto inside = [&](int off, long n) { return off >= 0 && off + n <= a.ldy; };
  TORCH_CHECK(a.i_off >= 0 && a.i_off + 2 * a.H <= a.ldg &&
              inside(a.q_off, a.H * a.dim) && inside(a.k_off, a.H * a.dim) &&
              inside(a.v_off, a.H * a.vdim) && inside(a.g_off, a.H * a.vdim));
  TORCH_CHECK(len.numel() == chunks && ccu.numel() == list.numel() + 1 &&
              q_start.numel() == slots.numel() &&
              mprev.numel() == slots.numel() * a.H);
  CHECK_T(out, at::kBFloat16);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == N && out.size(1) >= a.H * a.vdim);
  if (chunks == 0) return;
  a.VT = (a.vdim + 15) / 16;
  auto bopt = y.options();
  auto fopt = bopt.dtype(at::kFloat);
  auto b = torch::empty({chunks, a.H, 3, MLSTM_C}, fopt);
  auto m0 = torch::empty({chunks, a.H}, fopt);
  auto n0 = torch::empty({chunks, a.H, DP}, fopt);
  auto Sb = torch::empty({chunks, a.H, a.VT, 2, DP * 16}, bopt);
  a.y = (const bf16_bits*)y.data_ptr();
  a.g = g.data_ptr<float>();
  a.gb = gb.data_ptr<float>();
  a.nw = nw.data_ptr<float>();
  a.St = S.data_ptr<float>();
  a.n = n.data_ptr<float>();
  a.m = m.data_ptr<float>();
  a.mprev = mprev.data_ptr<float>();
  a.b = b.data_ptr<float>();
  a.m0 = m0.data_ptr<float>();
  a.n0 = n0.data_ptr<float>();
  a.S = (bf16_bits*)Sb.data_ptr();
  a.out = (bf16_bits*)out.data_ptr();
  a.ldo = out.size(1);
  a.row0 = row0.data_ptr<int>();
  a.len = len.data_ptr<int>();
  a.ccu = ccu.data_ptr<int>();
  a.list = list.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.qscale = (float)consts[0];
  a.cap = (float)consts[1];
  a.eps = (float)consts[2];
  const bool vec = all_of_8({a.ldy, a.q_off, a.k_off, a.v_off, a.g_off, a.dim,
                             a.vdim, a.ldo});
  mlstm_gates_kernel<<<dim3(chunks, a.H), 64, 0, cur_stream()>>>(a);
  check_launch();
  auto go = [&](auto dp) {
    constexpr int D = decltype(dp)::value, C = MLSTM_C;
    by_bool(vec, [&](auto v) {
      constexpr bool VEC = decltype(v)::value;
      auto scan = mlstm_scan_kernel<D, VEC>;
      const size_t l2 = 2 * 2 * (C * (D == 32 ? 96 : D + 32) + 2 * C * 72);
      allow_lds(scan, l2);
      scan<<<dim3((a.vdim + 1 + 63) / 64, a.H, list.numel()), 256, l2,
             cur_stream()>>>(a);
      check_launch();
      auto fin = [&](auto nct) {
        constexpr int NCT = decltype(nct)::value;
        auto k = mlstm_out_kernel<D, NCT, VEC>;
        const size_t first = C * std::max(D + 8, NCT * 128 + 24);
        const size_t l3 = 2 * (first + C * (D + 8) + 2 * C * (C + 8));
        allow_lds(k, l3);
        k<<<dim3(chunks, a.H), 512, l3, cur_stream()>>>(a);
        check_launch();
      };
      if (a.vdim <= 128) fin(std::integral_constant<int, 1>{});
      else if (a.vdim <= 256) fin(std::integral_constant<int, 2>{});
      else fin(std::integral_constant<int, 4>{});
    });
  };
  if (DP == 32) go(std::integral_constant<int, 32>{});
  else if (DP == 64) go(std::integral_constant<int, 64>{});
  else if (DP == 128) go(std::integral_constant<int, 128>{});
  else go(std::integral_constant<int, 256>{});
}

// ---------------------------------------------------------------------------
// gated linear recurrent unit
// ---------------------------------------------------------------------------

// dims: [y_off, x_off, width, taps, blocks, stored size of a block]
static LruArgs lru_args(const Tensor& y, const std::vector<long>& dims,
                        const std::vector<Tensor>& w, const Tensor& S,
                        const Tensor& conv, const Tensor& u, const Tensor& slots,
                        const Tensor& tok_seq, const Tensor& tok_pos,
                        const Tensor& q_start, const Tensor& cu) {
  TORCH_CHECK(dims.size() == 6 && w.size() == 6);
  LruArgs a{};
  a.y = as_parts(y);
  a.N = y.size(1);
  int* f[6] = {&a.y_off, &a.x_off, &a.W, &a.K, &a.B, &a.Cp};
  for (int i = 0; i < 6; ++i) *f[i] = (int)dims[i];
  TORCH_CHECK(a.W >= 1 && a.K >= 1 && a.B >= 1 && a.W % a.B == 0);
  a.Cb = a.W / a.B;
  TORCH_CHECK(a.Cp >= a.Cb && a.y_off >= 0 && a.y_off + a.W <= a.y.ld &&
              a.x_off >= 0 && a.x_off + a.W <= a.y.ld);
  // y bias, x bias, taps, convolution bias, gate biases, decay
  const float** p[6] = {&a.yb, &a.xb, &a.taps, &a.cb, &a.gb, &a.decay};
  const long n[6] = {a.W, a.W, (long)a.K * a.W, a.W, 2L * a.W, a.W};
  for (int i = 0; i < 6; ++i) {
    CHECK_F32(w[i]);
    TORCH_CHECK(w[i].numel() == n[i]);
    *p[i] = w[i].data_ptr<float>();
  }
  CHECK_F32(S);
  CHECK_F32(conv);
  TORCH_CHECK(S.dim() == 2 && S.size(1) == a.W &&
              conv.numel() == S.size(0) * (a.K - 1) * a.W);
  a.S = S.data_ptr<float>();
  a.conv = conv.data_ptr<float>();
  check_act(u);
  TORCH_CHECK(u.is_contiguous() && u.dim() == 2 && u.size(0) == a.N &&
              u.size(1) == (long)a.B * a.Cp);
  a.u = u.data_ptr();
  for (const Tensor& t : {slots, tok_seq, tok_pos, q_start, cu}) CHECK_I32(t);
  TORCH_CHECK(tok_seq.numel() == a.N && tok_pos.numel() == a.N &&
              q_start.numel() == slots.numel() &&
              cu.numel() == slots.numel() + 1);
  a.slots = slots.data_ptr<int>();
  a.tok_seq = tok_seq.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.cu = cu.data_ptr<int>();
  return a;
}

static void lru_out(LruArgs& a, const Tensor& out, at::ScalarType t) {
  TORCH_CHECK(out.is_cuda() && out.dim() == 2 && out.size(0) == a.N &&
              out.stride(1) == 1 && out.scalar_type() == t &&
              out.size(1) >= a.W);
  a.out = out.data_ptr();
  a.ldo = out.stride(0);
}

void rglru_conv(Tensor y, std::vector<long> dims, std::vector<Tensor> w, Tensor S,
                Tensor conv, Tensor u, Tensor slots, Tensor tok_seq,
                Tensor tok_pos, Tensor q_start, Tensor cu) {
  auto a = lru_args(y, dims, w, S, conv, u, slots, tok_seq, tok_pos, q_start, cu);
  if (a.N == 0) return;
  const bool vec =
      all_of_8({a.y.ld, a.x_off, a.W, a.Cb, a.Cp}) && a.N > 32;
  by_type(y.scalar_type(), [&](auto p) {
    by_type(u.scalar_type(), [&](auto t) {
      by_bool(vec, [&](auto v) {
        constexpr int V = decltype(v)::value ? 8 : 1;
        rglru_conv_kernel<decltype(p), decltype(t), V>
            <<<dim3((a.W + 256 * V - 1) / (256 * V), a.N), 256, 0,
               cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

static void lru_gates(LruArgs& a, const Tensor& u, const Tensor& gw) {
  CHECK_T(u, at::kBFloat16);
  CHECK_T(gw, at::kBFloat16);
  TORCH_CHECK(a.Cp % 64 == 0 && gw.numel() == 2L * a.B * a.Cp * a.Cp,
              "blocks must be padded to 64");
  a.gw = gw.data_ptr();
}

// Listed one-token rows: everything after the convolution.
void rglru_step(Tensor y, std::vector<long> dims, std::vector<Tensor> w, Tensor S,
                Tensor conv, Tensor u, Tensor slots, Tensor tok_seq,
                Tensor tok_pos, Tensor q_start, Tensor cu, Tensor gw, Tensor list,
                Tensor out) {
  auto a = lru_args(y, dims, w, S, conv, u, slots, tok_seq, tok_pos, q_start, cu);
  lru_gates(a, u, gw);
  lru_out(a, out, at::kBFloat16);
  CHECK_I32(list);
  a.list = list.data_ptr<int>();
  a.n_list = list.numel();
  if (a.n_list == 0) return;
  by_type(y.scalar_type(), [&](auto p) {
    rglru_step_kernel<decltype(p)>
        <<<dim3(a.B * (a.Cp / 16), (a.n_list + 15) / 16), 64, 0,
           cur_stream()>>>(a);
  });
  check_launch();
}

long rglru_chunk() { return LRU_C; }

// Listed sequences in chunks. row0, len (chunks,); ccu (listed + 1,).
void rglru_chunks(Tensor y, std::vector<long> dims, std::vector<Tensor> w,
                  Tensor S, Tensor conv, Tensor u, Tensor slots, Tensor tok_seq,
                  Tensor tok_pos, Tensor q_start, Tensor cu, Tensor gw,
                  Tensor list, Tensor row0, Tensor len, Tensor ccu, Tensor out) {
  auto a = lru_args(y, dims, w, S, conv, u, slots, tok_seq, tok_pos, q_start, cu);
  lru_gates(a, u, gw);
  lru_out(a, out, at::kBFloat16);
  for (const Tensor& t : {list, row0, len, ccu}) CHECK_I32(t);
  const long chunks = row0.numel();
  TORCH_CHECK(len.numel() == chunks && ccu.numel() == list.numel() + 1);
  if (chunks == 0) return;
  a.list = list.data_ptr<int>();
  a.n_list = list.numel();
  a.row0 = row0.data_ptr<int>();
  a.len = len.data_ptr<int>();
  a.ccu = ccu.data_ptr<int>();
  auto fopt = u.options().dtype(at::kFloat);
  auto h = torch::empty({a.N, a.W}, fopt);
  auto F = torch::empty({a.N, a.W}, fopt);
  auto S0 = torch::empty({chunks, a.W}, fopt);
  a.h = h.data_ptr<float>();
  a.F = F.data_ptr<float>();
  a.S0 = S0.data_ptr<float>();
  const bool vec = all_of_8({a.y.ld, a.y_off, a.W, a.ldo});
  rglru_gates_kernel<<<dim3(a.B * (a.Cp / 64), chunks), 256, 0, cur_stream()>>>(a);
  check_launch();
  by_type(y.scalar_type(), [&](auto p) {
    using TP = decltype(p);
    rglru_carry_kernel<TP>
        <<<dim3((a.W + 63) / 64, a.n_list), 64, 0, cur_stream()>>>(a);
    check_launch();
    by_bool(vec, [&](auto v) {
      constexpr int V = decltype(v)::value ? 4 : 1;
      rglru_out_kernel<TP, bf16_bits, V>
          <<<dim3((a.W + 256 * V - 1) / (256 * V), LRU_C / 16, chunks), 256, 0,
             cur_stream()>>>(a);
    });
    check_launch();
  });
}

// Listed sequences token by token; z (blocks, N, 2 * width / blocks) f32 gate
// products without bias.
void rglru_seq(Tensor y, std::vector<long> dims, std::vector<Tensor> w, Tensor S,
               Tensor conv, Tensor u, Tensor slots, Tensor tok_seq,
               Tensor tok_pos, Tensor q_start, Tensor cu, Tensor z, Tensor list,
               Tensor out) {
  auto a = lru_args(y, dims, w, S, conv, u, slots, tok_seq, tok_pos, q_start, cu);
  lru_out(a, out, u.scalar_type());
  CHECK_F32(z);
  CHECK_I32(list);
  TORCH_CHECK(z.dim() == 3 && z.size(0) == a.B && z.size(1) == a.N &&
              z.size(2) == 2 * a.Cb);
  a.z = z.data_ptr<float>();
  a.list = list.data_ptr<int>();
  a.n_list = list.numel();
  if (a.n_list == 0) return;
  by_type(y.scalar_type(), [&](auto p) {
    by_type(u.scalar_type(), [&](auto t) {
      rglru_seq_kernel<decltype(p), decltype(t)>
          <<<dim3((a.W + 63) / 64, a.n_list), 64, 0, cur_stream()>>>(a);
    });
  });
  check_launch();
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("mlstm_step", &mlstm_step);
  m.def("mlstm_chunk", &mlstm_chunk);
  m.def("mlstm_chunks", &mlstm_chunks);
  m.def("rglru_conv", &rglru_conv);
  m.def("rglru_step", &rglru_step);
  m.def("rglru_chunk", &rglru_chunk);
  m.def("rglru_chunks", &rglru_chunks);
  m.def("rglru_seq", &rglru_seq);
}
