// Torch bindings of latent attention and gated linear attention over ragged
// batches (module _hip_mixers).
//
// Host side: shape checks, template dispatch, launch shapes.

#include "host.h"
#include "common.h"
#include "rows.hip"
#include "latent.hip"
#include "gla.hip"
#include "gla_host.h"

static void check_turns(const OptTensor& t, long rdims) {
  TORCH_CHECK(rdims % 2 == 0 && t.has_value() && t->is_cuda() &&
                  t->is_contiguous() && t->scalar_type() == at::kDouble &&
                  t->numel() == rdims / 2,
              "rotary frequencies: one double per pair");
}

// dims: [q_off, c_off, g_off, q_rank, rank, rot, rdims, rp, gate columns,
//        has_kv]
void latent_post(Tensor y, std::vector<long> dims, double eps, double amp, Tensor qn,
                 OptTensor cn, OptTensor turns, Tensor cq, OptTensor gate,
                 Tensor kp, Tensor table, Tensor tok_seq, Tensor tok_pos) {
  TORCH_CHECK(dims.size() == 10);
  LatentPostArgs a{};
  a.y = as_parts(y);
  const long N = y.size(1);
  int* f[10] = {&a.q_off, &a.c_off, &a.g_off, &a.q_rank, &a.rank, &a.rot,
                &a.rdims, &a.rp, &a.gn, &a.has_kv};
  for (int i = 0; i < 10; ++i) *f[i] = (int)dims[i];
  a.eps = (float)eps;
  a.amp = (float)amp;
  check_act(cq);
  const auto ta = cq.scalar_type();
  CHECK_F32(qn);
  TORCH_CHECK(qn.numel() == a.q_rank && cq.dim() == 2 && cq.is_contiguous() &&
              cq.size(0) == N && cq.size(1) >= a.q_rank);
  TORCH_CHECK(a.q_off >= 0 && a.q_off + a.q_rank <= a.y.ld);
  a.qn = qn.data_ptr<float>();
  a.cq = cq.data_ptr();
  a.ldq = cq.size(1);
  CHECK_T(kp, ta);
  CHECK_I32(table);
  CHECK_I32(tok_seq);
  CHECK_I32(tok_pos);
  TORCH_CHECK(kp.dim() == 4 && kp.size(1) == 1 && table.dim() == 2 &&
              tok_seq.numel() == N && tok_pos.numel() == N);
  a.kp = kp.data_ptr();
  a.P = kp.size(2);
  a.ck = kp.size(3);
  a.table = table.data_ptr<int>();
  a.maxp = table.size(1);
  a.tok_seq = tok_seq.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  if (a.has_kv) {
    TORCH_CHECK(a.c_off >= 0 && a.c_off + a.rank + a.rot <= a.y.ld &&
                a.rank <= a.rp && a.rp + a.rot <= a.ck && a.rdims <= a.rot);
    TORCH_CHECK(cn.has_value());
    CHECK_F32((*cn));
    TORCH_CHECK(cn->numel() == a.rank);
    check_turns(turns, a.rdims);
    a.cn = cn->data_ptr<float>();
    a.turns = turns->data_ptr<double>();
  }
  if (gate.has_value()) {
    CHECK_T((*gate), ta);
    TORCH_CHECK(gate->numel() == N * a.gn && a.g_off >= 0 &&
                a.g_off + a.gn <= a.y.ld);
    a.gate = gate->data_ptr();
  } else {
    a.gn = 0;
  }
  if (N == 0) return;
  const bool vec = all_of_8({a.y.ld, a.q_off, a.q_rank, a.c_off, a.rank,
                             a.g_off, a.gn, a.ldq, a.rp, a.ck});
  const dim3 grid(N, 2 + (a.gn + 2047) / 2048);
  const size_t lds = 4 * (size_t)std::max(a.q_rank, a.rank);
  by_type(y.scalar_type(), [&](auto p) {
    by_type(ta, [&](auto t) {
      by_bool(vec, [&](auto v) {
        auto k = latent_post_kernel<decltype(p), decltype(t),
                                    decltype(v)::value ? 8 : 1>;
        allow_lds(k, lds);
        k<<<grid, 256, lds, cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

static LatentQueryArgs query_args(const Tensor& y, const OptTensor& turns,
                                  const Tensor& tok_pos, long dim, long rot,
                                  long rdims, double amp, long H) {
  LatentQueryArgs a{};
  a.y = as_parts(y);
  CHECK_I32(tok_pos);
  check_turns(turns, rdims);
  TORCH_CHECK(tok_pos.numel() == y.size(1) && rdims <= rot &&
              H * (dim + rot) <= a.y.ld);
  a.turns = turns->data_ptr<double>();
  a.tok_pos = tok_pos.data_ptr<int>();
  a.H = (int)H;
  a.dim = (int)dim;
  a.rot = (int)rot;
  a.rdims = (int)rdims;
  a.amp = (float)amp;
  return a;
}

// q (N, H, ld) from the query GEMM
void latent_rope(Tensor y, OptTensor turns, Tensor tok_pos, long dim, long rot,
                 long rdims, double amp, Tensor q) {
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && q.size(0) == y.size(1) &&
              q.size(2) >= dim + rot);
  check_act(q);
  auto a = query_args(y, turns, tok_pos, dim, rot, rdims, amp, q.size(1));
  a.q = q.data_ptr();
  a.ldq = q.size(2);
  if (q.size(0) == 0) return;
  const bool vec = all_of_8({a.y.ld, dim, rot, a.ldq});
  by_type(y.scalar_type(), [&](auto p) {
    by_type(q.scalar_type(), [&](auto t) {
      by_bool(vec, [&](auto v) {
        latent_rope_kernel<decltype(p), decltype(t), decltype(v)::value ? 8 : 1>
            <<<q.size(0), 256, 4 * rdims, cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

// Latents of a context in pages -> per-head keys and values in pages.
void latent_scatter(Tensor y, Tensor ctx, Tensor valid, long dim, long rot,
                    long vdim, long rp, Tensor k, Tensor v) {
  for (const Tensor& t : {y, ctx, k, v}) CHECK_T(t, at::kBFloat16);
  CHECK_I32(valid);
  TORCH_CHECK(y.dim() == 2 && ctx.dim() == 3 && k.dim() == 4 && v.dim() == 4);
  LatentScatterArgs a{};
  const long npg = ctx.size(0);
  a.P = ctx.size(1);
  a.ck = ctx.size(2);
  a.H = k.size(1);
  a.dkp = k.size(3);
  a.dvp = v.size(2);
  a.ldy = y.size(1);
  a.dim = (int)dim;
  a.rot = (int)rot;
  a.vdim = (int)vdim;
  a.rp = (int)rp;
  TORCH_CHECK(y.size(0) == npg * a.P && k.size(0) == npg && v.size(0) == npg &&
              k.size(2) == a.P && v.size(3) == a.P && v.size(1) == a.H &&
              valid.numel() == npg && a.P % 8 == 0);
  TORCH_CHECK(a.dkp >= dim + rot && a.dvp >= vdim && rp + rot <= a.ck &&
              a.H * (dim + vdim) <= a.ldy);
  a.y = (const bf16_bits*)y.data_ptr();
  a.ctx = (const bf16_bits*)ctx.data_ptr();
  a.valid = valid.data_ptr<int>();
  a.k = (bf16_bits*)k.data_ptr();
  a.v = (bf16_bits*)v.data_ptr();
  if (npg == 0) return;
  by_bool(all_of_8({a.ldy, dim, vdim, a.dkp, a.dvp}), [&](auto vec) {
    latent_scatter_kernel<decltype(vec)::value ? 8 : 1>
        <<<dim3(npg, a.H), 256, 0, cur_stream()>>>(a);
  });
  check_launch();
}

template <int ND, int NR>
static void launch_decode(LatentDecodeArgs& a, long n) {
  constexpr int CK = ND * 64 + NR * 32;
  by_bool(a.H > 16, [&](auto two) {
    constexpr int HG = decltype(two)::value ? 2 : 1;
    constexpr size_t lds = 64 * latent_tile_ld(CK) * 2 + HG * 16 * 68 * 4;
    auto k = attn_latent_decode_kernel<ND, NR, HG>;
    allow_lds(k, lds);
    const long units = n * ((a.H + 16 * HG - 1) / (16 * HG));
    k<<<dim3(units, a.n_split), 256 * HG, lds, cur_stream()>>>(a);
  });
  check_launch();
}

// Sizes the decode kernel is compiled for.
bool latent_decode_fits(long rp, long rtp) {
  return (rp == 64 || rp == 128 || rp == 256 || rp == 512) &&
         (rtp == 32 || rtp == 64 || rtp == 128);
}

// Listed one-token rows: query GEMM output y -> gated attention in out.
void latent_decode(Tensor y, OptTensor turns, Tensor kp, Tensor table,
                   Tensor tok_pos, Tensor cu, Tensor q_start, Tensor dec,
                   long max_ctx, long dim, long rot, long rdims, double amp,
                   long vdim, double scale,
                   long window, Tensor wk, Tensor wv, OptTensor sinks,
                   OptTensor gate, Tensor out) {
  for (const Tensor& t : {kp, wk, wv}) CHECK_T(t, at::kBFloat16);
  for (const Tensor& t : {table, cu, q_start, dec}) CHECK_I32(t);
  TORCH_CHECK(kp.dim() == 4 && kp.size(1) == 1 && wk.dim() == 3 &&
              wv.dim() == 3 && table.dim() == 2 &&
              cu.numel() == table.size(0) + 1 &&
              q_start.numel() == table.size(0));
  const long H = wk.size(0), rp = wk.size(1), ck = kp.size(3);
  TORCH_CHECK(latent_decode_fits(rp, ck - rp) && rot <= ck - rp);
  TORCH_CHECK(wk.size(2) % 32 == 0 && wk.size(2) >= dim && wv.size(0) == H &&
              wv.size(1) % 64 == 0 && wv.size(1) >= vdim && wv.size(2) == rp);
  TORCH_CHECK(out.is_cuda() && out.dim() == 2 && out.size(0) == y.size(1) &&
              out.stride(1) == 1 && out.scalar_type() == at::kBFloat16 &&
              out.size(1) >= H * vdim);
  const long n = dec.numel();
  if (n == 0) return;
  auto qa = query_args(y, turns, tok_pos, dim, rot, rdims, amp, H);
  auto bopt = kp.options();
  auto fopt = bopt.dtype(at::kFloat);
  auto q = torch::empty({n, H, ck}, bopt);
  qa.cu = cu.data_ptr<int>();
  qa.list = dec.data_ptr<int>();
  qa.wk = wk.data_ptr();
  qa.q = q.data_ptr();
  qa.n_list = (int)n;
  qa.rp = (int)rp;
  qa.ck = (int)ck;
  qa.dimp = wk.size(2);
  {
    const size_t lds = 32 * (qa.dimp + 8) * 2;
    by_type(y.scalar_type(), [&](auto p) {
      by_bool(all_of_8({qa.y.ld, dim, rot}), [&](auto v) {
        auto k = latent_absorb_kernel<decltype(p), decltype(v)::value ? 8 : 1>;
        allow_lds(k, lds);
        k<<<dim3((rp + 127) / 128 + 1, H, (n + 31) / 32), 256, lds,
            cur_stream()>>>(qa);
      });
    });
    check_launch();
  }

  LatentDecodeArgs a{};
  a.q = (const bf16_bits*)q.data_ptr();
  a.kp = (const bf16_bits*)kp.data_ptr();
  a.table = table.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.list = qa.list;
  a.H = (int)H;
  const int P = kp.size(2);
  TORCH_CHECK((P & (P - 1)) == 0, "page size must be a power of two");
  while (1 << a.p_log2 < P) ++a.p_log2;
  a.maxp = table.size(1);
  a.window = (int)window;
  a.scale = (float)scale;
  // a workgroup a CU, two tiles of 64 keys each at least
  const long units = n * (H > 16 ? (H + 31) / 32 : 1);
  const long seen = window > 0 ? std::min<long>(window, max_ctx) : max_ctx;
  const long tiles = (seen + 63) / 64 + 1;
  const long fill = (H > 16 ? 256 : 512) / std::max<long>(1, units);
  a.n_split = (int)std::max<long>(1, std::min<long>({16, fill, tiles / 2}));
  auto pml = torch::empty({n, H, a.n_split, 2}, fopt);
  auto pacc = torch::empty({n, H, a.n_split, rp}, fopt);
  auto olat = torch::empty({n, H, rp}, bopt);
  a.pml = pml.data_ptr<float>();
  a.pacc = pacc.data_ptr<float>();
  auto by_rot = [&](auto nd) {
    constexpr int ND = decltype(nd)::value;
    if (ck - rp == 32) launch_decode<ND, 1>(a, n);
    else if (ck - rp == 64) launch_decode<ND, 2>(a, n);
    else launch_decode<ND, 4>(a, n);
  };
  if (rp == 64) by_rot(std::integral_constant<int, 1>{});
  else if (rp == 128) by_rot(std::integral_constant<int, 2>{});
  else if (rp == 256) by_rot(std::integral_constant<int, 4>{});
  else by_rot(std::integral_constant<int, 8>{});

  const float* sp = nullptr;
  if (sinks.has_value()) {
    CHECK_F32((*sinks));
    TORCH_CHECK(sinks->numel() == H);
    sp = sinks->data_ptr<float>();
  }
  LatentOutputArgs o{};
  o.o = (const bf16_bits*)olat.data_ptr();
  by_bool(a.n_split > 4, [&](auto many) {
    latent_combine_kernel<decltype(many)::value ? 16 : 4>
        <<<n * H, 128, 0, cur_stream()>>>(a.pml, a.pacc, sp,
                                          (bf16_bits*)olat.data_ptr(), (int)n,
                                          (int)H, (int)rp, a.n_split);
  });
  check_launch();
  if (gate.has_value()) {
    TORCH_CHECK(gate->is_cuda() && gate->dim() == 2 &&
                gate->size(0) == out.size(0) && gate->stride(1) == 1 &&
                gate->scalar_type() == at::kBFloat16 &&
                gate->size(1) >= H * vdim);
    o.gate = (const bf16_bits*)gate->data_ptr();
    o.ldg = gate->stride(0);
  }
  o.wv = (const bf16_bits*)wv.data_ptr();
  o.out = (bf16_bits*)out.data_ptr();
  o.ldo = out.stride(0);
  o.cu = qa.cu;
  o.list = qa.list;
  o.n_list = (int)n;
  o.H = (int)H;
  o.rp = (int)rp;
  o.vdim = (int)vdim;
  o.vp = wv.size(1);
  latent_output_kernel<<<dim3(o.vp / 64, H, (n + 15) / 16), 256, 0,
                         cur_stream()>>>(o);
  check_launch();
}

// ---------------------------------------------------------------------------

static void check_gla(const Tensor& a2, const Tensor& a2b, const Tensor& nw,
                      const Tensor& state, const Tensor& slots, long H,
                      long dim, long vdim) {
  CHECK_F32(a2);
  CHECK_F32(a2b);
  CHECK_F32(nw);
  CHECK_F32(state);
  CHECK_I32(slots);
  TORCH_CHECK(a2.dim() == 2 && a2.size(1) == H * dim && a2b.numel() == H * dim &&
              nw.numel() == vdim && state.dim() == 4 && state.size(1) == H &&
              state.size(2) == dim && state.size(3) == vdim);
}

// dims: [q_off, k_off, v_off, g_off, a1_off, H, dim, vdim];
// consts: [query scale, 1 / tau, eps]
void gla_step(Tensor y, Tensor a1, std::vector<long> dims,
              std::vector<double> consts, Tensor a2, Tensor a2b, Tensor nw,
              Tensor state, Tensor slots, Tensor tok_pos, Tensor cu,
              Tensor list, Tensor out) {
  TORCH_CHECK(dims.size() == 8 && consts.size() == 3);
  GlaArgs a{};
  a.y = as_parts(y);
  CHECK_F32(a1);
  a.a1 = as_parts(a1);
  int* f[8] = {&a.q_off, &a.k_off, &a.v_off, &a.g_off, &a.a1_off,
               &a.H, &a.dim, &a.vdim};
  for (int i = 0; i < 8; ++i) *f[i] = (int)dims[i];
  check_gla(a2, a2b, nw, state, slots, a.H, a.dim, a.vdim);
  for (const Tensor& t : {tok_pos, cu, list}) CHECK_I32(t);
  a.r = a2.size(0);
  const long N = y.size(1);
  auto inside = [&](int off, long n) { return off >= 0 && off + n <= a.y.ld; };
  TORCH_CHECK(a1.size(1) == N && a.a1_off >= 0 && a.a1_off + a.r <= a.a1.ld &&
              inside(a.q_off, a.H * a.dim) && inside(a.k_off, a.H * a.dim) &&
              inside(a.v_off, a.H * a.vdim) && inside(a.g_off, a.H * a.vdim));
  TORCH_CHECK(tok_pos.numel() == N && cu.numel() == slots.numel() + 1);
  check_act(out);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == N && out.stride(1) == 1 &&
              out.size(1) >= a.H * a.vdim);
  a.qscale = (float)consts[0];
  a.inv_tau = (float)consts[1];
  a.eps = (float)consts[2];
  a.a2 = a2.data_ptr<float>();
  a.a2b = a2b.data_ptr<float>();
  a.nw = nw.data_ptr<float>();
  a.state = state.data_ptr<float>();
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
          const size_t lds = 4 * (((3 * a.dim + 3) & ~3) + B * V +
                                  2 * ((a.vdim + 3) & ~3) + (size_t)a.r);
          auto k = gla_step_kernel<decltype(p), decltype(t), V, B>;
          allow_lds(k, lds);
          k<<<dim3(a.H, list.numel()), B, lds, cur_stream()>>>(a);
        });
      });
    });
  });
  check_launch();
}

// Tokens of a chunk, 0 where the chunk form does not take these sizes.
long gla_chunk(long dim, long vdim, long r) {
  if (dim > 256 || vdim < 1 || vdim > 512) return 0;
  const int C = chunk_of(dim);
  return prep_lds(pad_dim(dim), C, r) <= 150 * 1024 ? C : 0;
}

// Listed sequences in chunks; y (N, ldy) bf16, a1 (N, ld1) f32; dims, consts as
// gla_step. row0, len (chunks,); ccu (listed + 1,).
void gla_chunks(Tensor y, Tensor a1, std::vector<long> dims,
                std::vector<double> consts, Tensor a2, Tensor a2b, Tensor nw,
                Tensor state, Tensor slots, Tensor q_start, Tensor list,
                Tensor row0, Tensor len, Tensor ccu, Tensor out) {
  TORCH_CHECK(dims.size() == 8 && consts.size() == 3);
  CHECK_T(y, at::kBFloat16);
  CHECK_F32(a1);
  TORCH_CHECK(y.dim() == 2 && a1.dim() == 2 && a1.size(0) == y.size(0));
  GlaChunkArgs a{};
  int* f[8] = {&a.q_off, &a.k_off, &a.v_off, &a.g_off, &a.a1_off,
               &a.H, &a.dim, &a.vdim};
  for (int i = 0; i < 8; ++i) *f[i] = (int)dims[i];
  check_gla(a2, a2b, nw, state, slots, a.H, a.dim, a.vdim);
  for (const Tensor& t : {q_start, list, row0, len, ccu}) CHECK_I32(t);
  a.r = a2.size(0);
  const int C = (int)gla_chunk(a.dim, a.vdim, a.r);
  TORCH_CHECK(C > 0, "sizes beyond the chunk kernels");
  const int DP = pad_dim(a.dim);
  const long N = y.size(0), chunks = row0.numel();
  a.ldy = y.size(1);
  a.ld1 = a1.size(1);
  auto inside = [&](int off, long n) { return off >= 0 && off + n <= a.ldy; };
  TORCH_CHECK(a.a1_off >= 0 && a.a1_off + a.r <= a.ld1 &&
              inside(a.q_off, a.H * a.dim) && inside(a.k_off, a.H * a.dim) &&
              inside(a.v_off, a.H * a.vdim) && inside(a.g_off, a.H * a.vdim));
  TORCH_CHECK(len.numel() == chunks && ccu.numel() == list.numel() + 1 &&
              q_start.numel() == slots.numel());
  CHECK_T(out, at::kBFloat16);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == N && out.size(1) >= a.H * a.vdim);
  if (chunks == 0) return;
  a.VT = (a.vdim + 15) / 16;
  auto bopt = y.options();
  auto b = torch::empty({chunks, a.H, C, DP}, bopt.dtype(at::kFloat));
  auto kd = torch::empty({chunks, a.H, 2, C, DP}, bopt);
  auto S = torch::empty({chunks, a.H, a.VT, 2, DP * 16}, bopt);
  a.y = (const bf16_bits*)y.data_ptr();
  a.a1 = a1.data_ptr<float>();
  a.a2 = a2.data_ptr<float>();
  a.a2b = a2b.data_ptr<float>();
  a.nw = nw.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.b = b.data_ptr<float>();
  a.kd = (bf16_bits*)kd.data_ptr();
  a.S = (bf16_bits*)S.data_ptr();
  a.out = (bf16_bits*)out.data_ptr();
  a.ldo = out.size(1);
  a.row0 = row0.data_ptr<int>();
  a.len = len.data_ptr<int>();
  a.ccu = ccu.data_ptr<int>();
  a.list = list.data_ptr<int>();
  a.slots = slots.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  a.qscale = (float)consts[0];
  a.inv_tau = (float)consts[1];
  a.eps = (float)consts[2];
  const bool vec = all_of_8({a.ldy, a.q_off, a.k_off, a.v_off, a.g_off, a.dim,
                             a.vdim, a.ldo});
  launch_chunks<false>(a, chunks, list.numel(), vec);
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_post", &latent_post);
  m.def("latent_rope", &latent_rope);
  m.def("latent_scatter", &latent_scatter);
  m.def("latent_decode_fits", &latent_decode_fits);
  m.def("latent_decode", &latent_decode);
  m.def("gla_step", &gla_step);
  m.def("gla_chunk", &gla_chunk);
  m.def("gla_chunks", &gla_chunks);
}
