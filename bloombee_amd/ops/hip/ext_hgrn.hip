// Torch bindings of gated linear attention whose forget gate also decides what is
// written (module _hip_hgrn).
//
// Host side: shape checks, template dispatch, launch shapes.

#include "host.h"
#include "common.h"
#include "rows.hip"
#include "gla.hip"
#include "gla_host.h"

// dims: [q_off, v_off, z_off, H, dim, vdim]
template <typename Args>
static void set_dims(Args& a, const std::vector<long>& dims, double eps,
                     const Tensor& fb, const Tensor& lower, const Tensor& nw,
                     const Tensor& state, const Tensor& slots, int ldy, int ldz) {
  TORCH_CHECK(dims.size() == 6);
  int* f[6] = {&a.q_off, &a.v_off, &a.a1_off, &a.H, &a.dim, &a.vdim};
  for (int i = 0; i < 6; ++i) *f[i] = (int)dims[i];
  const long n = (long)a.H * a.dim;
  for (const Tensor& t : {fb, lower, nw, state}) CHECK_F32(t);
  CHECK_I32(slots);
  TORCH_CHECK(a.H >= 1 && a.dim >= 1 && a.vdim >= 1 && fb.numel() == n &&
              lower.numel() == n && nw.numel() == a.vdim && state.dim() == 4 &&
              state.size(1) == a.H && state.size(2) == a.dim &&
              state.size(3) == a.vdim);
  TORCH_CHECK(a.q_off >= 0 && a.q_off + n <= ldy && a.v_off >= 0 &&
              a.v_off + a.H * a.vdim <= ldy && a.a1_off >= 0 &&
              a.a1_off + n <= ldz);
  a.a2b = fb.data_ptr<float>();
  a.lower = lower.data_ptr<float>();
  a.nw = nw.data_ptr<float>();
  a.state = state.data_ptr<float>();
  a.slots = slots.data_ptr<int>();
  a.qscale = 1.f;
  a.eps = (float)eps;
}

void hgrn_step(Tensor y, Tensor z, std::vector<long> dims, double eps, Tensor fb,
               Tensor lower, Tensor nw, Tensor state, Tensor slots, Tensor tok_pos,
               Tensor cu, Tensor list, Tensor out) {
  GlaArgs a{};
  a.y = as_parts(y);
  CHECK_F32(z);
  a.a1 = as_parts(z);
  set_dims(a, dims, eps, fb, lower, nw, state, slots, a.y.ld, a.a1.ld);
  for (const Tensor& t : {tok_pos, cu, list}) CHECK_I32(t);
  const long N = y.size(1);
  TORCH_CHECK(z.size(1) == N && tok_pos.numel() == N &&
              cu.numel() == slots.numel() + 1);
  check_act(out);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == N && out.stride(1) == 1 &&
              out.size(1) >= a.H * a.vdim);
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
                                  2 * (size_t)((a.vdim + 3) & ~3));
          auto k = gla_step_kernel<decltype(p), decltype(t), V, B, true>;
          allow_lds(k, lds);
          k<<<dim3(a.H, list.numel()), B, lds, cur_stream()>>>(a);
        });
      });
    });
  });
  check_launch();
}

// Tokens of a chunk, 0 where the chunk form does not take these sizes.
long hgrn_chunk(long dim, long vdim) {
  return dim > 256 || vdim < 1 || vdim > 512 ? 0 : chunk_of(dim);
}

// Listed sequences in chunks; y (N, ldy) bf16, z (N, ldz) f32. row0, len
// (chunks,); ccu (listed + 1,).
void hgrn_chunks(Tensor y, Tensor z, std::vector<long> dims, double eps, Tensor fb,
                 Tensor lower, Tensor nw, Tensor state, Tensor slots,
                 Tensor q_start, Tensor list, Tensor row0, Tensor len, Tensor ccu,
                 Tensor out) {
  CHECK_T(y, at::kBFloat16);
  CHECK_F32(z);
  TORCH_CHECK(y.dim() == 2 && z.dim() == 2 && z.size(0) == y.size(0));
  GlaChunkArgs a{};
  a.ldy = y.size(1);
  a.ld1 = z.size(1);
  set_dims(a, dims, eps, fb, lower, nw, state, slots, a.ldy, a.ld1);
  for (const Tensor& t : {q_start, list, row0, len, ccu}) CHECK_I32(t);
  const int C = (int)hgrn_chunk(a.dim, a.vdim);
  TORCH_CHECK(C > 0, "sizes beyond the chunk kernels");
  const int DP = pad_dim(a.dim);
  const long chunks = row0.numel();
  TORCH_CHECK(len.numel() == chunks && ccu.numel() == list.numel() + 1 &&
              q_start.numel() == slots.numel());
  CHECK_T(out, at::kBFloat16);
  TORCH_CHECK(out.dim() == 2 && out.size(0) == y.size(0) &&
              out.size(1) >= a.H * a.vdim);
  if (chunks == 0) return;
  a.VT = (a.vdim + 15) / 16;
  auto bopt = y.options();
  auto b = torch::empty({chunks, a.H, C, DP}, bopt.dtype(at::kFloat));
  auto kd = torch::empty({chunks, a.H, 2, C, DP}, bopt);
  auto S = torch::empty({chunks, a.H, a.VT, 2, DP * 16}, bopt);
  a.y = (const bf16_bits*)y.data_ptr();
  a.a1 = z.data_ptr<float>();
  a.b = b.data_ptr<float>();
  a.kd = (bf16_bits*)kd.data_ptr();
  a.S = (bf16_bits*)S.data_ptr();
  a.out = (bf16_bits*)out.data_ptr();
  a.ldo = out.size(1);
  a.row0 = row0.data_ptr<int>();
  a.len = len.data_ptr<int>();
  a.ccu = ccu.data_ptr<int>();
  a.list = list.data_ptr<int>();
  a.q_start = q_start.data_ptr<int>();
  launch_chunks<true>(a, chunks, list.numel(),
                      all_of_8({a.ldy, a.ld1, a.q_off, a.v_off, a.a1_off, a.dim,
                                a.vdim, a.ldo}));
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("hgrn_step", &hgrn_step);
  m.def("hgrn_chunk", &hgrn_chunk);
  m.def("hgrn_chunks", &hgrn_chunks);
}
