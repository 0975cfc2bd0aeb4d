// Torch bindings of the ragged-batch kernels (module _hip_ragged): attention
// over mixed batches, row-wise fused steps, routed experts, and the split-K
// decode GEMM that hands its f32 partials to the fused consumer. A module of
// its own, so that a model that needs only these compiles only these.
//
// Host side: shape checks, template dispatch, launch shapes.

#include "host.h"
#include "common.h"
#include "rows.hip"
#include "attn_ragged.hip"
#include "moe_routed.hip"
#include "gemm_skinny.hip"

// pair: [buckets, mul_prev, mul_cur] with prev and pair_table
Tensor embed_rows(Tensor ids, Tensor pos, Tensor table, OptTensor pos_table,
                  OptTensor prev, OptTensor pair_table, std::vector<long> pair,
                  OptTensor turns, double scale, long copies) {
  CHECK_I32(ids);
  CHECK_I32(pos);
  check_act(table);
  TORCH_CHECK(table.is_contiguous() && table.dim() == 2 &&
              ids.numel() == pos.numel());
  EmbedArgs a{};
  const long N = ids.numel();
  a.W = table.size(1);
  a.vocab = table.size(0);
  a.ids = ids.data_ptr<int>();
  a.pos = pos.data_ptr<int>();
  a.table = table.data_ptr();
  if (pos_table.has_value()) {
    CHECK_T((*pos_table), table.scalar_type());
    TORCH_CHECK(pos_table->dim() == 2 && a.W == pos_table->size(1));
    a.pos_table = pos_table->data_ptr();
    a.max_pos = pos_table->size(0);
  }
  if (pair_table.has_value()) {
    CHECK_T((*pair_table), table.scalar_type());
    TORCH_CHECK(prev.has_value(), "rows of token pairs need the previous tokens");
    CHECK_I32((*prev));
    TORCH_CHECK(pair.size() == 3 && pair[0] >= 1 && pair[1] >= 0 && pair[2] >= 0 &&
                pair_table->dim() == 2 && pair_table->size(0) == pair[0] + 1 &&
                pair_table->size(1) == a.W && prev->numel() == N);
    a.pair_table = pair_table->data_ptr();
    a.prev = prev->data_ptr<int>();
    a.buckets = pair[0];
    a.mul_prev = pair[1];
    a.mul_cur = pair[2];
  }
  if (turns.has_value()) {
    CHECK_T((*turns), at::kDouble);
    TORCH_CHECK(turns->numel() == (a.W + 1) / 2);
    a.turns = turns->data_ptr<double>();
  }
  TORCH_CHECK(copies >= 1);
  a.scale = (float)scale;
  a.copies = (int)copies;
  auto x = torch::empty({N, copies * a.W}, table.options().dtype(at::kFloat));
  if (N == 0) return x;
  a.x = x.data_ptr<float>();
  by_type(table.scalar_type(), [&](auto t) {
    embed_rows_kernel<decltype(t)><<<N, 256, 0, cur_stream()>>>(a);
  });
  check_launch();
  return x;
}

// ---------------------------------------------------------------------------
// residual fold + grouped norm
// ---------------------------------------------------------------------------

void residual_norm(Tensor x, OptTensor parts, OptTensor routed, OptTensor ids,
                   OptTensor idw, OptTensor hprev, OptTensor nw, long groups,
                   double eps, OptTensor h, double alpha, OptTensor bias,
                   bool post, OptTensor bw, OptTensor other) {
  // rows may lie apart (columns of a wider matrix)
  auto rows_f32 = [](const Tensor& t) {
    TORCH_CHECK(t.is_cuda() && t.dim() == 2 && t.scalar_type() == at::kFloat &&
                    (t.stride(1) == 1 || t.size(1) == 1) && t.stride(0) >= t.size(1),
                "f32 rows on the device");
  };
  rows_f32(x);
  const long N = x.size(0);
  const int W = x.size(1);
  ResidualArgs a{};
  a.x = x.data_ptr<float>();
  a.ldx = x.stride(0);
  a.W = W;
  a.eps = (float)eps;
  a.groups = (int)groups;
  a.alpha = (float)alpha;
  a.post = post;
  TORCH_CHECK(!post || nw.has_value(), "a norm after the sum needs its weight");
  if (bias.has_value()) {
    CHECK_F32((*bias));
    TORCH_CHECK(parts.has_value() && bias->numel() == W);
    a.bias = bias->data_ptr<float>();
  }
  if (bw.has_value()) {
    CHECK_F32((*bw));
    TORCH_CHECK(bw->numel() == W && (parts.has_value() || routed.has_value()));
    a.bw = bw->data_ptr<float>();
  }
  auto aligned = [](const Tensor& t) {
    return t.stride(0) % 4 == 0 && (size_t)t.data_ptr() % 16 == 0;
  };
  bool vec = W % 4 == 0 && aligned(x);
  at::ScalarType tp = at::kFloat, ta = at::kFloat;
  if (parts.has_value()) {
    check_act(*parts);
    TORCH_CHECK(parts->is_contiguous() && parts->dim() == 3 &&
                parts->size(1) == N && parts->size(2) >= W);
    tp = parts->scalar_type();
    a.parts = parts->data_ptr();
    a.ks = parts->size(0);
    a.ldp = parts->size(2);
    a.pstride = (long)N * a.ldp;
    vec = vec && a.ldp % 4 == 0;
  }
  if (routed.has_value()) {
    TORCH_CHECK(ids.has_value());
    check_act(*routed);
    CHECK_I32((*ids));
    TORCH_CHECK(routed->is_contiguous() && routed->dim() == 3 &&
                routed->size(0) == N && routed->size(2) >= W);
    a.routed = routed->data_ptr();
    a.top = routed->size(1);
    a.ldr = routed->size(2);
    TORCH_CHECK(ids->numel() == N * a.top);
    a.ids = ids->data_ptr<int>();
    ta = routed->scalar_type();
    vec = vec && a.ldr % 4 == 0;
  }
  if (idw.has_value()) {
    TORCH_CHECK(parts.has_value() && hprev.has_value());
    CHECK_F32((*idw));
    check_act(*hprev);
    TORCH_CHECK(idw->numel() == N && hprev->is_contiguous() &&
                hprev->size(0) == N && hprev->size(1) >= W);
    a.idw = idw->data_ptr<float>();
    a.hprev = hprev->data_ptr();
    a.ldhp = hprev->size(1);
    TORCH_CHECK(!routed.has_value() || hprev->scalar_type() == ta);
    ta = hprev->scalar_type();
    vec = vec && a.ldhp % 4 == 0;
  }
  if (nw.has_value()) {
    CHECK_F32((*nw));
    TORCH_CHECK(h.has_value() && nw->numel() == W && groups >= 1 &&
                W % groups == 0);
    check_act(*h);
    TORCH_CHECK(h->is_contiguous() && h->size(0) == N && h->size(1) >= W);
    TORCH_CHECK(!(routed.has_value() || idw.has_value()) ||
                h->scalar_type() == ta, "one activation type per call");
    ta = h->scalar_type();
    a.nw = nw->data_ptr<float>();
    a.h = h->data_ptr();
    a.ldh = h->size(1);
    vec = vec && a.ldh % 4 == 0;
  }
  if (other.has_value()) {
    rows_f32(*other);
    TORCH_CHECK(!nw.has_value() && h.has_value() && other->size(0) == N &&
                other->size(1) == W);
    check_act(*h);
    TORCH_CHECK(h->is_contiguous() && h->size(0) == N && h->size(1) >= 2 * W);
    TORCH_CHECK(!(routed.has_value() || idw.has_value()) ||
                h->scalar_type() == ta, "one activation type per call");
    ta = h->scalar_type();
    a.other = other->data_ptr<float>();
    a.ldx2 = other->stride(0);
    a.h = h->data_ptr();
    a.ldh = h->size(1);
    vec = vec && a.ldh % 4 == 0 && aligned(*other);
  }
  if (N == 0) return;
  const size_t lds = 4 * (((W + 3) & ~3) + (size_t)a.groups + 32);
  by_type(tp, [&](auto p) {
    by_type(ta, [&](auto t) {
      by_bool(vec, [&](auto v) {
        constexpr int V = decltype(v)::value ? 4 : 1;
        auto go = [&](auto blk) {
          auto k = residual_norm_kernel<decltype(p), decltype(t), V,
                                        decltype(blk)::value>;
          allow_lds(k, lds);
          k<<<N, decltype(blk)::value, lds, cur_stream()>>>(a);
        };
        // few rows: more waves on each; many: more rows at a time
        if (W > 2048 && N <= 256) go(std::integral_constant<int, 1024>{});
        else go(std::integral_constant<int, 256>{});
      });
    });
  });
  check_launch();
}

// [gate | up] GEMM output -> clamped gated product, (N, ldo).
void clamped_glu(Tensor parts, long g_off, long u_off, long ff, OptTensor gb,
                 OptTensor ub, double limit, double slope, Tensor out) {
  check_act(parts);
  check_act(out);
  TORCH_CHECK(parts.dim() == 3 && parts.is_contiguous() && out.dim() == 2 &&
              out.is_contiguous() && out.size(0) == parts.size(1) &&
              out.size(1) >= ff && ff >= 1);
  GluArgs a{};
  const long N = parts.size(1);
  a.N = N;
  a.parts = parts.data_ptr();
  a.ks = parts.size(0);
  a.ldp = parts.size(2);
  a.pstride = N * (long)a.ldp;
  a.g_off = (int)g_off;
  a.u_off = (int)u_off;
  a.ff = (int)ff;
  a.out = out.data_ptr();
  a.ldo = out.size(1);
  a.limit = (float)limit;
  a.slope = (float)slope;
  TORCH_CHECK(g_off >= 0 && u_off >= 0 && g_off + ff <= a.ldp &&
              u_off + ff <= a.ldp);
  for (const OptTensor* b : {&gb, &ub})
    if (b->has_value()) {
      CHECK_F32((**b));
      TORCH_CHECK((*b)->numel() == ff);
    }
  if (gb.has_value()) a.gb = gb->data_ptr<float>();
  if (ub.has_value()) a.ub = ub->data_ptr<float>();
  if (N == 0) return;
  bool vec = true;
  for (int v : {a.ldp, a.g_off, a.u_off, a.ff, a.ldo}) vec = vec && v % 8 == 0;
  by_type(parts.scalar_type(), [&](auto p) {
    by_type(out.scalar_type(), [&](auto t) {
      by_bool(vec, [&](auto v) {
        by_bool(N > 256, [&](auto many) {
          constexpr int V = decltype(v)::value ? 8 : 1;
          constexpr int R = decltype(many)::value ? 4 : 1;
          clamped_glu_kernel<decltype(p), decltype(t), V, R>
              <<<dim3((a.ldo + 256 * V - 1) / (256 * V), (N + R - 1) / R), 256,
                 0, cur_stream()>>>(a);
        });
      });
    });
  });
  check_launch();
}

void softcap(Tensor z, double cap) {
  CHECK_F32(z);
  TORCH_CHECK(cap > 0);
  const long n = z.numel();
  if (n == 0) return;
  softcap_kernel<<<std::min<long>((n + 255) / 256, 2048), 256, 0,
                   cur_stream()>>>(z.data_ptr<float>(), n, (float)cap);
  check_launch();
}

// ---------------------------------------------------------------------------
// input GEMM -> q, K/V pages, gate, activation, routing
// ---------------------------------------------------------------------------

static void set_logits(RouteArgs& r, const Tensor& rparts, long N) {
  CHECK_F32(rparts);
  TORCH_CHECK(rparts.dim() == 3 && rparts.size(1) == N);
  r.parts = rparts.data_ptr<float>();
  r.ks = rparts.size(0);
  r.ld = rparts.size(2);
  r.stride = N * (long)r.ld;
}

static void set_routing(RouteArgs& r, long N, const OptTensor& corr, Tensor ids,
                        Tensor wts, const OptTensor& idw) {
  const int n = r.E + r.NI;
  TORCH_CHECK(n <= MAX_ROUTED && r.top >= 1 && r.top <= n);
  TORCH_CHECK(r.off >= 0 && r.off + n <= r.ld);
  CHECK_I32(ids);
  CHECK_F32(wts);
  TORCH_CHECK(ids.numel() == N * r.top && wts.numel() == N * r.top);
  r.ids = ids.data_ptr<int>();
  r.wts = wts.data_ptr<float>();
  if (corr.has_value()) {
    CHECK_F32((*corr));
    TORCH_CHECK(corr->numel() == n);
    r.corr = corr->data_ptr<float>();
  }
  TORCH_CHECK(r.NI == 0 || idw.has_value());
  if (idw.has_value()) {
    CHECK_F32((*idw));
    TORCH_CHECK(idw->numel() == N);
    r.idw = idw->data_ptr<float>();
  }
}

// dims: [q,k,v,g,u,u2,r,sg offsets, H, G, dim, vdim, has_kv, act, ff, act_col,
//        E, NI, top]; consts: [eps, xp, xq, rscale]
void proj_post(Tensor parts, OptTensor rparts, std::vector<long> dims,
               std::vector<double> consts, Tensor qn, OptTensor kn,
               OptTensor corr, Tensor q, OptTensor gate, Tensor a2, Tensor kp,
               Tensor vp, Tensor table, Tensor tok_seq, Tensor tok_pos,
               OptTensor ids, OptTensor wts, OptTensor idw) {
  check_act(parts);
  check_act(q);
  TORCH_CHECK(parts.dim() == 3 && parts.is_contiguous());
  TORCH_CHECK(dims.size() == 19 && consts.size() == 4);
  PostArgs a{};
  const long N = parts.size(1);
  a.parts = parts.data_ptr();
  a.ks = parts.size(0);
  a.ldp = parts.size(2);
  a.pstride = N * (long)a.ldp;
  int* f[19] = {&a.q_off, &a.k_off, &a.v_off, &a.g_off, &a.u_off, &a.u2_off,
                &a.rt.off, &a.sg_off, &a.H, &a.G, &a.dim, &a.vdim, &a.has_kv,
                &a.act, &a.ff, &a.act_col, &a.rt.E, &a.rt.NI, &a.rt.top};
  for (int i = 0; i < 19; ++i) *f[i] = (int)dims[i];
  a.eps = (float)consts[0];
  a.xp = (float)consts[1];
  a.xq = (float)consts[2];
  a.rt.scale = (float)consts[3];
  const auto ta = q.scalar_type();
  for (const Tensor& t : {q, a2, kp, vp})
    TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == ta,
                "q, a2 and the pages share one element type");
  TORCH_CHECK(q.dim() == 3 && q.size(0) == N && q.size(1) == a.H &&
              q.size(2) >= a.dim);
  a.q = q.data_ptr();
  a.dkp = q.size(2);
  TORCH_CHECK(a2.size(0) == N && a2.size(1) >= a.H * a.vdim);
  a.a2 = a2.data_ptr();
  a.lda2 = a2.size(1);
  TORCH_CHECK(kp.dim() == 4 && vp.dim() == 4 && kp.size(1) == a.G &&
              vp.size(1) == a.G && kp.size(3) == a.dkp &&
              vp.size(3) == kp.size(2) && vp.size(2) >= a.vdim &&
              vp.size(0) == kp.size(0));
  a.kp = kp.data_ptr();
  a.vp = vp.data_ptr();
  a.P = kp.size(2);
  a.dvp = vp.size(2);
  CHECK_I32(table);
  CHECK_I32(tok_seq);
  CHECK_I32(tok_pos);
  TORCH_CHECK(tok_seq.numel() == N && tok_pos.numel() == N && table.dim() == 2);
  a.table = table.data_ptr<int>();
  a.maxp = table.size(1);
  a.tok_seq = tok_seq.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  const int HV = a.H * a.vdim;
  auto inside = [&](int off, int n) { return off >= 0 && off + n <= a.ldp; };
  TORCH_CHECK(inside(a.q_off, a.H * a.dim) && inside(a.g_off, HV));
  CHECK_F32(qn);
  TORCH_CHECK(qn.numel() == a.H * a.dim);
  a.qn = qn.data_ptr<float>();
  if (a.has_kv) {
    TORCH_CHECK(kn.has_value() && inside(a.k_off, a.G * a.dim) &&
                inside(a.v_off, a.G * a.vdim));
    CHECK_F32((*kn));
    TORCH_CHECK(kn->numel() == a.G * a.dim);
    a.kn = kn->data_ptr<float>();
  }
  if (gate.has_value()) {
    TORCH_CHECK(gate->is_cuda() && gate->is_contiguous() &&
                gate->scalar_type() == ta && gate->numel() == N * (long)HV);
    a.gate = gate->data_ptr();
  }
  if (a.act) {
    TORCH_CHECK(inside(a.u_off, a.ff) && a.act_col >= HV &&
                a.act_col + a.ff <= a.lda2);
    TORCH_CHECK(a.act != 2 || inside(a.u2_off, a.ff));
  } else {
    a.act_col = HV;
    a.ff = 0;
  }
  const int routed = a.rt.E + a.rt.NI;
  if (routed > 0 || a.act == 2) {
    TORCH_CHECK(rparts.has_value());
    set_logits(a.rt, *rparts, N);
    TORCH_CHECK(a.act != 2 || (a.sg_off >= 0 && a.sg_off < a.rt.ld));
  }
  if (routed > 0) {
    TORCH_CHECK(corr.has_value() && ids.has_value() && wts.has_value() &&
                idw.has_value());
    set_routing(a.rt, N, corr, *ids, *wts, idw);
  }
  if (N == 0) return;
  bool vec = true;
  for (int v : {a.ldp, a.q_off, a.k_off, a.g_off, a.u_off, a.u2_off, a.dim,
                a.vdim, a.ff, a.act_col, a.lda2})
    vec = vec && (v < 0 || v % 8 == 0);  // -1: no such section
  const int cols = (a.gate ? HV : 0) + a.lda2 - HV;
  const dim3 grid(N, 3 + (cols + POST_CHUNK - 1) / POST_CHUNK);
  const size_t lds = 4 * (size_t)std::max({a.H * a.dim, a.G * a.dim,
                                           2 * MAX_ROUTED});
  by_type(parts.scalar_type(), [&](auto p) {
    by_type(ta, [&](auto t) {
      by_bool(vec, [&](auto v) {
        auto k = proj_post_kernel<decltype(p), decltype(t),
                                  decltype(v)::value ? 8 : 1>;
        allow_lds(k, lds);
        k<<<grid, POST_BLOCK, lds, cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

// dims: [q,k,v offsets, H, G, dim, vdim]; consts: [eps, temperature's
// coefficient and step]
void head_post(Tensor parts, std::vector<long> dims, std::vector<double> consts,
               OptTensor qb, OptTensor kb, OptTensor vb, Tensor qn, Tensor kn,
               Tensor q, Tensor kp, Tensor vp, Tensor table, Tensor tok_seq,
               Tensor tok_pos) {
  TORCH_CHECK(dims.size() == 7 && consts.size() == 3);
  HeadPostArgs a{};
  a.y = as_parts(parts);
  const long N = parts.size(1);
  int* f[7] = {&a.q_off, &a.k_off, &a.v_off, &a.H, &a.G, &a.dim, &a.vdim};
  for (int i = 0; i < 7; ++i) *f[i] = (int)dims[i];
  a.eps = (float)consts[0];
  a.temp_coef = (float)consts[1];
  a.temp_every = consts[2];
  TORCH_CHECK(a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.dim >= 1 &&
              a.vdim >= 1 && a.temp_every > 0);
  auto inside = [&](int off, int n) { return off >= 0 && off + n <= a.y.ld; };
  TORCH_CHECK(inside(a.q_off, a.H * a.dim) && inside(a.k_off, a.G * a.dim) &&
              inside(a.v_off, a.G * a.vdim));
  const OptTensor* bs[3] = {&qb, &kb, &vb};
  const float** bp[3] = {&a.qb, &a.kb, &a.vb};
  const int bn[3] = {a.H * a.dim, a.G * a.dim, a.G * a.vdim};
  for (int i = 0; i < 3; ++i)
    if (bs[i]->has_value()) {
      CHECK_F32((**bs[i]));
      TORCH_CHECK((*bs[i])->numel() == bn[i]);
      *bp[i] = (*bs[i])->data_ptr<float>();
    }
  CHECK_F32(qn);
  CHECK_F32(kn);
  TORCH_CHECK(qn.numel() == a.dim && kn.numel() == a.dim);
  a.qn = qn.data_ptr<float>();
  a.kn = kn.data_ptr<float>();
  check_act(q);
  const auto ta = q.scalar_type();
  for (const Tensor& t : {q, kp, vp})
    TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == ta,
                "q and the pages share one element type");
  a.dkp = q.size(2);
  TORCH_CHECK(q.dim() == 3 && q.size(0) == N && q.size(1) == a.H &&
              a.dkp >= a.dim);
  TORCH_CHECK(kp.dim() == 4 && vp.dim() == 4 && kp.size(1) == a.G &&
              vp.size(1) == a.G && kp.size(3) == a.dkp &&
              vp.size(3) == kp.size(2) && vp.size(2) >= a.vdim &&
              vp.size(0) == kp.size(0));
  a.q = q.data_ptr();
  a.kp = kp.data_ptr();
  a.vp = vp.data_ptr();
  a.P = kp.size(2);
  a.dvp = vp.size(2);
  CHECK_I32(table);
  CHECK_I32(tok_seq);
  CHECK_I32(tok_pos);
  TORCH_CHECK(tok_seq.numel() == N && tok_pos.numel() == N && table.dim() == 2);
  a.table = table.data_ptr<int>();
  a.maxp = table.size(1);
  a.tok_seq = tok_seq.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  if (N == 0) return;
  bool vec = true;
  for (int v : {a.y.ld, a.q_off, a.k_off, a.dim, a.dkp}) vec = vec && v % 4 == 0;
  const size_t lds = 4 * 4 * ((size_t)(a.dim + 7) & ~7);
  by_type(parts.scalar_type(), [&](auto p) {
    by_type(ta, [&](auto t) {
      by_bool(vec, [&](auto v) {
        auto k = head_post_kernel<decltype(p), decltype(t),
                                  decltype(v)::value ? 4 : 1>;
        allow_lds(k, lds);
        k<<<dim3(N, (a.H + 2 * a.G + 3) / 4), 256, lds, cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

// dims: [q,k,v offsets, H, G, maps, dim, vdim, rotated dimensions]
void rope_post(Tensor parts, std::vector<long> dims, double amp, Tensor turns,
               Tensor q, Tensor kp, Tensor vp, Tensor table, Tensor tok_seq,
               Tensor tok_pos) {
  TORCH_CHECK(dims.size() == 9);
  RopePostArgs a{};
  a.y = as_parts(parts);
  const long N = parts.size(1);
  int* f[9] = {&a.q_off, &a.k_off, &a.v_off, &a.H, &a.G, &a.M, &a.dim, &a.vdim,
               &a.rdims};
  for (int i = 0; i < 9; ++i) *f[i] = (int)dims[i];
  a.amp = (float)amp;
  TORCH_CHECK(a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.M >= 1 && a.dim >= 1 &&
              a.vdim >= 1 && a.rdims >= 2 && a.rdims % 2 == 0 && a.rdims <= a.dim);
  auto inside = [&](int off, int n) { return off >= 0 && off + n <= a.y.ld; };
  TORCH_CHECK(inside(a.q_off, a.H * a.M * a.dim) &&
              inside(a.k_off, a.G * a.M * a.dim) && inside(a.v_off, a.G * a.vdim));
  CHECK_T(turns, at::kDouble);
  TORCH_CHECK(turns.numel() == a.rdims / 2);
  a.turns = turns.data_ptr<double>();
  check_act(q);
  const auto ta = q.scalar_type();
  for (const Tensor& t : {q, kp, vp})
    TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == ta,
                "q and the pages share one element type");
  TORCH_CHECK(q.dim() == 4 && q.size(0) == N && q.size(1) == a.H &&
              q.size(2) == a.M && q.size(3) >= a.dim);
  a.dk = q.size(3);
  TORCH_CHECK(kp.dim() == 4 && vp.dim() == 4 && kp.size(1) == a.G &&
              vp.size(1) == a.G && kp.size(3) == (long)a.M * a.dk &&
              vp.size(3) == kp.size(2) && vp.size(2) >= a.vdim &&
              vp.size(0) == kp.size(0));
  a.q = q.data_ptr();
  a.kp = kp.data_ptr();
  a.vp = vp.data_ptr();
  a.P = kp.size(2);
  a.dvp = vp.size(2);
  CHECK_I32(table);
  CHECK_I32(tok_seq);
  CHECK_I32(tok_pos);
  TORCH_CHECK(tok_seq.numel() == N && tok_pos.numel() == N && table.dim() == 2);
  a.table = table.data_ptr<int>();
  a.maxp = table.size(1);
  a.tok_seq = tok_seq.data_ptr<int>();
  a.tok_pos = tok_pos.data_ptr<int>();
  if (N == 0) return;
  bool vec = true;
  for (int v : {a.y.ld, a.q_off, a.k_off, a.v_off, a.dim, a.vdim, a.dk, a.dvp})
    vec = vec && v % 8 == 0;
  // few rows: more workgroups on each
  const int units = (a.H + a.G) * a.M + a.G;
  a.per = N >= 256 ? units : 8;
  const size_t lds = 4 * (size_t)a.rdims;
  by_type(parts.scalar_type(), [&](auto p) {
    by_type(ta, [&](auto t) {
      by_bool(vec, [&](auto v) {
        rope_post_kernel<decltype(p), decltype(t), decltype(v)::value ? 8 : 1>
            <<<dim3(N, (units + a.per - 1) / a.per), 256, lds, cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

// dims: [act, gate or up, up, ff, router offset, E, NI, top, sigmoid scores,
//        renormalize]
void ff_post(OptTensor parts, OptTensor rparts, std::vector<long> dims,
             double rscale, OptTensor corr, Tensor out, OptTensor ids,
             OptTensor wts, OptTensor idw) {
  TORCH_CHECK(dims.size() == 10);
  FfPostArgs a{};
  int* f[10] = {&a.act, &a.u_off, &a.u2_off, &a.ff, &a.rt.off, &a.rt.E,
                &a.rt.NI, &a.rt.top, &a.rt.sigmoid, &a.rt.renorm};
  for (int i = 0; i < 10; ++i) *f[i] = (int)dims[i];
  check_act(out);
  TORCH_CHECK(out.dim() == 2 && out.is_contiguous());
  const long N = out.size(0);
  a.out = out.data_ptr();
  a.ldo = out.size(1);
  TORCH_CHECK(a.act >= 0 && a.act <= 2 && a.ff >= 0 && a.ff <= a.ldo);
  auto tp = at::kFloat;
  if (a.act) {
    TORCH_CHECK(parts.has_value());
    a.y = as_parts(*parts);
    tp = parts->scalar_type();
    auto inside = [&](int off) { return off >= 0 && off + a.ff <= a.y.ld; };
    TORCH_CHECK(parts->size(1) == N && inside(a.u_off) &&
                (a.act != 1 || inside(a.u2_off)));
  } else {
    a.ff = 0;
  }
  if (a.rt.E + a.rt.NI > 0) {
    TORCH_CHECK(rparts.has_value() && ids.has_value() && wts.has_value());
    a.rt.scale = (float)rscale;
    set_logits(a.rt, *rparts, N);
    set_routing(a.rt, N, corr, *ids, *wts, idw);
  }
  if (N == 0) return;
  bool vec = a.ldo % 8 == 0 && a.ff % 8 == 0;
  if (a.act)
    for (int v : {a.y.ld, a.u_off, a.u2_off}) vec = vec && (v < 0 || v % 8 == 0);
  const dim3 grid(N, 1 + (a.ldo + POST_CHUNK - 1) / POST_CHUNK);
  by_type(tp, [&](auto p) {
    by_type(out.scalar_type(), [&](auto t) {
      by_bool(vec, [&](auto v) {
        ff_post_kernel<decltype(p), decltype(t), decltype(v)::value ? 8 : 1>
            <<<grid, POST_BLOCK, 0, cur_stream()>>>(a);
      });
    });
  });
  check_launch();
}

Tensor router_gemm(Tensor A, Tensor W) {
  CHECK_T(A, at::kBFloat16);
  CHECK_T(W, at::kBFloat16);
  TORCH_CHECK(A.dim() == 2 && W.dim() == 2 && A.size(1) == W.size(1) &&
              A.size(1) % 32 == 0);
  const int M = A.size(0), N = W.size(0), K = A.size(1);
  auto C = torch::empty({1, M, N}, A.options().dtype(at::kFloat));
  if (M == 0) return C;
  router_gemm_kernel<<<dim3((N + 63) / 64, (M + 31) / 32), 256, 0,
                       cur_stream()>>>(
      (const bf16_bits*)A.data_ptr(), (const bf16_bits*)W.data_ptr(),
      C.data_ptr<float>(), M, N, K);
  check_launch();
  return C;
}

// (ksplit, M, N) f32 partials of A @ W^T, M <= 32.
Tensor gemm_parts(Tensor A, Tensor W, long ksplit_req) {
  CHECK_T(A, at::kBFloat16);
  CHECK_T(W, at::kBFloat16);
  TORCH_CHECK(A.dim() == 2 && W.dim() == 2 && A.size(1) == W.size(1));
  const int M = A.size(0), N = W.size(0), K = A.size(1);
  TORCH_CHECK(M >= 1 && M <= 32 && K % 32 == 0 && N % 64 == 0,
              "need M <= 32, K % 32 == 0, N % 64 == 0");
  int ks = (int)ksplit_req;
  if (ks <= 0) {
    // as gemm_skinny: one split once N alone covers the chip, else up to
    // eight so that narrow outputs still fill it
    ks = N / 64 >= 256 ? 1
                       : (int)std::min<long>(
                             K / 512, std::max<long>(
                                          1, std::min<long>(8, 1024 / (N / 64))));
  }
  ks = std::max(1, ks);
  const bool v2 = K % 256 == 0;
  int kchunk = K;
  if (v2) {
    const int nch = K / 256, per = (nch + ks - 1) / ks;
    ks = (nch + per - 1) / per;
    kchunk = per * 256;
  }
  auto part = torch::empty({ks, M, N}, A.options().dtype(at::kFloat));
  const bf16_bits* ap = (const bf16_bits*)A.data_ptr();
  const bf16_bits* wp = (const bf16_bits*)W.data_ptr();
  float* pp = part.data_ptr<float>();
  const dim3 grid(N / 64, ks);
  by_bool(M > 16, [&](auto two) {
    constexpr int MT = decltype(two)::value ? 2 : 1;
    if (v2)
      gemm_skinny_v2_kernel<MT><<<grid, 256, 0, cur_stream()>>>(
          ap, wp, nullptr, nullptr, nullptr, pp, M, N, K, kchunk, ks, nullptr,
          0.f, 0, nullptr, 0, nullptr);
    else
      gemm_skinny_kernel<MT><<<grid, 256, 0, cur_stream()>>>(
          ap, wp, nullptr, nullptr, nullptr, pp, M, N, K, ks);
  });
  check_launch();
  return part;
}

// ---------------------------------------------------------------------------
// attention
// ---------------------------------------------------------------------------

template <int DK, int DV>
static void launch_mfma(AttnArgs& a, const Tensor& pre, const Tensor& dec,
                        long max_new, long max_ctx, const Tensor& like) {
  const int Hg = a.H / a.G;
  if (pre.numel() > 0) {
    constexpr int QC = (DK > 128 || DV > 128) ? 1 : 2;
    a.list = pre.data_ptr<int>();
    const long rows = max_new * Hg;
    attn_ragged_prefill_kernel<DK, DV, QC>
        <<<dim3((rows + 64 * QC - 1) / (64 * QC), a.G, pre.numel()), 256, 0,
           cur_stream()>>>(a);
    check_launch();
  }
  if (dec.numel() > 0) {
    a.list = dec.data_ptr<int>();
    const int nch = (Hg + 15) / 16;
    const long units = dec.numel() * a.G * nch;
    // tiles a sequence can see, and enough workgroups to fill the chip with
    // at least two tiles for each wave of them
    const long tiles = (seen_keys(a, max_ctx) + 31) / 32 + 1;
    a.n_split = (int)std::max<long>(
        1, std::min<long>({32, 512 / std::max<long>(1, units), tiles / 8}));
    Tensor pml, pacc;
    if (a.n_split > 1) {
      auto o = like.options().dtype(at::kFloat);
      pml = torch::empty({units * a.n_split, 16, 2}, o);
      pacc = torch::empty({units * a.n_split, 16, DV}, o);
      a.pml = pml.data_ptr<float>();
      a.pacc = pacc.data_ptr<float>();
    }
    attn_ragged_decode_kernel<DK, DV>
        <<<dim3(units, a.n_split), 256, 0, cur_stream()>>>(a);
    check_launch();
    if (a.n_split > 1) {
      attn_ragged_combine_kernel<<<units, 256, 0, cur_stream()>>>(a);
      check_launch();
    }
  }
}

void attn_ragged(Tensor q, Tensor kp, OptTensor vp, Tensor table,
                 Tensor tok_seq, Tensor tok_pos, Tensor cu, Tensor q_start,
                 Tensor pre, Tensor dec, long max_new, long max_ctx, long dim,
                 long vdim, double scale, long window, long chunk,
                 OptTensor slopes, OptTensor sinks, OptTensor gate, Tensor out) {
  check_act(q);
  const auto ta = q.scalar_type();
  TORCH_CHECK(q.dim() == 3 && q.is_contiguous());
  AttnArgs a{};
  const long N = q.size(0);
  a.H = q.size(1);
  a.dkp = q.size(2);
  TORCH_CHECK(kp.dim() == 4);
  a.G = kp.size(1);
  a.P = kp.size(2);
  a.dvp = a.dkp;
  a.dim = (int)dim;
  a.vdim = (int)vdim;
  if (vp.has_value()) {
    TORCH_CHECK(vp->dim() == 4 && vp->size(1) == a.G && vp->size(3) == a.P &&
                vp->size(0) == kp.size(0));
    a.dvp = vp->size(2);
    a.vp = vp->data_ptr();
  }
  TORCH_CHECK(a.H % a.G == 0 && kp.size(3) == a.dkp && dim >= 1 && vdim >= 1 &&
              dim <= a.dkp && vdim <= a.dvp);
  for (const Tensor& t : {kp, vp.value_or(kp)})
    TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == ta,
                "pages must have the element type of q");
  for (const Tensor& t : {table, tok_seq, tok_pos, cu, q_start, pre, dec})
    CHECK_I32(t);
  TORCH_CHECK(table.dim() == 2 && tok_seq.numel() == N && tok_pos.numel() == N &&
              cu.numel() == table.size(0) + 1 &&
              q_start.numel() == table.size(0));
  TORCH_CHECK(out.is_cuda() && out.dim() == 2 && out.size(0) == N &&
              out.stride(1) == 1 && out.scalar_type() == ta &&
              out.size(1) >= a.H * vdim);
  if (slopes.has_value()) {
    CHECK_F32((*slopes));
    TORCH_CHECK(slopes->numel() == a.H);
    a.slopes = slopes->data_ptr<float>();
  }
  if (sinks.has_value()) {
    CHECK_F32((*sinks));
    TORCH_CHECK(sinks->numel() == a.H);
    a.sinks = sinks->data_ptr<float>();
  }
  if (gate.has_value()) {
    TORCH_CHECK(gate->is_cuda() && gate->dim() == 2 && gate->size(0) == N &&
                gate->stride(1) == 1 && gate->scalar_type() == ta &&
                gate->size(1) >= a.H * vdim);
    a.gate = gate->data_ptr();
    a.ldg = gate->stride(0);
  }
  if (N == 0) return;
  a.q = q.data_ptr();
  a.kp = kp.data_ptr();
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
  a.maps = 1;
  a.scale = (float)scale;
  a.n_split = 1;

  auto size_ok = [](int d) { return d == 32 || d == 64 || d == 128 || d == 256; };
  if (ta == at::kBFloat16 && a.vp && (size_ok(a.dkp) || a.dkp == 192) &&
      size_ok(a.dvp) && a.P % 8 == 0 && 32 % a.P == 0) {
    auto by_dim = [](int d, auto f) {
      if (d == 32) f(std::integral_constant<int, 32>{});
      else if (d == 64) f(std::integral_constant<int, 64>{});
      else if (d == 128) f(std::integral_constant<int, 128>{});
      else f(std::integral_constant<int, 256>{});
    };
    auto by_key = [&](int d, auto f) {
      if (d == 192) f(std::integral_constant<int, 192>{});
      else by_dim(d, f);
    };
    by_key(a.dkp, [&](auto dk) {
      by_dim(a.dvp, [&](auto dv) {
        launch_mfma<decltype(dk)::value, decltype(dv)::value>(
            a, pre, dec, max_new, max_ctx, q);
      });
    });
    return;
  }
  TORCH_CHECK(dim <= SIMPLE_MAXD && vdim <= SIMPLE_MAXD,
              "head size above ", SIMPLE_MAXD);
  by_type(ta, [&](auto t) {
    attn_ragged_simple_kernel<decltype(t), decltype(t)>
        <<<dim3(N, a.H), 64, 0, cur_stream()>>>(a);
  });
  check_launch();
}

// ---------------------------------------------------------------------------
// routed experts
// ---------------------------------------------------------------------------

// h (N, K), up (E, planes, F, K), down (E, Wp, F), ids/wts (N, top)
// -> y (N, top, Wp); rows of skipped choices are not written. Two planes:
// gated activation (limit, slope, shift), one: relu(up)^2. win: the weight
// multiplies the expert's input, else its output.
Tensor moe_experts(Tensor h, Tensor up, Tensor down, Tensor ids, Tensor wts,
                   bool win, double limit, double slope, double shift) {
  const GluConst glu{(float)limit, (float)slope, (float)shift};
  check_act(h);
  const auto ta = h.scalar_type();
  for (const Tensor& t : {h, up, down})
    TORCH_CHECK(t.is_cuda() && t.is_contiguous() && t.scalar_type() == ta);
  CHECK_I32(ids);
  CHECK_F32(wts);
  TORCH_CHECK(h.dim() == 2 && up.dim() == 4 && down.dim() == 3 &&
              ids.dim() == 2 && (up.size(1) == 1 || up.size(1) == 2));
  const int N = h.size(0), K = h.size(1);
  const int E = up.size(0), F = up.size(2), Wp = down.size(1);
  const int top = ids.size(1), S = N * top;
  TORCH_CHECK(ids.size(0) == N && wts.numel() == S && up.size(3) == K &&
              down.size(0) == E && down.size(2) == F && E >= 1 &&
              E <= MOE_MAX_E && top >= 1);
  TORCH_CHECK(K % 64 == 0 && F % 64 == 0 && Wp % 64 == 0,
              "expert sizes must be padded to 64");
  auto y = torch::empty({N, top, Wp}, h.options());
  if (N == 0) return y;
  auto act = torch::empty({S, F}, h.options());
  const int* idp = ids.data_ptr<int>();
  const float* wp = wts.data_ptr<float>();
  const float* w1 = win ? wp : nullptr;
  const float* w2 = win ? nullptr : wp;
  auto st = cur_stream();
  auto by_planes = [&](auto f) {
    if (up.size(1) == 2) f(std::integral_constant<int, 2>{});
    else f(std::integral_constant<int, 1>{});
  };

  if (ta == at::kBFloat16 && N <= 32) {
    const bf16_bits* hp = (const bf16_bits*)h.data_ptr();
    bf16_bits* actp = (bf16_bits*)act.data_ptr();
    by_bool(K % 256 == 0, [&](auto full) {
      by_planes([&](auto np) {
        moe_skinny_kernel<decltype(np)::value, decltype(full)::value>
            <<<dim3(F / 64, E), 256, 0, st>>>(
                hp, (const bf16_bits*)up.data_ptr(), idp, w1, actp, S, top, F,
                K, K, F, glu);
      });
    });
    check_launch();
    by_bool(F % 256 == 0, [&](auto full) {
      moe_skinny_kernel<0, decltype(full)::value>
          <<<dim3(Wp / 64, E), 256, 0, st>>>(
              actp, (const bf16_bits*)down.data_ptr(), idp, w2,
              (bf16_bits*)y.data_ptr(), S, top, Wp, F, F, Wp, glu);
    });
    check_launch();
    return y;
  }

  const int BM = ta == at::kBFloat16 && S / E >= 96 ? 128 : 64;
  const int max_tiles = S / BM + std::min(S, E);  // the count goes behind
  auto iopt = ids.options();
  auto off = torch::empty({E + 1}, iopt);
  auto sorted = torch::empty({S}, iopt);
  auto tiles = torch::empty({max_tiles + 1, 2}, iopt);
  int* offp = off.data_ptr<int>();
  int* sp = sorted.data_ptr<int>();
  int* tp = tiles.data_ptr<int>();
  moe_sort_kernel<<<1, 1024, 0, st>>>(idp, offp, sp, tp, S, E, BM, max_tiles);
  check_launch();
  if (ta == at::kFloat) {
    by_planes([&](auto np) {
      moe_simple_kernel<decltype(np)::value>
          <<<dim3(F / 64, max_tiles), 256, 0, st>>>(
              h.data_ptr<float>(), up.data_ptr<float>(), offp, sp, tp, w1,
              act.data_ptr<float>(), top, F, K, K, F, glu);
    });
    check_launch();
    moe_simple_kernel<0><<<dim3(Wp / 64, max_tiles), 256, 0, st>>>(
        act.data_ptr<float>(), down.data_ptr<float>(), offp, sp, tp, w2,
        y.data_ptr<float>(), top, Wp, F, F, Wp, glu);
    check_launch();
    return y;
  }
  auto tile = [&](auto bm) {
    constexpr int B = decltype(bm)::value;
    const int per = up.size(1) == 2 ? 128 : 256;
    const int nu = (F + per - 1) / per, nd = (Wp + 255) / 256;
    by_planes([&](auto np) {
      moe_tile_kernel<B, decltype(np)::value><<<nu * max_tiles, 256, 0, st>>>(
          (const bf16_bits*)h.data_ptr(), (const bf16_bits*)up.data_ptr(), offp,
          sp, tp, w1, (bf16_bits*)act.data_ptr(), max_tiles, nu, top, F, K, K,
          F, glu);
    });
    check_launch();
    moe_tile_kernel<B, 0><<<nd * max_tiles, 256, 0, st>>>(
        (const bf16_bits*)act.data_ptr(), (const bf16_bits*)down.data_ptr(),
        offp, sp, tp, w2, (bf16_bits*)y.data_ptr(), max_tiles, nd, top, Wp, F,
        F, Wp, glu);
    check_launch();
  };
  if (BM == 128) tile(std::integral_constant<int, 128>{});
  else tile(std::integral_constant<int, 64>{});
  return y;
}

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_rows", &embed_rows);
  m.def("residual_norm", &residual_norm);
  m.def("clamped_glu", &clamped_glu);
  m.def("softcap", &softcap);
  m.def("proj_post", &proj_post);
  m.def("head_post", &head_post);
  m.def("rope_post", &rope_post);
  m.def("ff_post", &ff_post);
  m.def("router_gemm", &router_gemm);
  m.def("gemm_parts", &gemm_parts);
  m.def("attn_ragged", &attn_ragged);
  m.def("moe_experts", &moe_experts);
}
