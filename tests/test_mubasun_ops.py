"""The Mubasun mechanisms one by one against the plain oracle: grouped norm and
residual fold, projections to q/k/v/gate/activation, routing, experts, paged
ragged attention. CPU forms run here, the HIP kernels under -m gpu."""
import math

import pytest
import torch

import mubasun_oracle as oracle
from bloombee_amd.kv.batch import DecodeSlots, build_batch
from bloombee_amd.kv.paged import PagedKVCache
from bloombee_amd.ops import ragged
from bloombee_amd.ops.reference import distance_slopes
from bloombee_amd.ops.ragged import (Pending, ProjSpec, Routing, pad_head,
                                     round_up)

GPU = pytest.mark.gpu
KINDS = [pytest.param("cpu", torch.float32, id="cpu-f32"),
         pytest.param("cuda:0", torch.float32, id="gpu-f32", marks=GPU),
         pytest.param("cuda:0", torch.bfloat16, id="gpu-bf16", marks=GPU)]
kinds = pytest.mark.parametrize("dev,dt", KINDS)


def tol(dt):
    return dict(rtol=2e-5, atol=2e-5) if dt == torch.float32 else \
        dict(rtol=2e-2, atol=2e-2)


def rnd(*shape, seed=0, scale=1.0):
    g = torch.Generator().manual_seed(seed)
    return (torch.randn(*shape, generator=g) * scale).bfloat16().float()


# ---------------------------------------------------------------------------
# grouped norm and residual fold
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("W,groups,cols", [
    (96, 3, 128), (250, 5, 256), (4096, 8, 4096), (2304, 1, 2304), (60, 30, 64)])
def test_grouped_norm(dev, dt, W, groups, cols):
    N, eps = 5, 1e-3
    x = rnd(N, W, seed=1, scale=3.0)
    x[:, : W // groups] *= 50          # parts of very different sizes
    x[1] *= 1e-3                       # eps shows
    w = 1 + rnd(W, seed=2, scale=0.3)
    xd = x.to(dev)
    h = ragged.residual_norm(xd, None, w.to(dev), groups, eps, cols, dt)
    want = oracle.grouped_rms(x.double(), w.double(), groups, eps)
    torch.testing.assert_close(h[:, :W].cpu().double(), want, **tol(dt))
    assert (h[:, W:] == 0).all()
    torch.testing.assert_close(xd.cpu(), x)        # nothing pending


@kinds
@pytest.mark.parametrize("W,ks", [(96, 1), (250, 3), (2560, 4)])
@pytest.mark.parametrize("top", [0, 3])
def test_residual_fold(dev, dt, W, ks, top):
    """x += sum of split-K parts + chosen experts' rows + identity weight * h."""
    N, ld = 6, round_up(W, 64)
    x = rnd(N, W, seed=1, scale=4.0)
    parts = rnd(ks, N, ld, seed=2)
    want = x.double() + parts.double().sum(0)[:, :W]
    p = Pending(parts.to(dev))
    if top:
        y = rnd(N, top, ld, seed=3)
        ids = torch.tensor([[0, -1, 2]] * N, dtype=torch.int32)
        y_dev = y.clone()
        y_dev[:, 1] = float("nan") if dev != "cpu" else 0.0   # never read
        y[:, 1] = 0
        idw = rnd(N, seed=4).abs()
        idw[2] = 0
        h = rnd(N, ld, seed=5)
        want = want + y.double().sum(1)[:, :W] + idw.double()[:, None] * h.double()[:, :W]
        p = Pending(parts.to(dev), y_dev.to(dev, dt),
                    Routing(ids.to(dev), torch.zeros(N, top, device=dev),
                            idw.to(dev)), h.to(dev, dt))
    xd = x.to(dev)
    assert ragged.residual_norm(xd, p) is None
    torch.testing.assert_close(xd.cpu().double(), want, rtol=1e-5, atol=1e-5)
    assert xd.dtype == torch.float32


# ---------------------------------------------------------------------------
# projections
# ---------------------------------------------------------------------------

def run_post(dev, dt, spec, y, rlog, qn, kn, corr, poses, G, D, V, ks=1,
             as_parts=False):
    """proj_post on projection output y (N, cols), rows of one sequence at
    positions `poses`; returns its outputs and the pages as dense k, v."""
    cache = PagedKVCache(1, G, pad_head(D), v_head_dim=pad_head(V),
                         page_size=16, max_tokens=128, device=dev, dtype=dt)
    n = len(poses)
    pages = [5, 2, 7, 0]
    b = build_batch(cache, [poses[0]], [n], [pages])
    parts = y.unsqueeze(0)
    if as_parts:      # f32 split-K partials that sum to y
        cut = rnd(ks, *y.shape, seed=9)
        cut[-1] = y - cut[:-1].sum(0)
        parts = cut
    parts = parts.to(dev) if as_parts or dt == torch.float32 else parts.to(dev, dt)
    q, gate, a2, rt = ragged.proj_post(
        parts.contiguous(), None if rlog is None else rlog.unsqueeze(0).to(dev),
        0, spec, qn.to(dev), None if kn is None else kn.to(dev),
        None if corr is None else corr.to(dev), b, cache.k_pages(0),
        cache.v_pages(0), dt)
    k, v = cache.k_pages(0).cpu().float(), cache.v_pages(0).cpu().float()
    kd = torch.stack([k[pages[p // 16], :, p % 16] for p in poses])
    vd = torch.stack([v[pages[p // 16], :, :, p % 16] for p in poses])
    return q.cpu().float(), gate.cpu().float(), a2.cpu().float(), rt, kd, vd


@kinds
@pytest.mark.parametrize("as_parts", [False, True])
@pytest.mark.parametrize("H,G,D,V", [(6, 2, 48, 40), (3, 1, 33, 17), (8, 8, 64, 128)])
def test_projection_norms_and_pages(dev, dt, as_parts, H, G, D, V):
    """q and k are normed over all heads at once, then split; k and v land in
    their page slots; the gate and the zero columns are as stated."""
    N, eps = 7, 1e-4
    sec = {}
    at = 0
    for name, n in (("q", H * D), ("k", G * D), ("v", G * V), ("g", H * V)):
        sec[name] = at
        at = round_up(at + n, 8)
    spec = ProjSpec(heads=H, kv_heads=G, dim=D, vdim=V, eps=eps, q_off=sec["q"],
                    k_off=sec["k"], v_off=sec["v"], g_off=sec["g"],
                    act_col=round_up(H * V, 8), a2_cols=round_up(H * V, 64) + 64)
    y = rnd(N, round_up(at, 64), seed=3)
    # one loud head: a per-head norm would show
    y[:, sec["q"]:sec["q"] + D] *= 16
    y[:, sec["k"]:sec["k"] + D] *= 16
    qn, kn = 1 + rnd(H * D, seed=4, scale=0.4), 1 + rnd(G * D, seed=5, scale=0.4)
    poses = list(range(12, 12 + N))    # crosses a page border
    q, gate, a2, rt, k, v = run_post(dev, dt, spec, y, None, qn, kn, None, poses,
                                     G, D, V, ks=3, as_parts=as_parts)
    yd = y.double()
    cut = lambda o, n: yd[:, o:o + n]
    qw = (oracle.rms(cut(sec["q"], H * D), eps) * qn.double()).view(N, H, D)
    kw = (oracle.rms(cut(sec["k"], G * D), eps) * kn.double()).view(N, G, D)
    t = tol(dt)
    torch.testing.assert_close(q[..., :D].double(), qw, **t)
    torch.testing.assert_close(k[..., :D].double(), kw, **t)
    torch.testing.assert_close(v[..., :V].double(),
                               cut(sec["v"], G * V).reshape(N, G, V), **t)
    torch.testing.assert_close(gate.double(), cut(sec["g"], H * V), **t)
    assert (q[..., D:] == 0).all() and (k[..., D:] == 0).all()
    assert (v[..., V:] == 0).all() and (a2[:, H * V:] == 0).all()
    assert rt is None


@kinds
@pytest.mark.parametrize("ff", [320, 75])
def test_xielu(dev, dt, ff):
    H = G = 1
    D = V = 32
    N = 4
    w = torch.tensor([0.8, -1.3])
    z = torch.linspace(-9, 9, N * ff).view(N, ff).bfloat16().float()
    z[0, :6] = torch.tensor([0.0, -0.0, 1e-3, -1e-3, 1e-5, -1e-5])
    y = torch.zeros(N, round_up(128 + ff, 64))
    y[:, 128:128 + ff] = z
    b = torch.nn.functional.softplus(w.double())
    spec = ProjSpec(heads=H, kv_heads=G, dim=D, vdim=V, eps=1e-5, q_off=0,
                    k_off=32, v_off=64, g_off=96, u_off=128, act=1, ff=ff,
                    act_col=32, a2_cols=round_up(32 + ff, 64),
                    xielu_pos=float(b[0]), xielu_neg=0.5 + float(b[1]))
    one = torch.ones(32)
    _, _, a2, _, _, _ = run_post(dev, dt, spec, y, None, one, one, None,
                                 list(range(N)), G, D, V)
    want = oracle.xielu(z.double(), w[0], w[1])
    torch.testing.assert_close(a2[:, 32:32 + ff].double(), want,
                               **(dict(rtol=1e-5, atol=1e-6)
                                  if dt == torch.float32 else tol(dt)))
    assert (a2[:, 32 + ff:] == 0).all()


def routed_spec(E, NI, top, scale, act=0, ff=0):
    return ProjSpec(heads=1, kv_heads=1, dim=32, vdim=32, eps=1e-5, q_off=0,
                    k_off=32, v_off=64, g_off=96, u_off=128 if act else -1,
                    u2_off=128 + round_up(ff, 8) if act else -1, act=act, ff=ff,
                    act_col=32, a2_cols=round_up(32 + ff, 64), experts=E,
                    identity=NI, top=top, router_scale=scale)


@kinds
@pytest.mark.parametrize("E,NI,top,scale", [
    (8, 3, 2, 2.5), (5, 0, 5, 1.0), (1, 1, 1, 0.7), (70, 60, 9, 1.5), (0, 4, 2, 1.0)])
def test_routing(dev, dt, E, NI, top, scale):
    """Correction moves the choice, not the weights; identity experts take
    part; no renormalization."""
    N, n = 33, E + NI
    g = torch.Generator().manual_seed(n)
    z = torch.randn(N, n, generator=g) * 2
    corr = torch.randn(n, generator=g) * 0.3
    spec = routed_spec(E, NI, top, scale)
    one = torch.ones(32)
    *_, rt, _, _ = run_post(dev, dt, spec, torch.zeros(N, 128), z, one, one, corr,
                            list(range(N)), 1, 32, 32)
    mlp = dict(experts=E, identity=NI, top=top, scale=scale)
    want = oracle.route(torch.eye(N).double(), {"router": z.double().T,
                                                "correction": corr.double()},
                        "", mlp)
    got = torch.zeros(N, n, dtype=torch.double)
    ids, wts = rt.ids.cpu(), rt.wts.cpu().double()
    for t in range(N):
        chosen = [int(i) for i in ids[t] if i >= 0]
        assert len(set(chosen)) == len(chosen)
        for k in range(top):
            if ids[t, k] >= 0:
                got[t, ids[t, k]] = wts[t, k]
    torch.testing.assert_close(got[:, :E], want[:, :E], rtol=1e-5, atol=1e-7)
    torch.testing.assert_close(rt.idw.cpu().double(), want[:, E:].sum(-1),
                               rtol=1e-5, atol=1e-7)


@kinds
@pytest.mark.parametrize("ff", [112, 50])
def test_shared_expert_gate(dev, dt, ff):
    """silu(gate) * up times one sigmoid per token."""
    E, NI, N = 4, 1, 6
    spec = routed_spec(E, NI, 2, 1.0, act=2, ff=ff)
    y = rnd(N, round_up(128 + 2 * round_up(ff, 8), 64), seed=7)
    rlog = rnd(N, E + NI + 1, seed=8)
    one = torch.ones(32)
    _, _, a2, _, _, _ = run_post(dev, dt, spec, y, rlog, one, one,
                                 torch.zeros(E + NI), list(range(N)), 1, 32, 32)
    yd = y.double()
    want = (oracle.silu(yd[:, 128:128 + ff])
            * yd[:, spec.u2_off:spec.u2_off + ff]
            * torch.sigmoid(rlog[:, -1:].double()))
    torch.testing.assert_close(a2[:, 32:32 + ff].double(), want, **tol(dt))


@GPU
def test_router_gemm_is_32_bit():
    h, w = rnd(77, 192, seed=1), rnd(83, 192, seed=2)
    got = ragged._ext().router_gemm(h.cuda().bfloat16(), w.cuda().bfloat16())
    torch.testing.assert_close(got[0].cpu().double(), h.double() @ w.double().T,
                               rtol=1e-5, atol=1e-4)


@GPU
@pytest.mark.parametrize("M,N,K", [(1, 64, 64), (17, 192, 96), (32, 320, 512),
                                   (9, 128, 4096), (32, 16448, 256)])
def test_gemm_parts(M, N, K):
    a, w = rnd(M, K, seed=1), rnd(N, K, seed=2)
    p = ragged.linear_parts(a.cuda().bfloat16(), w.cuda().bfloat16())
    assert p.dtype == torch.float32
    torch.testing.assert_close(p.double().sum(0).cpu(), a.double() @ w.double().T,
                               rtol=1e-5, atol=2e-3)


# ---------------------------------------------------------------------------
# experts
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("N,E,top,K,F,W", [
    (1, 3, 2, 192, 80, 192), (5, 4, 2, 96, 64, 96), (32, 6, 3, 256, 100, 250),
    (33, 5, 2, 96, 130, 96), (300, 2, 1, 512, 300, 512), (150, 9, 4, 192, 65, 190)])
def test_experts(dev, dt, N, E, top, K, F, W):
    g = torch.Generator().manual_seed(N)
    Kp, Fp, Wp = round_up(K, 64), round_up(F, 64), round_up(W, 64)
    h = torch.zeros(N, Kp)
    h[:, :K] = rnd(N, K, seed=1)
    gu, dn = torch.zeros(E, 2, Fp, Kp), torch.zeros(E, Wp, Fp)
    gu[:, :, :F, :K] = rnd(E, 2, F, K, seed=2, scale=K ** -0.5)
    dn[:, :W, :F] = rnd(E, W, F, seed=3, scale=F ** -0.5)
    # -1 (identity) among the choices, one expert that nobody takes
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(N)]).int()
    ids[ids == E - 1] = -1
    wts = torch.rand(N, top, generator=g)
    y = ragged.moe_experts(h.to(dev, dt), gu.to(dev, dt), dn.to(dev, dt),
                           Routing(ids.to(dev), wts.to(dev), None)).cpu().double()
    for t in range(N):
        for k in range(top):
            e = int(ids[t, k])
            if e < 0:
                continue
            w = {"gate": gu[e, 0].double(), "up": gu[e, 1].double(),
                 "down": dn[e].double()}
            want = oracle.glu(h[t].double(), w, "") * wts[t, k].double()
            torch.testing.assert_close(y[t, k], want, **tol(dt))


# ---------------------------------------------------------------------------
# attention
# ---------------------------------------------------------------------------

class Seqs:
    """Sequences whose keys and values are in a paged cache."""

    def __init__(self, dev, dt, G, D, V, lens, seed=0, page=16):
        self.dev, self.dt, self.G, self.D, self.V = dev, dt, G, D, V
        self.cache = PagedKVCache(
            1, G, pad_head(D), v_head_dim=pad_head(V), page_size=page,
            max_tokens=sum(round_up(n, page) for n in lens) + 4 * page,
            device=dev, dtype=dt)
        # stale values in every slot
        for t in self.cache.pools[0]:
            t.fill_(1e4)
        g = torch.Generator().manual_seed(seed)
        order = torch.randperm(self.cache.n_pages, generator=g).tolist()
        self.k = [rnd(n, G, D, seed=seed + 1 + i) for i, n in enumerate(lens)]
        self.v = [rnd(n, G, V, seed=seed + 51 + i) for i, n in enumerate(lens)]
        self.pages = []
        for n in lens:
            m = (n + page - 1) // page
            self.pages.append(order[:m])
            order = order[m:]

    def write(self):
        kp, vp = self.cache.k_pages(0), self.cache.v_pages(0)
        P = self.cache.page_size
        for k, v, pg in zip(self.k, self.v, self.pages):
            for p in range(k.shape[0]):
                page, s = pg[p // P], p % P
                kp[page, :, s, :] = 0
                kp[page, :, s, :self.D] = k[p].to(self.dev, self.dt)
                vp[page, :, :, s] = 0
                vp[page, :, :self.V, s] = v[p].to(self.dev, self.dt)

    def attend(self, qs, starts, scale, window, slopes, gate=None):
        """qs[i] (T_i, H, D): new tokens of sequence i from starts[i] on."""
        H, D, V = qs[0].shape[1], self.D, self.V
        b = build_batch(self.cache, starts, [q.shape[0] for q in qs], self.pages)
        q = torch.zeros(b.n_tokens, H, pad_head(D))
        q[..., :D] = torch.cat(qs)
        out = torch.full((b.n_tokens, H * V + 8), 7.0, device=self.dev).to(self.dt)
        ragged.attn_ragged(
            q.to(self.dev, self.dt), self.cache.k_pages(0),
            self.cache.v_pages(0), b, out, D, V, scale, window,
            slopes.to(self.dev) if slopes is not None else None,
            gate.to(self.dev, self.dt) if gate is not None else None)
        assert (out[:, H * V:] == 7).all()          # nothing beyond its columns
        out = out[:, :H * V].cpu().double().view(-1, H, V)
        return list(out.split([t.shape[0] for t in qs]))


def attend_ref(q, start, k, v, scale, window):
    """Oracle rows for new tokens `q` at `start`: a full square of queries of
    which only the new ones matter."""
    full = torch.zeros(start + q.shape[0], *q.shape[1:], dtype=torch.double)
    full[start:] = q.double()
    n = full.shape[0]
    return oracle.attend(full, k[:n].double(), v[:n].double(), scale, window)[start:]


ATOL = {torch.float32: dict(rtol=1e-5, atol=1e-5),
        torch.bfloat16: dict(rtol=2e-2, atol=2e-2)}


@kinds
@pytest.mark.parametrize("H,G,D,V", [
    (6, 2, 48, 40), (4, 1, 64, 128), (3, 3, 32, 24), (20, 1, 16, 16),
    (5, 1, 128, 64), (8, 2, 96, 200), (2, 1, 256, 256), (2, 2, 300, 20)])
@pytest.mark.parametrize("window", [0, 1, 37, 64])
def test_attention_ragged(dev, dt, H, G, D, V, window):
    """Portions of every size beside single tokens, each sequence against the
    oracle alone."""
    lens = [150, 1, 67, 90, 130, 3]
    new = [150, 1, 1, 2, 35, 3]
    s = Seqs(dev, dt, G, D, V, lens)
    s.write()
    qs = [rnd(t, H, D, seed=100 + i, scale=1.5) for i, t in enumerate(new)]
    starts = [n - t for n, t in zip(lens, new)]
    scale = D ** -0.5
    got = s.attend(qs, starts, scale, window, distance_slopes(H))
    for i, o in enumerate(got):
        want = attend_ref(qs[i], starts[i], s.k[i], s.v[i], scale, window)
        torch.testing.assert_close(o, want, **ATOL[dt], msg=lambda m: f"seq {i}: {m}")


@kinds
def test_attention_gate_and_no_bias(dev, dt):
    H, G, D, V = 4, 2, 32, 48
    s = Seqs(dev, dt, G, D, V, [70, 20])
    s.write()
    qs = [rnd(30, H, D, seed=1), rnd(1, H, D, seed=2)]
    gate = rnd(31, H * V, seed=3, scale=2.0)
    got = torch.cat(s.attend(qs, [40, 19], 0.2, 0, None, gate))
    want = []
    for q, st, k, v in zip(qs, [40, 19], s.k, s.v):
        kk = k.double().repeat_interleave(H // G, 1)
        vv = v.double().repeat_interleave(H // G, 1)
        sc = torch.einsum("thd,jhd->htj", q.double(), kk) * 0.2
        see = torch.arange(k.shape[0]) <= torch.arange(st, st + q.shape[0])[:, None]
        p = torch.softmax(sc.masked_fill(~see, -math.inf), -1)
        want.append(torch.einsum("htj,jhv->thv", p, vv))
    want = torch.cat(want) * torch.sigmoid(gate.double()).view(-1, H, V)
    torch.testing.assert_close(got, want, **ATOL[dt])


@kinds
@pytest.mark.parametrize("window", [16, 33, 40])
@pytest.mark.parametrize("decode", [False, True])
def test_window_edges(dev, dt, window, decode):
    """One key stands out so far that its value is the output wherever it is
    visible; the last query that sees it and the first that does not must
    differ. The key sits on, before and after page and tile borders."""
    H, G, D, V = 4, 2, 64, 32
    for key in (0, 15, 16, 31, 32, 63, 64):
        last = key + window - 1
        n = last + 3
        s = Seqs(dev, dt, G, D, V, [n], seed=key)
        loud = torch.zeros(D)
        loud[3] = 30.0
        s.k[0][:] *= 0.1
        s.k[0][..., 3] = 0
        s.k[0][key] = loud
        s.write()
        for pos, seen in ((last, True), (last + 1, False)):
            q = torch.zeros(1 if decode else 2, H, D)
            q[..., 3] = 30.0
            start = pos - (0 if decode else 1)
            o = s.attend([q], [start], 0.5, window, distance_slopes(H))[0][-1]
            v = s.v[0][key].double().repeat_interleave(H // G, 0)
            close = (o - v).abs().max() < 0.05
            assert bool(close) == seen, (key, pos)


@kinds
def test_far_key(dev, dt):
    """A key hundreds of tokens back, in prompts and decoded tokens; slopes
    take their share off its score."""
    H, G, D, V, n = 6, 2, 48, 40, 700
    for key in (0, 3, 255, 256, 511):
        s = Seqs(dev, dt, G, D, V, [n], seed=key)
        s.k[0][key] = 0
        s.k[0][key, :, 5] = 60.0
        s.write()
        q = rnd(9, H, D, seed=key)
        q[..., 5] = 60.0
        for new in (q, q[-1:]):
            st = n - new.shape[0]
            o = s.attend([new], [st], 0.02, 0, distance_slopes(H))[0]
            want = attend_ref(new, st, s.k[0], s.v[0], 0.02, 0)
            torch.testing.assert_close(o, want, **ATOL[dt])


@kinds
def test_long_decode_splits(dev, dt):
    """Long contexts at a small batch: the visible range is split over
    workgroups and folded again."""
    H, G, D, V = 4, 1, 64, 64
    lens = [1900, 333, 5]
    s = Seqs(dev, dt, G, D, V, lens)
    s.write()
    qs = [rnd(1, H, D, seed=i, scale=2.0) for i in range(3)]
    for window in (0, 1500):
        got = s.attend(qs, [n - 1 for n in lens], 0.125, window,
                       distance_slopes(H) * 0.01)
        for i in range(3):
            k, v = s.k[i].double(), s.v[i].double()
            sc = (qs[i][0].double() @ k[:, 0].T) * 0.125
            dist = lens[i] - 1 - torch.arange(lens[i])
            sc = sc - distance_slopes(H).double()[:, None] * 0.01 * dist
            if window:
                sc = sc.masked_fill(dist >= window, -math.inf)
            want = torch.softmax(sc, -1) @ v[:, 0]
            torch.testing.assert_close(got[i][0], want, **ATOL[dt])


@kinds
def test_empty_slots(dev, dt):
    """Rows at position -1 write nothing and disturb nobody."""
    H, G, D, V = 4, 2, 32, 32
    s = Seqs(dev, dt, G, D, V, [40])
    s.write()
    slots = DecodeSlots(s.cache, 4, 64)
    slots.fill([1], [39], s.pages)
    before = [t.clone() for t in s.cache.pools[0]]
    spec = ProjSpec(heads=H, kv_heads=G, dim=D, vdim=V, eps=1e-5, q_off=0,
                    k_off=128, v_off=192, g_off=256, act_col=128, a2_cols=128)
    y = rnd(4, 384, seed=1)
    q, gate, a2, _ = ragged.proj_post(
        y[None].to(dev), None, 0, spec, torch.ones(128, device=dev),
        torch.ones(64, device=dev), None, slots.batch, s.cache.k_pages(0),
        s.cache.v_pages(0), dt)
    changed = [(a != b).flatten(1).any(1).nonzero()[:, 0].tolist()
               for a, b in zip(before, s.cache.pools[0])]
    assert changed == [[s.pages[0][2]], [s.pages[0][2]]]
    ragged.attn_ragged(q, s.cache.k_pages(0), s.cache.v_pages(0), slots.batch,
                       a2, D, V, 0.2, 0, None, gate)
    assert torch.isfinite(a2[0]).all()


def test_slopes_are_not_alibi_off_powers_of_two():
    from bloombee_amd.ops.reference import alibi_slopes
    torch.testing.assert_close(distance_slopes(8), alibi_slopes(8))
    for h in (3, 6, 12):
        torch.testing.assert_close(distance_slopes(h).double(),
                                   oracle.slopes(h, torch.double), rtol=1e-6,
                                   atol=0)
        assert not torch.allclose(distance_slopes(h), alibi_slopes(h))


@kinds
def test_embedding(dev, dt):
    table, pos = rnd(50, 36, seed=1).to(dt), rnd(20, 36, seed=2).to(dt)
    ids, p = torch.tensor([[3, 49, 0]]), torch.tensor([[0, 19, 7]])
    x = ragged.embed_rows(ids.to(dev), p.to(dev), table.to(dev), pos.to(dev))
    assert x.dtype == torch.float32
    torch.testing.assert_close(x.cpu(), table.float()[ids] + pos.float()[p])
