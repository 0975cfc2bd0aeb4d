"""The Risepel mechanisms one by one against the plain oracle: norm after the
sum, clamped feed-forward, capped logits, latents and rotation, latent attention
with a sink, gated linear attention. CPU forms run here, the HIP kernels under
-m gpu."""
import math

import pytest
import torch

import risepel_oracle as oracle
from bloombee_amd.kv.batch import DecodeSlots, build_batch
from bloombee_amd.kv.paged import PagedKVCache
from bloombee_amd.ops import mixers, ragged
from bloombee_amd.ops.mixers import GlaSpec, LatentSpec, LatentWeights
from bloombee_amd.ops.ragged import round_up

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


def as_parts(y, dev, dt, splits):
    """y (N, cols) as a GEMM leaves it: one part of the activation type, or
    f32 partials."""
    if splits == 1:
        return y.unsqueeze(0).to(dev, dt).contiguous()
    cut = rnd(splits, *y.shape, seed=9)
    cut[-1] = y - cut[:-1].sum(0)
    return cut.to(dev).contiguous()


# ---------------------------------------------------------------------------
# rows
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("W,cols,splits,bias,alpha", [
    (96, 128, 1, True, 2.5), (250, 256, 3, False, 1.0), (2560, 2560, 4, True, 0.7),
    (4096, 4096, 1, True, 3.25)])
def test_norm_after_the_sum(dev, dt, W, cols, splits, bias, alpha):
    N, eps = 5, 1e-3
    x = rnd(N, W, seed=1, scale=2.0)
    x[1] *= 2.0 ** -10                        # eps shows
    y = rnd(N, round_up(W, 64), seed=2)
    y[1] *= 2.0 ** -10
    b = rnd(W, seed=3, scale=0.01) if bias else None
    w = rnd(W, seed=4, scale=0.3)
    xd = x.clone().to(dev)
    h = ragged.sum_norm(xd, as_parts(y, dev, dt, splits),
                        b.to(dev) if bias else None, (1 + w).to(dev), alpha, eps,
                        cols, dt)
    s = alpha * x.double() + y[:, :W].double() + (b.double() if bias else 0)
    want = oracle.zero_norm(s, w.double(), eps)
    assert xd.dtype == torch.float32
    torch.testing.assert_close(xd.cpu().double(), want, rtol=1e-4, atol=1e-4)
    torch.testing.assert_close(h[:, :W].cpu().double(), want, **tol(dt))
    assert (h[:, W:] == 0).all()


@kinds
@pytest.mark.parametrize("ff,splits,limit,slope", [
    (320, 1, 1.5, 1.702), (77, 3, 0.6, 1.0), (128, 2, 7.0, 1.702)])
def test_clamped_glu(dev, dt, ff, splits, limit, slope):
    N, up, cols = 6, round_up(ff, 8), round_up(ff, 64) + 64
    y = rnd(N, round_up(up + ff, 64), seed=1, scale=3.0)
    gb, ub = rnd(ff, seed=2), rnd(ff, seed=3)
    # on, just above and just below the limits
    edge = torch.tensor([limit, limit + 0.25, limit - 0.25, -limit, -limit - 0.25,
                         -limit + 0.25, 40.0, -40.0])
    y[0, :8] = edge - gb[:8]
    y[0, up:up + 8] = edge - ub[:8]
    out = ragged.clamped_glu(as_parts(y, dev, torch.float32, splits), 0, up, ff,
                             gb.to(dev), ub.to(dev), limit, slope, cols, dt)
    g = (y[:, :ff] + gb).double().clamp(max=limit)
    u = (y[:, up:up + ff] + ub).double().clamp(-limit, limit)
    want = g * oracle.sigmoid(slope * g) * (u + 1)
    if slope == 1.702:
        torch.testing.assert_close(want, oracle.clamped_glu(
            (y[:, :ff] + gb).double(), (y[:, up:up + ff] + ub).double(), limit))
    torch.testing.assert_close(out[:, :ff].cpu().double(), want, **tol(dt))
    assert (out[:, ff:] == 0).all()


@kinds
def test_softcap(dev, dt):
    z = torch.linspace(-200, 200, 4001)
    for cap in (5.0, 30.0):
        got = ragged.softcap_(z.clone().to(dev), cap)
        torch.testing.assert_close(got.cpu().double(),
                                   oracle.softcap(z.double(), cap),
                                   rtol=1e-5, atol=1e-5)


@kinds
def test_embedding_without_positions(dev, dt):
    table = rnd(50, 36, seed=1).to(dt)
    ids = torch.tensor([[3, 49, 0]])
    x = ragged.embed_rows(ids.to(dev), ids.to(dev), table.to(dev), None)
    assert x.dtype == torch.float32
    torch.testing.assert_close(x.cpu(), table.float()[ids])


# ---------------------------------------------------------------------------
# latents
# ---------------------------------------------------------------------------

def latent_spec(H, D, E, V, R, Q=48, scale=None, window=0, turned=None, eps=1e-3):
    s = LatentSpec(heads=H, dim=D, rot=E, rot_dims=turned or E, vdim=V, q_rank=Q,
                   rank=R, scale=scale or (D + E) ** -0.5, window=window, eps=eps)
    s.c_off = round_up(Q, 8)
    s.g_off = round_up(s.c_off + R + E, 8)
    s.out_cols, s.q_cols = round_up(H * V, 64) + 64, round_up(Q, 64)
    return s


def page_cache(s, tokens, dev, dt, page=16, seqs=4):
    return PagedKVCache(1, 1, s.ck, layout=["k"], page_size=page,
                        max_tokens=tokens, device=dev, dtype=dt, max_seqs=seqs)


@kinds
@pytest.mark.parametrize("splits", [1, 3])
@pytest.mark.parametrize("E,turned,R,Q", [(16, 16, 80, 96), (6, 6, 30, 27),
                                          (64, 32, 200, 128)])
def test_latent_norms_rotation_and_pages(dev, dt, splits, E, turned, R, Q):
    """Positions around a page border and far out; the part of the rotated
    vector beyond its turned dimensions passes."""
    H, D, V, N, base = 3, 32, 24, 7, 5e4
    s = latent_spec(H, D, E, V, R, Q, turned=turned)
    y = rnd(N, round_up(s.g_off + H * V, 64), seed=1)
    qn, cn = 1 + rnd(Q, seed=2, scale=0.3), 1 + rnd(R, seed=3, scale=0.3)
    turns = mixers.rotary_turns(base, turned)
    for first in (12, 4000):
        cache = page_cache(s, first + 64, dev, dt)
        pages = list(range(cache.n_pages - 1, -1, -1))
        b = build_batch(cache, [first], [N], [pages])
        kp = cache.k_pages(0)
        kp.fill_(7)
        cq, gate = mixers.latent_post(
            as_parts(y, dev, dt, splits), s, qn.to(dev), cn.to(dev),
            turns.to(dev), b, kp, dt)
        yd = y.double()
        want = oracle.rms(yd[:, :Q], s.eps) * qn.double()
        torch.testing.assert_close(cq[:, :Q].cpu().double(), want, **tol(dt))
        assert (cq[:, Q:] == 0).all()
        torch.testing.assert_close(gate.cpu().double(),
                                   yd[:, s.g_off:s.g_off + H * V], **tol(dt))
        got = torch.stack([kp[pages[p // 16], 0, p % 16]
                           for p in range(first, first + N)]).cpu().double()
        c = oracle.rms(yd[:, s.c_off:s.c_off + R], s.eps) * cn.double()
        r = oracle.rotate(yd[:, s.c_off + R:s.c_off + R + E], base, turned, first)
        torch.testing.assert_close(got[:, :R], c, **tol(dt))
        torch.testing.assert_close(got[:, s.rp:s.rp + E], r, **tol(dt))
        # nothing else was written
        assert int((kp != 7).any(-1).sum()) == N


@kinds
def test_shared_latents_write_nothing(dev, dt):
    s = latent_spec(2, 32, 16, 32, 48)
    s.c_off = -1
    s.g_off = 48
    cache = page_cache(s, 64, dev, dt)
    b = build_batch(cache, [3], [2], [[0, 1]])
    mixers.latent_post(as_parts(rnd(2, 128), dev, dt, 1), s,
                       torch.ones(48, device=dev), None,
                       mixers.rotary_turns(1e4, 16).to(dev), b, cache.k_pages(0), dt)
    assert (cache.k_pages(0) == 0).all()


class Latents:
    """Sequences whose latents and rotated key parts are in a paged cache."""

    def __init__(self, dev, dt, s, lens, seed=0, page=16, base=1e4, uk=1.0):
        self.dev, self.dt, self.s, self.base = dev, dt, s, base
        self.cache = page_cache(s, sum(round_up(n, page) for n in lens) + 4 * page,
                                dev, dt, page)
        self.cache.k_pages(0).fill_(1e3)       # stale values in every slot
        g = torch.Generator().manual_seed(seed)
        order = torch.randperm(self.cache.n_pages, generator=g).tolist()
        self.c = [rnd(n, s.rank, seed=seed + 1 + i) for i, n in enumerate(lens)]
        self.r = [rnd(n, s.rot, seed=seed + 51 + i) for i, n in enumerate(lens)]
        self.uk = rnd(s.heads * s.dim, s.rank, seed=seed + 97,
                      scale=uk * s.rank ** -0.5)
        self.uv = rnd(s.heads * s.vdim, s.rank, seed=seed + 98,
                      scale=s.rank ** -0.5)
        self.sink = rnd(s.heads, seed=seed + 99)
        self.pages = []
        for n in lens:
            m = (n + page - 1) // page
            self.pages.append(order[:m])
            order = order[m:]

    def write(self):
        kp, P, s = self.cache.k_pages(0), self.cache.page_size, self.s
        for c, r, pg in zip(self.c, self.r, self.pages):
            for p in range(c.shape[0]):
                row = kp[pg[p // P], 0, p % P]
                row[:] = 0
                row[:s.rank] = c[p].to(self.dev, self.dt)
                row[s.rp:s.rp + s.rot] = r[p].to(self.dev, self.dt)

    def weights(self):
        s = self.s
        H, D, V, R = s.heads, s.dim, s.vdim, s.rank
        uk = torch.zeros(H, s.rp, round_up(D, 32))
        uk[:, :R, :D] = self.uk.view(H, D, R).transpose(1, 2)
        uv = torch.zeros(H, round_up(V, 64), s.rp)
        uv[:, :V, :R] = self.uv.view(H, V, R)
        ukv = torch.zeros(round_up(H * (D + V), 64), s.ck)
        ukv[:H * (D + V), :R] = torch.cat([self.uk, self.uv])
        to = lambda t: t.to(self.dev, self.dt)
        return LatentWeights(to(uk), to(uv), to(ukv), self.sink.to(self.dev))

    def attend(self, qs, starts, gate=None, splits=1):
        """qs[i] (T_i, H, D + E): unrotated queries of sequence i."""
        s = self.s
        counts = [q.shape[0] for q in qs]
        b = build_batch(self.cache, starts, counts, self.pages)
        N, used = b.n_tokens, s.heads * s.vdim
        y = torch.zeros(N, round_up(s.heads * (s.dim + s.rot), 64))
        y[:, :s.heads * (s.dim + s.rot)] = torch.cat(qs).reshape(N, -1)
        if gate is None:
            gate = torch.full((N, used), 40.0)        # sigmoid = 1
        out = mixers.latent_attention(
            as_parts(y, self.dev, self.dt, splits), s, self.weights(),
            mixers.rotary_turns(self.base, s.rot_dims).to(self.dev), b,
            gate.to(self.dev, self.dt).contiguous(), self.cache.k_pages(0), self.dt)
        assert (out[:, used:] == 0).all()
        return list(out[:, :used].cpu().double().view(N, s.heads, s.vdim)
                    .split(counts))

    def want(self, i, q, start):
        """Oracle rows for the new tokens q of sequence i."""
        s = self.s
        H, D, V = s.heads, s.dim, s.vdim
        n = start + q.shape[0]
        full = torch.zeros(n, H, D + s.rot, dtype=torch.double)
        full[start:] = q.double()
        full = torch.cat([full[..., :D], oracle.rotate(
            full[..., D:], self.base, s.rot_dims)], -1)
        c = self.c[i][:n].double()
        k = torch.cat([(c @ self.uk.double().T).view(n, H, D),
                       self.r[i][:n].double()[:, None].expand(n, H, s.rot)], -1)
        v = (c @ self.uv.double().T).view(n, H, V)
        return oracle.attend(full, k, v, s.scale, s.window,
                             self.sink.double())[start:]


ATOL = {torch.float32: dict(rtol=2e-5, atol=2e-5),
        torch.bfloat16: dict(rtol=3e-2, atol=3e-2)}


@kinds
@pytest.mark.parametrize("H,D,E,V,R", [
    (6, 48, 16, 40, 80), (3, 18, 6, 21, 30), (20, 32, 32, 64, 128),
    (2, 128, 64, 128, 512), (5, 64, 128, 128, 200), (1, 160, 16, 200, 64),
    (2, 200, 96, 300, 600)])
@pytest.mark.parametrize("window", [0, 1, 37, 64])
def test_latent_attention(dev, dt, H, D, E, V, R, window):
    """Portions of every size beside single tokens, each sequence against the
    oracle alone."""
    lens, new = [150, 1, 67, 90, 130, 3], [150, 1, 1, 2, 35, 3]
    s = latent_spec(H, D, E, V, R, window=window)
    m = Latents(dev, dt, s, lens)
    m.write()
    qs = [rnd(t, H, D + E, seed=100 + i, scale=1.5) for i, t in enumerate(new)]
    starts = [n - t for n, t in zip(lens, new)]
    for i, o in enumerate(m.attend(qs, starts)):
        torch.testing.assert_close(o, m.want(i, qs[i], starts[i]), **ATOL[dt],
                                   msg=lambda t: f"seq {i}: {t}")


@kinds
@pytest.mark.parametrize("page", [8, 16, 32])
def test_latent_attention_pages_splits_and_gate(dev, dt, page):
    s = latent_spec(4, 32, 16, 48, 96, window=50)
    lens, new = [70, 120, 40], [30, 1, 2]
    m = Latents(dev, dt, s, lens, page=page)
    m.write()
    qs = [rnd(t, 4, 48, seed=i) for i, t in enumerate(new)]
    starts = [n - t for n, t in zip(lens, new)]
    gate = rnd(33, 4 * 48, seed=3, scale=2.0)
    got = torch.cat(m.attend(qs, starts, gate, splits=3))
    want = torch.cat([m.want(i, q, st) for i, (q, st) in enumerate(zip(qs, starts))])
    want = want * oracle.sigmoid(gate.double()).view(-1, 4, 48)
    torch.testing.assert_close(got, want, **ATOL[dt])


@kinds
@pytest.mark.parametrize("level", [-30.0, 0.0, 4.0, 30.0])
def test_sink(dev, dt, level):
    """From a sink that takes nothing to one that takes all; a scale far from
    one shows that the sink is not scaled. The first token, too."""
    s = latent_spec(3, 32, 16, 32, 64, scale=0.01, window=20)
    m = Latents(dev, dt, s, [90, 1, 40, 2])
    m.write()
    m.sink = torch.tensor([level, level + 1, -level])
    qs = [rnd(t, 3, 48, seed=t) for t in (40, 1, 1, 2)]
    starts = [50, 0, 39, 0]
    for i, o in enumerate(m.attend(qs, starts)):
        torch.testing.assert_close(o, m.want(i, qs[i], starts[i]), **ATOL[dt])


def loud_key(m, key):
    """Makes key `key` of sequence 0 stand out so far (for queries that are
    zero but for a turn-proof element) that its value is the output."""
    s = m.s
    m.uk[:, 0] = 0
    m.uk[::s.dim, 0] = 8.0           # latent element 0 -> key element 0
    m.c[0][:, 0] = 0
    m.c[0][key] = 0.25 * m.c[0][key]
    m.c[0][key, 0] = 8.0
    m.uv[:, 0] = 0
    m.sink[:] = -5


@kinds
@pytest.mark.parametrize("window", [16, 33, 40])
@pytest.mark.parametrize("decode", [False, True])
def test_window_edges(dev, dt, window, decode):
    """The last query that sees the loud key and the first that does not, for
    keys on, before and after page and tile borders."""
    H, D, E, V = 2, 32, 16, 32
    for key in (0, 15, 16, 31, 32, 63, 64):
        last = key + window - 1
        s = latent_spec(H, D, E, V, 64, scale=0.5, window=window)
        m = Latents(dev, dt, s, [last + 3], seed=key)
        loud_key(m, key)
        m.write()
        v = (m.c[0][key].double() @ m.uv.double().T).view(H, V)
        for pos, seen in ((last, True), (last + 1, False)):
            q = torch.zeros(1 if decode else 2, H, D + E)
            q[..., 0] = 8.0
            start = pos - (0 if decode else 1)
            o = m.attend([q], [start])[0][-1]
            close = (o - v).abs().max() < 0.02 * v.abs().max()
            assert bool(close) == seen, (key, pos)
            torch.testing.assert_close(o, m.want(0, q, start)[-1], **ATOL[dt])


@kinds
def test_far_key_and_far_rotation(dev, dt):
    """A key hundreds of tokens back, found by its latent and by its rotated
    part, in prompts and decoded tokens."""
    H, D, E, V, n = 3, 32, 16, 40, 700
    for key in (0, 3, 255, 256, 511):
        s = latent_spec(H, D, E, V, 80, scale=0.05)
        m = Latents(dev, dt, s, [n], seed=key, base=100.0)
        m.r[0][:] *= 0.2
        q = rnd(9, H, D + E, seed=key)
        # the query that turns onto the key's rotated part at its own position
        target = torch.zeros(n, E, dtype=torch.double)
        target[:, 1] = 12.0
        m.r[0][key] = target[0].float()
        back = oracle.rotate(target, 100.0, E)        # turned by +p
        back[:, E // 2:] *= -1                        # ... so this is by -p
        q[:, :, D:] = back[n - 9:, None].float()
        m.write()
        for new in (q, q[-1:]):
            st = n - new.shape[0]
            torch.testing.assert_close(m.attend([new], [st])[0],
                                       m.want(0, new, st), **ATOL[dt])


@kinds
def test_long_decode_splits(dev, dt):
    """Long contexts at a small batch: the visible range is split over
    workgroups and folded again, with the sink once."""
    lens = [1900, 333, 5]
    for window in (0, 1500):
        s = latent_spec(4, 64, 32, 64, 128, window=window)
        m = Latents(dev, dt, s, lens, uk=2.0)
        m.write()
        qs = [rnd(1, 4, 96, seed=i, scale=2.0) for i in range(3)]
        for i, o in enumerate(m.attend(qs, [n - 1 for n in lens])):
            torch.testing.assert_close(o, m.want(i, qs[i], lens[i] - 1), **ATOL[dt])


# ---------------------------------------------------------------------------
# gated linear attention
# ---------------------------------------------------------------------------

class Gla:
    """A recurrent layer's inputs for a step, given as projection outputs."""

    def __init__(self, dev, dt, H, D, V, r, tau, slots=6, eps=1e-3, seed=0,
                 bias=1.5):
        self.dev, self.dt = dev, dt
        s = self.s = GlaSpec(heads=H, dim=D, vdim=V, tau=tau, eps=eps)
        at = 0
        for name, n in (("q_off", H * D), ("k_off", H * D), ("v_off", H * V),
                        ("g_off", H * V)):
            setattr(s, name, at)
            at = round_up(at + n, 8)
        s.router_n, s.out_cols = r, round_up(H * V, 64) + 64
        self.cols = round_up(at, 64)
        self.a2 = rnd(H * D, r, seed=seed + 1, scale=1.5 * r ** -0.5)
        self.a2b = bias + rnd(H * D, seed=seed + 2)
        self.nw = 1 + rnd(V, seed=seed + 3, scale=0.3)
        self.cache = PagedKVCache(1, 0, 0, layout=["none"], max_tokens=4096,
                                  state_shapes=[(H, D, V)], max_seqs=slots,
                                  device=dev, dtype=dt)
        self.cache.state(0).fill_(float("nan"))       # what earlier owners left

    def inputs(self, n, seed):
        return rnd(n, self.cols, seed=seed), rnd(n, self.s.router_n, seed=seed + 1)

    def run(self, ys, a1s, starts, slots, splits=1):
        s = self.s
        counts = [y.shape[0] for y in ys]
        pages = [list(range(st + n)) for st, n in zip(starts, counts)]
        b = build_batch(self.cache, starts, counts, pages, slots)
        a = torch.zeros(1, b.n_tokens, s.router_n + 5)
        a[0, :, 5:] = torch.cat(a1s)
        out = mixers.gla_mix(
            as_parts(torch.cat(ys), self.dev, self.dt, splits), a.to(self.dev), 5,
            s, self.a2.t().contiguous().to(self.dev), self.a2b.to(self.dev),
            self.nw.to(self.dev), self.cache.state(0), b, self.dt)
        used = s.heads * s.vdim
        assert (out[:, used:] == 0).all()
        return list(out[:, :used].cpu().double().split(counts))

    def want(self, y, a1):
        """(output before W_o, last state) of a whole sequence."""
        s, T = self.s, y.shape[0]
        H, D, V = s.heads, s.dim, s.vdim
        y = y.double()
        cut = lambda off, d: y[:, off:off + H * d].reshape(T, H, d)
        z = a1.double() @ self.a2.double().T + self.a2b.double()
        a = torch.exp(torch.nn.functional.logsigmoid(z) / s.tau).view(T, H, D)
        o, S = oracle.recurrence(cut(s.q_off, D) * D ** -0.5, cut(s.k_off, D),
                                 cut(s.v_off, V), a)
        o = (oracle.rms(o, s.eps) * self.nw.double()).reshape(T, H * V)
        return o * oracle.silu(y[:, s.g_off:s.g_off + H * V]), S


GTOL = {torch.float32: dict(rtol=1e-4, atol=1e-4),
        torch.bfloat16: dict(rtol=3e-2, atol=3e-2)}


def state_close(got, want, dt):
    scale = want.abs().max()
    assert (got.cpu().double() - want).abs().max() < \
        (1e-5 if dt == torch.float32 else 3e-4) * scale


@kinds
@pytest.mark.parametrize("H,D,V,r,tau", [
    (3, 32, 48, 16, 16.0), (2, 18, 21, 5, 1.0), (1, 64, 64, 40, 4.0),
    (2, 128, 256, 16, 16.0), (2, 96, 100, 7, 8.0), (1, 256, 32, 3, 16.0),
    (1, 260, 30, 4, 2.0)])
def test_gla_portions(dev, dt, H, D, V, r, tau):
    """Whole prompts, portions around chunk borders, pairs and single tokens,
    three sequences side by side, on slots full of garbage."""
    m = Gla(dev, dt, H, D, V, r, tau)
    cuts = {4: [150], 0: [1, 2, 3, 5, 68, 69, 70, 134, 150],
            2: [63, 65, 128, 129, 149, 150]}
    data = {slot: m.inputs(150, seed=slot) for slot in cuts}
    got = {slot: [] for slot in cuts}
    at = dict.fromkeys(cuts, 0)
    for step in range(9):
        live = [slot for slot in cuts if step < len(cuts[slot])]
        ends = [cuts[slot][step] for slot in live]
        outs = m.run([data[s][0][at[s]:e] for s, e in zip(live, ends)],
                     [data[s][1][at[s]:e] for s, e in zip(live, ends)],
                     [at[s] for s in live], live)
        for s, e, o in zip(live, ends, outs):
            got[s].append(o)
            at[s] = e
    for slot in cuts:
        o, S = m.want(*data[slot])
        torch.testing.assert_close(torch.cat(got[slot]), o, **GTOL[dt],
                                   msg=lambda t: f"slot {slot}: {t}")
        state_close(m.cache.state(0)[slot], S, dt)
    assert torch.isnan(m.cache.state(0)[[1, 3, 5]]).all()    # nobody else's


@kinds
@pytest.mark.parametrize("bias,tau", [(-40.0, 1.0), (-6.0, 1.0), (-3.0, 0.5),
                                      (12.0, 1.0)])
def test_gla_decays(dev, dt, bias, tau):
    """From channels that forget within a token to ones that never do: no
    overflow, no lost tokens."""
    m = Gla(dev, dt, 2, 48, 40, 6, tau, bias=bias)
    m.a2b[::3] = 3.0                     # channels of very different memory
    y, a1 = m.inputs(140, seed=5)
    o, S = m.want(y, a1)
    got = m.run([y], [a1], [0], [1])[0]
    torch.testing.assert_close(got, o, **GTOL[dt])
    state_close(m.cache.state(0)[1], S, dt)


@kinds
def test_gla_remembers_a_far_token(dev, dt):
    """One loud key early, asked for hundreds of tokens later."""
    m = Gla(dev, dt, 1, 32, 32, 4, 16.0, bias=9.0)
    n, s = 400, m.s
    y, a1 = m.inputs(n, seed=2)
    a1 *= 0.1
    y[:, s.k_off:s.k_off + 32] *= 0.05
    y[3, s.k_off + 7] = 20.0
    y[n - 1, s.q_off:s.q_off + 32] = 0
    y[n - 1, s.q_off + 7] = 20.0
    o, _ = m.want(y, a1)
    v = y[3, s.v_off:s.v_off + 32].double()
    cos = torch.cosine_similarity(o[-1] / oracle.silu(
        y[-1, s.g_off:s.g_off + 32].double()) / m.nw.double(), v, 0)
    assert cos > 0.95                          # the oracle's answer is that token
    whole = m.run([y], [a1], [0], [0])[0]
    torch.testing.assert_close(whole, o, **GTOL[dt])
    part = m.run([y[:390]], [a1[:390]], [0], [3])[0]
    for t in range(390, n):
        part = m.run([y[t:t + 1]], [a1[t:t + 1]], [t], [3])[0]
    torch.testing.assert_close(part, o[-1:], **GTOL[dt])


@kinds
@pytest.mark.parametrize("splits", [1, 3])
def test_gla_splits(dev, dt, splits):
    m = Gla(dev, dt, 3, 24, 40, 5, 4.0)
    y, a1 = m.inputs(30, seed=8)
    a = m.run([y[:20], y[:1]], [a1[:20], a1[:1]], [0, 0], [0, 1], splits)[0]
    b = m.run([y[20:21], y[1:30]], [a1[20:21], a1[1:30]], [20, 1], [0, 1], splits)
    o, _ = m.want(y, a1)
    torch.testing.assert_close(torch.cat([a, b[0]]), o[:21], **GTOL[dt])
    torch.testing.assert_close(b[1], o[1:], **GTOL[dt])


@kinds
def test_empty_slots(dev, dt):
    """Rows at position -1 write nothing and disturb nobody."""
    m = Gla(dev, dt, 2, 32, 32, 4, 4.0)
    slots = DecodeSlots(m.cache, 4, 64)
    slots.fill([1], [0], [[0]], [2])
    y, a1 = m.inputs(4, seed=1)
    m.cache.state(0).fill_(5.0)
    out = mixers.gla_mix(
        as_parts(y, dev, dt, 1), a1[None].to(dev).contiguous(), 0, m.s,
        m.a2.t().contiguous().to(dev), m.a2b.to(dev), m.nw.to(dev),
        m.cache.state(0), slots.batch, dt)
    torch.testing.assert_close(out[0, :64].cpu().double(),
                               m.want(y[:1], a1[:1])[0][0], **GTOL[dt])
    assert (m.cache.state(0)[[0, 1, 3, 4, 5]] == 5).all()
    # attention: an empty slot's row is finite
    s = latent_spec(2, 32, 16, 32, 64)
    lat = Latents(dev, dt, s, [40])
    lat.write()
    slots = DecodeSlots(lat.cache, 4, 64)
    slots.fill([1], [39], lat.pages)
    q = rnd(4, 2, 48, seed=3)
    before = lat.cache.k_pages(0).clone()
    y = torch.zeros(4, 128)
    y[:, :96] = q.view(4, -1)
    out = mixers.latent_attention(
        as_parts(y, dev, dt, 1), s, lat.weights(),
        mixers.rotary_turns(lat.base, 16).to(dev), slots.batch,
        torch.full((4, 64), 40.0).to(dev, dt), lat.cache.k_pages(0), dt)
    torch.testing.assert_close(out[0, :64].cpu().double().view(2, 32),
                               lat.want(0, q[:1], 39)[0], **ATOL[dt])
    assert torch.equal(before, lat.cache.k_pages(0))
