"""The Vumedra mechanisms one by one against the plain oracle: pair and position
embeddings, a norm around a sublayer, per-head projection step, attention with a
silent sink, matrix memory, gated linear recurrent unit, squared-relu experts.
CPU forms run here, the HIP kernels under -m gpu."""
import math

import pytest
import torch

import vumedra_oracle as oracle
from bloombee_amd.kv.batch import DecodeSlots, build_batch
from bloombee_amd.kv.paged import PagedKVCache
from bloombee_amd.ops import ragged, recurrent
from bloombee_amd.ops.ragged import (FfSpec, HeadSpec, PairTable, Pending,
                                     Routing, pad_head, round_up)
from bloombee_amd.ops.recurrent import MlstmSpec, RglruSpec, RglruWeights

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
    cut = rnd(splits, *y.shape, seed=9) * y.abs().mean(-1, keepdim=True)
    cut[-1] = y - cut[:-1].sum(0)
    return cut.to(dev).contiguous()


# ---------------------------------------------------------------------------
# embedding, norms
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("W,big", [
    (48, dict(buckets=31, mul_prev=7, mul_cur=3)),
    (33, dict(buckets=1, mul_prev=1, mul_cur=1)),
    # the hash leaves 32 bits
    (40, dict(buckets=1000003, mul_prev=2147483629, mul_cur=1500450271))])
def test_pair_and_position_embedding(dev, dt, W, big):
    """The first token's row, order within the pair, portions that continue, odd
    widths, positions far out."""
    V = 70
    table, pairs = rnd(V, W, seed=1), rnd(big["buckets"] + 1, W, seed=2)
    ids = torch.tensor([5, 69, 69, 0, 5, 0, 31])
    w = {"embed": table.double(), "bigram": pairs.double()}
    want = oracle.embed(ids, w, {"embedding": {"bigram": big}, "width": W})
    pt = PairTable(pairs.to(dev, dt), big["mul_prev"], big["mul_cur"])
    turns = ragged.sinusoid_turns(W).to(dev)
    for cuts in ([7], [1, 2, 5, 7], [3, 7]):
        at, last, out = 0, torch.tensor([-1]), []
        for c in cuts:
            part = ids[None, at:c]
            pos = torch.arange(at, c, dtype=torch.int32)[None]
            prev = ragged.previous_ids(part, last)
            out.append(ragged.embed_rows(part.to(dev), pos.to(dev),
                                         table.to(dev, dt), None, prev.to(dev),
                                         pt, turns)[0].cpu())
            at, last = c, part[:, -1]
        got = torch.cat(out)
        assert got.dtype == torch.float32
        torch.testing.assert_close(got.double(), want, rtol=1e-6, atol=2e-6)
    far = torch.tensor([0, 1, 999, 65537, 900001], dtype=torch.int32)
    got = ragged.embed_rows(torch.zeros(5, dtype=torch.int32).to(dev),
                            far.to(dev), torch.zeros(V, W, dtype=dt).to(dev),
                            None, turns=turns)
    want = torch.cat([oracle.sinusoid(int(p), 1, W) for p in far])
    torch.testing.assert_close(got.cpu().double(), want, rtol=1e-6, atol=2e-6)


@kinds
@pytest.mark.parametrize("W,cols,splits,top", [
    (96, 128, 1, 0), (250, 256, 3, 2), (2560, 2560, 4, 0), (4096, 4096, 1, 4),
    (192, 192, 0, 3)])
def test_norm_around_a_sublayer(dev, dt, W, cols, splits, top):
    """The sublayer's sum is normed, then added, then the next norm; eps shows
    in the small rows."""
    N, eps = 5, 1e-3
    x, y = rnd(N, W, seed=1, scale=2.0), rnd(N, round_up(W, 64), seed=2)
    routed = rnd(N, top, round_up(W, 64), seed=3)
    for t in (x, y, routed):
        t[1] *= 2.0 ** -10
    bw, w = rnd(W, seed=4, scale=0.2) + 0.7, rnd(W, seed=5, scale=0.2) + 1.3
    total = (y[:, :W].double() if splits else 0) + \
        routed[:, :, :W].double().sum(1)
    rt = Routing(torch.zeros(N, top, dtype=torch.int32, device=dev),
                 torch.ones(N, top, device=dev), None) if top else None
    pend = Pending(as_parts(y, dev, dt, splits) if splits else None,
                   routed.to(dev, dt) if top else None, rt, norm=bw.to(dev),
                   eps=eps)
    xd = x.clone().to(dev)
    h = ragged.residual_norm(xd, pend, w.to(dev), 1, eps, cols, dt)
    xw = x.double() + oracle.rms(total, eps) * bw.double()
    hw = oracle.rms(xw, eps) * w.double()
    assert xd.dtype == torch.float32
    torch.testing.assert_close(xd.cpu().double(), xw, rtol=1e-4, atol=1e-4)
    torch.testing.assert_close(h[:, :W].cpu().double(), hw, **tol(dt))
    assert (h[:, W:] == 0).all()
    xd = x.clone().to(dev)
    pend.settle(xd)
    torch.testing.assert_close(xd.cpu().double(), xw, rtol=1e-4, atol=1e-4)


# ---------------------------------------------------------------------------
# attention
# ---------------------------------------------------------------------------

class Attn:
    """A projection and its pages, several sequences."""

    def __init__(self, dev, dt, H, G, D, V, scale=None, coef=0.5, every=8,
                 eps=1e-3, seed=0, tokens=1024, page=16):
        self.dev, self.dt, self.scale = dev, dt, scale or D ** -0.5
        s = self.s = HeadSpec(heads=H, kv_heads=G, dim=D, vdim=V, eps=eps,
                              temp_coef=coef, temp_every=every)
        s.k_off = round_up(H * D, 8)
        s.v_off = round_up(s.k_off + G * D, 8)
        self.cols = round_up(s.v_off + G * V, 64)
        self.bias = [rnd(n, seed=seed + i, scale=0.5)
                     for i, n in enumerate((H * D, G * D, G * V))]
        self.qn = 1.5 + rnd(D, seed=seed + 5, scale=0.3)
        self.kn = 1.5 + rnd(D, seed=seed + 6, scale=0.3)
        self.cache = PagedKVCache(
            1, G, pad_head(D), v_head_dim=pad_head(V), layout="kv",
            page_size=page, max_tokens=tokens, device=dev, dtype=dt)
        for p in (self.cache.k_pages(0), self.cache.v_pages(0)):
            p.fill_(100.0)                  # what earlier owners left
        g = torch.Generator().manual_seed(seed)
        self.order = torch.randperm(self.cache.n_pages, generator=g).tolist()
        self.pages = {}

    def run(self, steps, splits=1):
        """steps: (name, rows, first position) -> outputs (T, H * V) each."""
        s, P = self.s, self.cache.page_size
        for name, y, at in steps:
            have = self.pages.setdefault(name, [])
            while len(have) * P < at + y.shape[0]:
                have.append(self.order.pop())
        b = build_batch(self.cache, [at for _, _, at in steps],
                        [y.shape[0] for _, y, _ in steps],
                        [self.pages[n] for n, _, _ in steps])
        d = lambda t: t.to(self.dev)
        kp, vp = self.cache.k_pages(0), self.cache.v_pages(0)
        q = ragged.head_post(
            as_parts(torch.cat([y for _, y, _ in steps]), self.dev, self.dt,
                     splits), s, [d(t) for t in self.bias], d(self.qn),
            d(self.kn), b, kp, vp, self.dt)
        self.q = q.cpu().double()[..., :s.dim]
        used = s.heads * s.vdim
        out = torch.zeros(b.n_tokens, round_up(used, 64), dtype=self.dt,
                          device=self.dev)
        ragged.attn_ragged(q, kp, vp, b, out, s.dim, s.vdim, self.scale,
                           sinks=torch.zeros(s.heads, device=self.dev))
        return list(out[:, :used].cpu().double().split(
            [y.shape[0] for _, y, _ in steps]))

    def parts(self, y):
        s, T = self.s, y.shape[0]
        y = y.double()
        cut = lambda off, n, d, b: (y[:, off:off + n * d] + b.double()).reshape(
            T, n, d)
        q = oracle.rms(cut(s.q_off, s.heads, s.dim, self.bias[0]), s.eps)
        k = oracle.rms(cut(s.k_off, s.kv_heads, s.dim, self.bias[1]), s.eps)
        return (q * self.qn.double(), k * self.kn.double(),
                cut(s.v_off, s.kv_heads, s.vdim, self.bias[2]))

    def want(self, y):
        s = self.s
        q, k, v = self.parts(y)
        q = q * oracle.temperature(y.shape[0], {
            "coef": s.temp_coef, "every": s.temp_every})[:, None, None]
        return oracle.attend(q, k, v, self.scale).reshape(y.shape[0], -1)


ATOL = {torch.float32: dict(rtol=2e-5, atol=2e-5),
        torch.bfloat16: dict(rtol=3e-2, atol=6e-2)}   # q and k are rounded
SIZES = [(6, 2, 48, 40), (5, 1, 96, 64), (3, 3, 18, 21), (8, 2, 32, 128),
         (4, 4, 128, 32), (24, 1, 64, 64), (2, 1, 200, 33), (2, 1, 300, 270)]


@kinds
@pytest.mark.parametrize("H,G,D,V", SIZES)
def test_attention(dev, dt, H, G, D, V):
    """Whole prompts, portions of unlike sizes and single tokens side by side."""
    m = Attn(dev, dt, H, G, D, V)
    n = {"a": 90, "b": 33, "c": 70}
    ys = {r: rnd(t, m.cols, seed=ord(r)) for r, t in n.items()}
    cuts = {"a": [90], "b": [1, 3, 16, 17, 33], "c": [48, 49, 50, 67, 70]}
    got, at = {r: [] for r in n}, dict.fromkeys(n, 0)
    for i in range(5):
        live = [r for r in n if i < len(cuts[r])]
        outs = m.run([(r, ys[r][at[r]:cuts[r][i]], at[r]) for r in live])
        for r, o in zip(live, outs):
            got[r].append(o)
            at[r] = cuts[r][i]
    for r in n:
        torch.testing.assert_close(torch.cat(got[r]), m.want(ys[r]), **ATOL[dt],
                                   msg=lambda t: f"{r}: {t}")


@kinds
@pytest.mark.parametrize("page,splits", [(8, 3), (32, 1), (16, 4)])
def test_attention_pages_and_splits(dev, dt, page, splits):
    m = Attn(dev, dt, 4, 2, 32, 48, page=page)
    y = rnd(60, m.cols, seed=2)
    o = [m.run([("a", y[:30], 0)], splits)[0], m.run([("a", y[30:31], 30)], splits)[0],
         m.run([("a", y[31:], 31)], splits)[0]]
    torch.testing.assert_close(torch.cat(o), m.want(y), **ATOL[dt])


@kinds
@pytest.mark.parametrize("level", [-12.0, -0.5, 0.5, 12.0])
def test_silent_sink(dev, dt, level):
    """All keys at one score: from a sink that takes almost everything to one
    that takes nothing, from the first token on."""
    m = Attn(dev, dt, 2, 1, 32, 32, coef=0.0, eps=1e-6)
    n = 70
    y = rnd(n, m.cols, seed=3)
    y[:, :m.s.v_off] = 0
    m.qn[:], m.kn[:] = 1, 1
    m.bias[0][:], m.bias[1][:] = 1, 1
    m.scale = level / 32
    o = m.run([("a", y[:60], 0)])[0]
    o = torch.cat([o] + [m.run([("a", y[t:t + 1], t)])[0] for t in range(60, n)])
    torch.testing.assert_close(o, m.want(y), **ATOL[dt])
    v = y[:, m.s.v_off:m.s.v_off + 32].double() + m.bias[2].double()
    c = torch.arange(1, n + 1, dtype=torch.double)[:, None]
    plain = v.cumsum(0) / (math.exp(-level) + c)
    torch.testing.assert_close(o[:, :32], plain, **ATOL[dt])


@kinds
@pytest.mark.parametrize("coef,every", [(0.5, 16), (2.0, 1), (-0.3, 7.5)])
def test_query_temperature_steps(dev, dt, coef, every):
    """The queries themselves, at positions around each step of the factor."""
    m = Attn(dev, dt, 2, 1, 32, 32, coef=coef, every=every)
    y = rnd(70, m.cols, seed=7)
    got = []
    for t0, t1 in [(0, 20)] + [(t, t + 1) for t in range(20, 70)]:
        m.run([("a", y[t0:t1], t0)])
        got.append(m.q)
    q = m.parts(y)[0]
    f = oracle.temperature(70, {"coef": coef, "every": every})[:, None, None]
    torch.testing.assert_close(torch.cat(got), q * f, **tol(dt))
    off = oracle.temperature(71, {"coef": coef, "every": every})[1:, None, None]
    assert (q * (off - f)).abs().max() > 0.1       # one position off is seen


@kinds
def test_far_key(dev, dt):
    """A loud key at page and tile borders, asked for hundreds of tokens
    later, in prompts and decoded."""
    for key in (0, 15, 16, 255, 256, 511):
        m = Attn(dev, dt, 3, 1, 64, 32, coef=0.0, scale=0.2, seed=key)
        n = 650
        y = rnd(n, m.cols, seed=key)
        for b in m.bias[:2]:
            b[:] = 0
        m.qn[:], m.kn[:] = 3, 3
        q, k = y[n - 3:, :3 * 64], y[:, m.s.k_off:m.s.k_off + 64]
        q.view(3, 3, 64)[:] = k[key]
        want = m.want(y)
        v = y[key, m.s.v_off:m.s.v_off + 32].double() + m.bias[2].double()
        assert (want[-1, :32] - v).abs().max() < 0.05
        a = m.run([("a", y[:n - 1], 0)])[0]
        b = m.run([("a", y[n - 1:], n - 1)])[0]
        torch.testing.assert_close(torch.cat([a, b])[-3:], want[-3:], **ATOL[dt])


@kinds
def test_long_context_decode(dev, dt):
    """The visible range is split over workgroups; the sink counts once."""
    m = Attn(dev, dt, 4, 2, 32, 32, scale=0.02, tokens=2048)
    y = rnd(1500, m.cols, seed=11)
    m.run([("a", y[:1499], 0)])
    torch.testing.assert_close(m.run([("a", y[1499:], 1499)])[0],
                               m.want(y)[-1:], **ATOL[dt])


# ---------------------------------------------------------------------------
# matrix memory
# ---------------------------------------------------------------------------

def cache_of_states(shapes, dev, dt, slots=6):
    c = PagedKVCache(1, 0, 0, layout=["none"], max_tokens=4096,
                     state_shapes=[shapes], max_seqs=slots, device=dev, dtype=dt)
    for t in c.state(0).values():
        t.fill_(float("nan"))               # what earlier owners left
    return c


def step_batch(cache, counts, starts, slots):
    pages = [list(range(st + n)) for st, n in zip(starts, counts)]
    return build_batch(cache, starts, counts, pages, slots)


class Memory:
    def __init__(self, dev, dt, H, D, V, cap=12.0, eps=1e-3, seed=0, bi=0.0,
                 bf=3.0):
        self.dev, self.dt = dev, dt
        s = self.s = MlstmSpec(heads=H, dim=D, vdim=V, cap=cap, eps=eps)
        at = 0
        for name, n in (("q_off", H * D), ("k_off", H * D), ("v_off", H * V),
                        ("g_off", H * V)):
            setattr(s, name, at)
            at = round_up(at + n, 8)
        s.router_n, s.out_cols = 2 * H, round_up(H * V, 64) + 64
        self.cols = round_up(at, 64)
        self.gb = torch.cat([bi + rnd(H, seed=seed + 1),
                             bf + rnd(H, seed=seed + 2)])
        self.nw = 1 + rnd(H * V, seed=seed + 3, scale=0.3)
        self.cache = cache_of_states(s.state_shapes(), dev, dt)

    def inputs(self, n, seed, spread=2.0):
        return (rnd(n, self.cols, seed=seed),
                rnd(n, 2 * self.s.heads, seed=seed + 1, scale=spread))

    def run(self, ys, gs, starts, slots, splits=1):
        s = self.s
        counts = [y.shape[0] for y in ys]
        b = step_batch(self.cache, counts, starts, slots)
        g = torch.zeros(1, b.n_tokens, s.router_n + 5)
        g[0, :, 5:] = torch.cat(gs)
        out = recurrent.mlstm_mix(
            as_parts(torch.cat(ys), self.dev, self.dt, splits), g.to(self.dev),
            5, s, self.gb.to(self.dev), self.nw.to(self.dev),
            self.cache.state(0), b, self.dt)
        used = s.heads * s.vdim
        assert (out[:, used:] == 0).all()
        return list(out[:, :used].cpu().double().split(counts))

    def want(self, y, g):
        """(output before W_o, last state) of a whole sequence."""
        s, T = self.s, y.shape[0]
        H, D, V = s.heads, s.dim, s.vdim
        y = y.double()
        cut = lambda off, d: y[:, off:off + H * d].reshape(T, H, d)
        z = oracle.capped(g.double() + self.gb.double(), s.cap)
        o, st = oracle.memory(cut(s.q_off, D) * D ** -0.5, cut(s.k_off, D),
                              cut(s.v_off, V), z[:, :H],
                              -oracle.softplus(-z[:, H:]))
        o = oracle.rms(o, s.eps).reshape(T, H * V) * self.nw.double()
        return o * oracle.sigmoid(y[:, s.g_off:s.g_off + H * V]), st

    def state_close(self, slot, want):
        for name, w in zip(("S", "n", "m"), want):
            got = self.cache.state(0)[name][slot].cpu().double()
            lim = 2e-5 if self.dt == torch.float32 else 4e-4
            assert (got - w).abs().max() < lim * max(1.0, float(w.abs().max())), name


GTOL = {torch.float32: dict(rtol=2e-4, atol=2e-4),
        torch.bfloat16: dict(rtol=3e-2, atol=3e-2)}


@kinds
@pytest.mark.parametrize("H,D,V,cap", [
    (3, 32, 48, 12.0), (2, 18, 21, 3.0), (1, 64, 64, 1.0), (2, 128, 256, 15.0),
    (2, 96, 100, 30.0), (1, 256, 32, 8.0), (1, 260, 30, 15.0), (1, 40, 400, 5.0),
    (5, 8, 530, 15.0), (2, 64, 63, 15.0)])
def test_memory_portions(dev, dt, H, D, V, cap):
    """Whole prompts, portions around chunk borders, pairs and single tokens,
    three sequences side by side, on slots full of garbage."""
    m = Memory(dev, dt, H, D, V, cap)
    cuts = {4: [150], 0: [1, 2, 3, 5, 68, 69, 70, 134, 150],
            2: [63, 65, 128, 129, 149, 150]}
    data = {slot: m.inputs(150, seed=slot) for slot in cuts}
    got, at = {slot: [] for slot in cuts}, dict.fromkeys(cuts, 0)
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
        o, st = m.want(*data[slot])
        torch.testing.assert_close(torch.cat(got[slot]), o, **GTOL[dt],
                                   msg=lambda t: f"slot {slot}: {t}")
        m.state_close(slot, st)
    for t in m.cache.state(0).values():
        assert torch.isnan(t[[1, 3, 5]]).all()       # nobody else's


@kinds
@pytest.mark.parametrize("bi,bf", [(-30.0, 30.0), (30.0, -30.0), (30.0, 30.0),
                                   (-30.0, -30.0), (-4.0, -1.0)])
def test_memory_gates(dev, dt, bi, bf):
    """Gates at and between the caps: no overflow and nothing lost, whether the
    maximum rises, falls or stays at its start, or the floor of the normalizer
    decides."""
    m = Memory(dev, dt, 2, 48, 40, cap=14.0, bi=bi, bf=bf)
    y, g = m.inputs(140, seed=5, spread=4.0)
    o, st = m.want(y, g)
    assert torch.isfinite(o).all()
    torch.testing.assert_close(m.run([y], [g], [0], [1])[0], o, **GTOL[dt])
    m.state_close(1, st)
    a = m.run([y[:100]], [g[:100]], [0], [3])[0]
    b = [m.run([y[t:t + 1]], [g[t:t + 1]], [t], [3])[0] for t in range(100, 140)]
    torch.testing.assert_close(torch.cat([a] + b), o, **GTOL[dt])


@kinds
def test_memory_normalizer_floor(dev, dt):
    """Keys and queries so small that exp(-m) is the divisor: with an eps that
    shows, the outputs' size depends on it."""
    m = Memory(dev, dt, 2, 32, 32, eps=1e-2, bi=-1.0, bf=2.0)
    y, g = m.inputs(90, seed=6, spread=1.0)
    y[:, :m.s.v_off] *= 0.125
    o, _ = m.want(y, g)
    torch.testing.assert_close(m.run([y], [g], [0], [0])[0], o, **GTOL[dt])
    got = [m.run([y[t:t + 1]], [g[t:t + 1]], [t], [2])[0] for t in range(90)]
    torch.testing.assert_close(torch.cat(got), o, **GTOL[dt])


@kinds
def test_memory_finds_a_far_token(dev, dt):
    """One loud key early, asked for hundreds of tokens later."""
    m = Memory(dev, dt, 1, 32, 32, bi=-2.0, bf=40.0)
    n, s = 400, m.s
    y, g = m.inputs(n, seed=2, spread=0.1)
    y[:, s.k_off:s.k_off + 32] *= 0.05
    y[3, s.k_off + 7] = 20.0
    y[n - 1, s.q_off:s.q_off + 32] = 0
    y[n - 1, s.q_off + 7] = 20.0
    o, _ = m.want(y, g)
    v = y[3, s.v_off:s.v_off + 32].double()
    cos = torch.cosine_similarity(o[-1] / oracle.sigmoid(
        y[-1, s.g_off:s.g_off + 32].double()) / m.nw.double(), v, 0)
    assert cos > 0.95                          # the oracle's answer is that token
    torch.testing.assert_close(m.run([y], [g], [0], [0])[0], o, **GTOL[dt])
    part = m.run([y[:390]], [g[:390]], [0], [3])[0]
    for t in range(390, n):
        part = m.run([y[t:t + 1]], [g[t:t + 1]], [t], [3])[0]
    torch.testing.assert_close(part, o[-1:], **GTOL[dt])


@kinds
@pytest.mark.parametrize("splits", [1, 3])
def test_memory_splits(dev, dt, splits):
    m = Memory(dev, dt, 3, 24, 40)
    y, g = m.inputs(30, seed=8)
    a = m.run([y[:20], y[:1]], [g[:20], g[:1]], [0, 0], [0, 1], splits)[0]
    b = m.run([y[20:21], y[1:30]], [g[20:21], g[1:30]], [20, 1], [0, 1], splits)
    o, _ = m.want(y, g)
    torch.testing.assert_close(torch.cat([a, b[0]]), o[:21], **GTOL[dt])
    torch.testing.assert_close(b[1], o[1:], **GTOL[dt])


# ---------------------------------------------------------------------------
# gated linear recurrent unit
# ---------------------------------------------------------------------------

class Unit:
    def __init__(self, dev, dt, W, B, K, seed=0, lam=None):
        self.dev, self.dt = dev, dt
        s = self.s = RglruSpec(width=W, blocks=B, taps=K)
        s.x_off = round_up(W, 8)
        self.cols, s.out_cols = round_up(s.x_off + W, 64), round_up(W, 64) + 64
        D = W // B
        self.w = dict(yb=rnd(W, seed=seed + 1, scale=0.3),
                      xb=rnd(W, seed=seed + 2, scale=0.3),
                      conv=rnd(W, K, seed=seed + 3, scale=0.6),
                      cb=rnd(W, seed=seed + 4, scale=0.3),
                      ra=rnd(B, D, D, seed=seed + 5, scale=D ** -0.5),
                      ri=rnd(B, D, D, seed=seed + 6, scale=D ** -0.5),
                      rab=rnd(B, D, seed=seed + 7), rib=rnd(B, D, seed=seed + 8),
                      lam=(-4 + rnd(W, seed=seed + 9, scale=2.0)) if lam is None
                      else torch.full((W,), lam))
        self.cache = cache_of_states(s.state_shapes(), dev, dt)

    def inputs(self, n, seed):
        return rnd(n, self.cols, seed=seed)

    def weights(self):
        s, w = self.s, self.w
        D, P = s.block, s.block_p
        gates = torch.zeros(s.blocks, 2, P, P)
        gates[:, 0, :D, :D], gates[:, 1, :D, :D] = w["ra"], w["ri"]
        d = lambda t: t.contiguous().to(self.dev)
        return RglruWeights(
            d(w["yb"]), d(w["xb"]), d(w["conv"].t()), d(w["cb"]),
            gates.to(self.dev, self.dt),
            d(torch.stack([w["rab"].flatten(), w["rib"].flatten()])),
            d(-8 * oracle.softplus(w["lam"].double()).float()))

    def run(self, ys, starts, slots, splits=1):
        s = self.s
        counts = [y.shape[0] for y in ys]
        b = step_batch(self.cache, counts, starts, slots)
        out = recurrent.rglru_mix(
            as_parts(torch.cat(ys), self.dev, self.dt, splits), s, self.weights(),
            self.cache.state(0), b, self.dt)
        assert (out[:, s.width:] == 0).all()
        return list(out[:, :s.width].cpu().double().split(counts))

    def want(self, y):
        """(output before W_o, last S, last inputs of the convolution)"""
        s, w = self.s, {k: v.double() for k, v in self.w.items()}
        y = y.double()
        branch = oracle.gelu(y[:, :s.width] + w["yb"])
        x = y[:, s.x_off:s.x_off + s.width] + w["xb"]
        u = oracle.causal_conv(x, w["conv"], w["cb"])
        S = oracle.unit(u, oracle.block_gate(u, w["ra"], w["rab"]),
                        oracle.block_gate(u, w["ri"], w["rib"]), w["lam"])
        past = torch.cat([x.new_zeros(s.taps - 1, s.width), x])
        return S * branch, S[-1], past[past.shape[0] - (s.taps - 1):]

    def state_close(self, slot, S, x):
        st = self.cache.state(0)
        lim = 2e-5 if self.dt == torch.float32 else 1e-2
        for got, want in ((st["S"][slot], S), (st["conv"][slot], x)):
            if want.numel():
                assert (got.cpu().double() - want).abs().max() < \
                    lim * max(1.0, float(want.abs().max()))


@kinds
@pytest.mark.parametrize("W,B,K", [
    (192, 4, 4), (96, 1, 1), (90, 3, 2), (256, 2, 7), (384, 6, 3), (64, 64, 4),
    (1024, 2, 4), (77, 7, 5)])
def test_unit_portions(dev, dt, W, B, K):
    """Whole prompts, portions around chunk borders and shorter than the
    convolution, pairs and single tokens, on slots full of garbage."""
    m = Unit(dev, dt, W, B, K)
    cuts = {4: [150], 0: [1, 2, 3, 5, 68, 69, 70, 134, 150],
            2: [2, 4, 63, 65, 128, 129, 149, 150], 1: [64, 128, 150]}
    data = {slot: m.inputs(150, seed=slot) for slot in cuts}
    got, at = {slot: [] for slot in cuts}, dict.fromkeys(cuts, 0)
    for step in range(9):
        live = [slot for slot in cuts if step < len(cuts[slot])]
        ends = [cuts[slot][step] for slot in live]
        outs = m.run([data[s][at[s]:e] for s, e in zip(live, ends)],
                     [at[s] for s in live], live)
        for s, e, o in zip(live, ends, outs):
            got[s].append(o)
            at[s] = e
    for slot in cuts:
        o, S, x = m.want(data[slot])
        torch.testing.assert_close(torch.cat(got[slot]), o, **GTOL[dt],
                                   msg=lambda t: f"slot {slot}: {t}")
        m.state_close(slot, S, x)
    for t in m.cache.state(0).values():
        assert torch.isnan(t[[3, 5]]).all()


@kinds
@pytest.mark.parametrize("lam", [-14.0, -6.0, 0.0, 6.0])
def test_unit_decays(dev, dt, lam):
    """From channels that never forget (where 1 - a^2 must not cancel) to ones
    that forget within a token."""
    m = Unit(dev, dt, 64, 2, 3, lam=lam)
    y = m.inputs(140, seed=5)
    o, S, x = m.want(y)
    tight = dict(rtol=3e-2, atol=3e-2 * float(o.abs().max())) \
        if dt == torch.bfloat16 else dict(rtol=2e-4,
                                          atol=2e-5 * float(o.abs().max()))
    torch.testing.assert_close(m.run([y], [0], [1])[0], o, **tight)
    a = [m.run([y[t:t + 1]], [t], [2])[0] for t in range(70)]
    a.append(m.run([y[70:]], [70], [2])[0])
    torch.testing.assert_close(torch.cat(a), o, **tight)


@kinds
def test_unit_remembers_a_far_token(dev, dt):
    """A loud input early in channels that do not forget."""
    m = Unit(dev, dt, 64, 1, 2, lam=-14.0)
    for n in ("xb", "cb", "ra", "ri"):
        m.w[n][:] = 0
    m.w["rib"][:] = 2
    y = m.inputs(400, seed=3)
    y[:, m.s.x_off:] *= 0.125
    y[3, m.s.x_off:m.s.x_off + 64] = 60.0
    o = m.want(y)[0]
    quiet = y.clone()
    quiet[3, m.s.x_off:m.s.x_off + 64] = 0
    assert (m.want(quiet)[0][-1] - o[-1]).abs().max() > 0.5 * o[-1].abs().max()
    lim = dict(rtol=3e-2, atol=2e-2 * float(o[-1].abs().max())) \
        if dt == torch.bfloat16 else GTOL[dt]
    torch.testing.assert_close(m.run([y], [0], [0])[0][-1], o[-1], **lim)
    m.run([y[:395]], [0], [3])
    for t in range(395, 400):
        last = m.run([y[t:t + 1]], [t], [3])[0]
    torch.testing.assert_close(last[0], o[-1], **lim)


@kinds
@pytest.mark.parametrize("splits", [1, 3])
def test_unit_splits(dev, dt, splits):
    m = Unit(dev, dt, 96, 2, 4)
    y = m.inputs(30, seed=8)
    a = m.run([y[:20], y[:1]], [0, 0], [0, 1], splits)[0]
    b = m.run([y[20:21], y[1:30]], [20, 1], [0, 1], splits)
    o = m.want(y)[0]
    torch.testing.assert_close(torch.cat([a, b[0]]), o[:21], **GTOL[dt])
    torch.testing.assert_close(b[1], o[1:], **GTOL[dt])


@kinds
def test_unit_many_decoded_rows(dev, dt):
    """More single tokens than one tile of rows, slots in no order."""
    m = Unit(dev, dt, 128, 2, 4)
    m.cache = cache_of_states(m.s.state_shapes(), dev, dt, slots=150)
    slots = torch.randperm(150, generator=torch.Generator().manual_seed(0))[:133]
    slots = slots.tolist()
    ys = [m.inputs(5, seed=i) for i in range(133)]
    m.run([y[:3] for y in ys], [0] * 133, slots)
    m.run([y[3:4] for y in ys], [3] * 133, slots)
    got = m.run([y[4:] for y in ys], [4] * 133, slots)
    for y, o in zip(ys, got):
        torch.testing.assert_close(o, m.want(y)[0][4:], **GTOL[dt])


@kinds
def test_empty_slots(dev, dt):
    """Rows at position -1 write nothing and disturb nobody."""
    m, u = Memory(dev, dt, 2, 32, 32), Unit(dev, dt, 64, 2, 3)
    for o in (m, u):
        for t in o.cache.state(0).values():
            t.fill_(5.0)
        slots = DecodeSlots(o.cache, 4, 64)
        slots.fill([1], [0], [[0]], [2])
        if o is m:
            y, g = m.inputs(4, seed=1)
            out = recurrent.mlstm_mix(
                as_parts(y, dev, dt, 1), g[None].to(dev).contiguous(), 0, m.s,
                m.gb.to(dev), m.nw.to(dev), m.cache.state(0), slots.batch, dt)
            want = m.want(y[:1], g[:1])[0]
        else:
            y = u.inputs(4, seed=1)
            out = recurrent.rglru_mix(as_parts(y, dev, dt, 1), u.s, u.weights(),
                                      u.cache.state(0), slots.batch, dt)
            want = u.want(y[:1])[0]
        torch.testing.assert_close(out[:1, :64].cpu().double(), want, **GTOL[dt])
        for t in o.cache.state(0).values():
            assert (t[[0, 1, 3, 4, 5]] == 5).all()


# ---------------------------------------------------------------------------
# feed-forwards
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("act", [0, 1, 2])
@pytest.mark.parametrize("ff,splits,E,top", [(320, 1, 8, 1), (77, 3, 5, 5),
                                             (128, 2, 70, 3)])
def test_activation_and_router(dev, dt, act, ff, splits, E, top):
    N, up = 6, round_up(ff, 8)
    s = FfSpec(act=act, ff=ff if act else 0, gate_off=0, up_off=up,
               cols=round_up(ff, 64) + 64 if act else 0, router_n=E, top=top,
               sigmoid=True)
    y = rnd(N, round_up(up + ff, 64), seed=1, scale=2.0)
    z = rnd(1, N, E + 3, seed=2, scale=3.0)
    z[0, 0, 3:] = z[0, 0, 3]                      # ties: the lowest index wins
    a, rt = ragged.ff_post(as_parts(y, dev, dt, splits) if act else None,
                           z.to(dev), 3, s, None, N, dev, dt)
    if act:
        u = y[:, up:up + ff].double()
        g = y[:, :ff].double()
        want = g * oracle.sigmoid(g) * u if act == 1 else torch.relu(u) ** 2
        torch.testing.assert_close(a[:, :ff].cpu().double(), want, **tol(dt))
        assert (a[:, ff:] == 0).all()
    sc = oracle.sigmoid(z[0, :, 3:].double())
    ids = rt.ids.cpu().long()
    assert ids[0].tolist() == list(range(top))
    torch.testing.assert_close(rt.wts.cpu().double(), sc.gather(1, ids),
                               rtol=1e-5, atol=1e-6)
    best = torch.topk(sc, top, -1).values
    torch.testing.assert_close(sc.gather(1, ids).sort(-1, descending=True).values,
                               best)


@kinds
@pytest.mark.parametrize("N,E,top,W,ff", [(1, 8, 1, 96, 96), (5, 6, 3, 128, 40),
                                          (70, 9, 2, 200, 130),
                                          (300, 4, 4, 64, 64)])
def test_experts_weighted_on_their_input(dev, dt, N, E, top, W, ff):
    """Under a square, a weight on the input is not a weight on the output."""
    K, F, Wp = round_up(W, 64), round_up(ff, 64), round_up(W, 64)
    w = {}
    up, down = torch.zeros(E, 1, F, K), torch.zeros(E, Wp, F)
    for e in range(E):
        w[f"e{e}.up"] = rnd(ff, W, seed=e, scale=W ** -0.5).double()
        w[f"e{e}.down"] = rnd(W, ff, seed=50 + e, scale=ff ** -0.5).double()
        up[e, 0, :ff, :W], down[e, :W, :ff] = w[f"e{e}.up"], w[f"e{e}.down"]
    w["router"] = rnd(E, W, seed=99, scale=2 * W ** -0.5).double()
    h = rnd(N, W, seed=7)
    sc = oracle.sigmoid(h.double() @ w["router"].T)
    best = torch.topk(sc, top, -1)
    rt = Routing(best.indices.int().to(dev), best.values.float().to(dev), None)
    hp = torch.zeros(N, K)
    hp[:, :W] = h
    y = ragged.moe_experts(hp.to(dev, dt), up.to(dev, dt), down.to(dev, dt), rt,
                           weight_input=True)
    got = y[:, :, :W].float().sum(1).cpu().double()
    want = oracle.moe(h.double(), w, "", {"router": {"top": top}})
    t = dict(rtol=1e-4, atol=1e-4) if dt == torch.float32 else \
        dict(rtol=3e-2, atol=3e-2)
    torch.testing.assert_close(got, want, **t)
