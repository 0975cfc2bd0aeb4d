"""The Zatusun mechanisms one by one against the plain oracle: scaled embeddings,
products that take the residual's place, stretched rotations, differential
attention in chunks, latent attention with a rotation factor, recurrence that
writes what it forgets, routing over the chosen, clamped gated experts. CPU forms
run here, the HIP kernels under -m gpu."""
import math

import pytest
import torch

import zatusun_oracle as oracle
from bloombee_amd.kv.batch import DecodeSlots, build_batch
from bloombee_amd.kv.paged import PagedKVCache
from bloombee_amd.ops import mixers, ragged
from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.mixers import (DiffSpec, HgrnSpec, LatentSpec,
                                     LatentWeights, half_order)
from bloombee_amd.ops.ragged import (FfSpec, GluSpec, Pending, RopeSpec, Routing,
                                     pad_head, round_up)

GPU = pytest.mark.gpu
KINDS = [pytest.param("cpu", torch.float32, id="cpu-f32"),
         pytest.param("cuda:0", torch.float32, id="gpu-f32", marks=GPU),
         pytest.param("cuda:0", torch.bfloat16, id="gpu-bf16", marks=GPU)]
kinds = pytest.mark.parametrize("dev,dt", KINDS)


def tol(dt):
    return dict(rtol=2e-5, atol=2e-5) if dt == torch.float32 else \
        dict(rtol=2e-2, atol=2e-2)


ATOL = {torch.float32: dict(rtol=3e-5, atol=3e-5),
        torch.bfloat16: dict(rtol=4e-2, atol=4e-2)}


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
@pytest.mark.parametrize("scale,copies", [(7.5, 2), (1.0, 1), (0.25, 3)])
def test_embedding(dev, dt, scale, copies):
    table, pos = rnd(50, 37, seed=1).to(dt), rnd(20, 37, seed=2).to(dt)
    ids, at = torch.tensor([[3, 49, 0, 7]]), torch.tensor([[0, 19, 5, 6]])
    x = ragged.embed_rows(ids.to(dev), at.to(dev), table.to(dev), pos.to(dev),
                          scale=scale, copies=copies)
    want = table.float()[ids] * scale + pos.float()[at]
    assert x.dtype == torch.float32 and x.shape == (1, 4, 37 * copies)
    torch.testing.assert_close(x.cpu(), want.repeat(1, 1, copies))


@kinds
@pytest.mark.parametrize("W,cols,splits", [(96, 192, 1), (250, 512, 3),
                                           (45, 128, 2), (2304, 4608, 4)])
def test_a_product_takes_the_residuals_place(dev, dt, W, cols, splits):
    """The sum joins the rows beside it, and what is made of them replaces the
    residual; both live in the columns of one wider matrix."""
    N, eps = 5, 1e-3
    hidden = rnd(N, 2 * W + 3, seed=1, scale=2.0).to(dev)
    keep = hidden.clone()
    x, other = hidden[:, :W], hidden[:, W:2 * W]
    y = rnd(N, round_up(W, 64), seed=2)
    rows = ragged.join_rows(x, Pending(as_parts(y, dev, dt, splits)), other, cols,
                            dt)
    total = keep[:, :W].cpu() + y[:, :W]
    torch.testing.assert_close(x.cpu(), total, rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(rows[:, :W].cpu().float(), total, **tol(dt))
    assert torch.equal(rows[:, W:2 * W], other.to(dt))
    assert (rows[:, 2 * W:] == 0).all()
    z, b, w = rnd(N, round_up(W, 64), seed=3), rnd(W, seed=4), rnd(W, seed=5)
    h = ragged.residual_norm(
        x, Pending(as_parts(z, dev, dt, splits), bias=b.to(dev), keep=0.0),
        (1 + w).to(dev), 1, eps, round_up(W, 64), dt)
    new = z[:, :W] + b
    torch.testing.assert_close(x.cpu(), new, rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(h[:, :W].cpu().double(),
                               oracle.norm(new.double(), w.double(), eps), **tol(dt))
    assert (h[:, W:] == 0).all()
    assert torch.equal(hidden[:, W:], keep[:, W:])
    # nothing pending: the rows as they are
    rows = ragged.join_rows(x, None, other, cols, dt)
    assert torch.equal(rows[:, :W], x.to(dt))


@kinds
def test_wide_sums_stay_in_32_bits(dev, dt):
    """More rows than the weight stream takes: the product is not rounded."""
    x, w = rnd(70, 256, seed=1), rnd(128, 256, seed=2)
    y = ragged.linear_sums(x.to(dev, dt), w.to(dev, dt))
    assert y.dtype == torch.float32
    torch.testing.assert_close(y.sum(0).cpu().double(), x.double() @ w.double().T,
                               rtol=1e-5, atol=1e-4)


# ---------------------------------------------------------------------------
# rotations
# ---------------------------------------------------------------------------

YARN = [dict(factor=4.0, original=64, fast=16.0, slow=0.5),
        dict(factor=2.0, original=4096, fast=32.0, slow=1.0),
        dict(factor=8.0, original=16, fast=1.0, slow=1.0),
        dict(factor=1.0, original=100, fast=3.0, slow=2.0)]
BANDS = [dict(factor=8.0, low=1.0, high=4.0, original=64),
         dict(factor=3.0, low=0.5, high=20.0, original=512)]


@pytest.mark.parametrize("base,dims", [(1e4, 32), (5e5, 6), (100.0, 64), (1e6, 2)])
def test_stretched_frequencies(base, dims):
    plain = oracle.plain_frequencies(base, dims)
    seen = set()
    for s in YARN:
        f, factor = oracle.yarn({"base": base, "dims": dims, "scaling": s})
        turns, amp = mixers.yarn_turns(base, dims, **s)
        torch.testing.assert_close(turns * 2 * math.pi,
                                   torch.tensor(f, dtype=torch.double),
                                   rtol=1e-12, atol=0)
        assert amp == pytest.approx(factor)
        for a, b in zip(f, plain):
            seen.add("kept" if a == b else "divided"
                     if abs(a * s["factor"] / b - 1) < 1e-12 else "between")
    for s in BANDS:
        f, _ = oracle.banded({"base": base, "dims": dims, "scaling": s})
        torch.testing.assert_close(
            mixers.banded_turns(base, dims, **s) * 2 * math.pi,
            torch.tensor(f, dtype=torch.double), rtol=1e-12, atol=0)
    if dims == 32:
        assert seen == {"kept", "divided", "between"}


def test_pairs_side_by_side():
    """Rows in half_order turn by halves as the others do pair by pair."""
    for dims, size in ((8, 8), (6, 11), (2, 5)):
        x = torch.randn(9, 3, size, dtype=torch.double)
        turns = mixers.rotary_turns(50.0, dims)
        order = half_order(dims, size)
        assert sorted(order.tolist()) == list(range(size))
        got = ref.rotate_half(x[..., order], torch.arange(4, 13), turns, 1.25)
        want = oracle.rotate(x, oracle.plain_frequencies(50.0, dims), 1.25, 4)
        torch.testing.assert_close(got, want[..., order])


# ---------------------------------------------------------------------------
# differential attention
# ---------------------------------------------------------------------------

class Diff:
    """Sequences whose keys and values are in a paged cache, written by the
    projection step itself."""

    def __init__(self, dev, dt, H, G, D, V, lens, chunk=0, window=0, rot=None,
                 scale=None, lam=0.6, factor=0.7, eps=1e-4, seed=0, page=16,
                 base=1e4, amp=1.0):
        self.dev, self.dt, self.base = dev, dt, base
        r = RopeSpec(heads=H, kv_heads=G, maps=2, dim=D, vdim=V,
                     rot_dims=rot or D - D % 2, amp=amp)
        r.k_off = round_up(2 * H * D, 8)
        r.v_off = round_up(r.k_off + 2 * G * D, 8)
        self.r = r
        self.s = DiffSpec(r, scale or D ** -0.5, lam, factor, eps, window=window,
                          chunk=chunk, out_cols=round_up(H * V, 64) + 64)
        self.turns = mixers.rotary_turns(base, r.rot_dims)
        self.cols = round_up(r.v_off + G * V, 64)
        self.cache = PagedKVCache(
            1, G, 2 * r.dk, v_head_dim=pad_head(V), page_size=page,
            max_tokens=sum(round_up(n, page) for n in lens) + 4 * page,
            device=dev, dtype=dt)
        for t in self.cache.pools[0]:
            t.fill_(1e3)                     # stale values in every slot
        order = torch.randperm(self.cache.n_pages, generator=torch.Generator()
                               .manual_seed(seed)).tolist()
        # projections, pairs side by side
        self.q = [rnd(n, H, 2, D, seed=seed + 11 + i) for i, n in enumerate(lens)]
        self.k = [rnd(n, G, 2, D, seed=seed + 31 + i) for i, n in enumerate(lens)]
        self.v = [rnd(n, G, V, seed=seed + 51 + i) for i, n in enumerate(lens)]
        self.pages = []
        for n in lens:
            m = (n + page - 1) // page
            self.pages.append(order[:m])
            order = order[m:]

    def rows(self, i, a, b):
        r, order = self.r, half_order(self.r.rot_dims, self.r.dim)
        y = torch.full((b - a, self.cols), 7.0)
        put = lambda off, t: y[:, off:off + t[0].numel()].copy_(t.flatten(1))
        put(r.q_off, self.q[i][a:b][..., order])
        put(r.k_off, self.k[i][a:b][..., order])
        put(r.v_off, self.v[i][a:b])
        return y

    def step(self, spans, splits=1):
        """spans: sequence -> (a, b) new tokens, in order."""
        b = build_batch(self.cache, [a for a, _ in spans.values()],
                        [e - a for a, e in spans.values()],
                        [self.pages[i] for i in spans])
        y = torch.cat([self.rows(i, *ab) for i, ab in spans.items()])
        out = mixers.differential_attention(
            as_parts(y, self.dev, self.dt, splits), self.s,
            self.turns.to(self.dev), b, self.cache.k_pages(0),
            self.cache.v_pages(0), self.dt)
        used = self.r.heads * self.r.vdim
        assert (out[:, used:] == 0).all()
        parts = out[:, :used].cpu().double().view(-1, self.r.heads, self.r.vdim)
        return dict(zip(spans, parts.split([e - a for a, e in spans.values()])))

    def want(self, i, n=None):
        s, n = self.s, n or self.q[i].shape[0]
        f = oracle.plain_frequencies(self.base, self.r.rot_dims)
        turn = lambda t: oracle.rotate(t[:n].double(), f, self.r.amp)
        assert not s.window
        return oracle.differential(turn(self.q[i]), turn(self.k[i]),
                                   self.v[i][:n].double(), s.scale, s.chunk, s.lam,
                                   1 - s.factor, s.eps)


@kinds
@pytest.mark.parametrize("H,G,D,V,rot", [
    (4, 2, 32, 56, 12), (3, 3, 18, 21, 18), (6, 1, 24, 40, 12), (2, 1, 64, 32, 64),
    (4, 2, 128, 256, 64), (20, 2, 48, 96, 32), (9, 1, 16, 16, 2),
    (2, 2, 150, 64, 100), (1, 1, 33, 300, 6)])
@pytest.mark.parametrize("chunk", [0, 1, 37, 64])
def test_differential_attention(dev, dt, H, G, D, V, rot, chunk):
    """Portions of every size beside single tokens, each sequence against the
    oracle alone."""
    lens = [130, 1, 67, 90, 3]
    m = Diff(dev, dt, H, G, D, V, lens, chunk=chunk, rot=rot, lam=0.45)
    m.step({0: (0, 70), 2: (0, 66), 3: (0, 37)})
    a = m.step({0: (70, 129), 1: (0, 1), 2: (66, 67), 3: (37, 39), 4: (0, 3)})
    b = m.step({3: (39, 90), 0: (129, 130)})
    for i, part, at in ((0, a[0], 70), (1, a[1], 0), (2, a[2], 66), (3, a[3], 37),
                        (4, a[4], 0), (3, b[3], 39), (0, b[0], 129)):
        torch.testing.assert_close(part, m.want(i)[at:at + part.shape[0]],
                                   **ATOL[dt], msg=lambda t: f"seq {i}: {t}")


@kinds
@pytest.mark.parametrize("page", [8, 16, 32])
@pytest.mark.parametrize("splits", [1, 3])
def test_differential_pages_and_splits(dev, dt, page, splits):
    m = Diff(dev, dt, 4, 2, 32, 48, [70, 50], chunk=50, page=page, rot=10, amp=1.3)
    a = m.step({0: (0, 45), 1: (0, 1)}, splits)
    b = m.step({1: (1, 50), 0: (45, 46)}, splits)
    c = m.step({0: (46, 70)}, splits)
    torch.testing.assert_close(torch.cat([a[0], b[0], c[0]]), m.want(0), **ATOL[dt])
    torch.testing.assert_close(torch.cat([a[1], b[1]]), m.want(1), **ATOL[dt])


@kinds
@pytest.mark.parametrize("lam,factor,eps,scale", [
    (0.0, 1.0, 1e-5, 0.3), (1.0, 0.2, 1e-3, 0.1), (-0.7, 0.9, 0.5, 0.2),
    (1.4, 0.5, 1e-2, 0.02)])
def test_how_the_maps_combine(dev, dt, lam, factor, eps, scale):
    m = Diff(dev, dt, 4, 2, 32, 40, [80], lam=lam, factor=factor, eps=eps,
             scale=scale)
    got = torch.cat([m.step({0: (0, 77)})[0]]
                    + [m.step({0: (t, t + 1)})[0] for t in (77, 78, 79)])
    torch.testing.assert_close(got, m.want(0), **ATOL[dt])


@kinds
@pytest.mark.parametrize("chunk", [16, 33, 50, 64])
@pytest.mark.parametrize("decode", [False, True])
def test_chunk_edges(dev, dt, chunk, decode):
    """A key that outshouts all others is the answer to the end of its chunk and
    gone with the next token, wherever the prompt was cut, for chunk borders on,
    before and after those of pages and tiles."""
    for key in (0, chunk - 1, chunk, 2 * chunk - 2, 2 * chunk - 1):
        end = (key // chunk + 1) * chunk      # first position that does not see it
        m = Diff(dev, dt, 2, 1, 32, 32, [end + 2], chunk=chunk, lam=0.0,
                 factor=1.0, scale=0.5, rot=8, seed=key)
        m.q[0][..., 31] = 8.0
        m.k[0][..., 31] = 0.0
        m.k[0][key, :, :, 31] = 8.0
        if end - 1 > 0:
            m.step({0: (0, end - 1)})
        if decode:
            got = torch.cat([m.step({0: (t, t + 1)})[0]
                             for t in (end - 1, end, end + 1)])
        else:
            got = m.step({0: (end - 1, end + 2)})[0]
        v = oracle.rms(m.v[0][key, 0].double(), m.s.eps)
        close = [(o - v).abs().max() < 0.05 for o in got]
        assert close == [True, False, False], (key, close)
        torch.testing.assert_close(got, m.want(0)[end - 1:], **ATOL[dt])


@kinds
def test_far_key_of_one_map(dev, dt):
    """A key hundreds of tokens back that only the second map finds: its value
    comes with the opposite sign."""
    n = 700
    for key in (0, 3, 255, 511):
        m = Diff(dev, dt, 2, 1, 32, 32, [n], lam=0.9, scale=0.5, rot=6, seed=key)
        m.q[0] *= 0.2
        m.q[0][..., 31] = 9.0
        m.k[0][..., 31] = 0.0
        m.k[0][key, 0, 1, 31] = 9.0
        m.step({0: (0, n - 10)})
        got = torch.cat([m.step({0: (n - 10, n - 1)})[0],
                         m.step({0: (n - 1, n)})[0]])
        cos = torch.cosine_similarity(got, m.v[0][key, 0].double(), -1)
        assert (cos < -0.6).all()
        torch.testing.assert_close(got, m.want(0)[n - 10:], **ATOL[dt])


@kinds
def test_differential_long_decode(dev, dt):
    """Long contexts at a small batch: the visible range is split over workgroups
    and folded again, map by map."""
    for chunk in (0, 1500):
        m = Diff(dev, dt, 4, 2, 64, 128, [1900, 333, 5], chunk=chunk, rot=32)
        m.step({0: (0, 1899), 1: (0, 332), 2: (0, 4)})
        out = m.step({0: (1899, 1900), 1: (332, 333), 2: (4, 5)})
        for i in range(3):
            torch.testing.assert_close(out[i], m.want(i)[-1:], **ATOL[dt])


@kinds
def test_differential_empty_slots(dev, dt):
    """Rows at position -1 write nothing and disturb nobody."""
    m = Diff(dev, dt, 2, 1, 32, 32, [40])
    m.step({0: (0, 39)})
    before = [t.clone() for t in m.cache.pools[0]]
    slots = DecodeSlots(m.cache, 4, 64)
    slots.fill([1], [39], m.pages)
    y = torch.cat([m.rows(0, 39, 40)] + [rnd(3, m.cols, seed=3)])
    out = mixers.differential_attention(
        as_parts(y, dev, dt, 1), m.s, m.turns.to(dev), slots.batch,
        m.cache.k_pages(0), m.cache.v_pages(0), dt)
    torch.testing.assert_close(out[0, :64].cpu().double().view(2, 32),
                               m.want(0)[39], **ATOL[dt])
    changed = sum(int((a != b).any(-1).sum()) for a, b in zip(
        [m.cache.k_pages(0)], before[:1]))
    assert changed == 1


@kinds
@pytest.mark.parametrize("H,G,D,V", [(4, 2, 32, 32), (3, 1, 20, 24)])
@pytest.mark.parametrize("chunk,window", [(24, 0), (50, 17), (17, 50)])
def test_plain_attention_in_chunks(dev, dt, H, G, D, V, chunk, window):
    """The ragged families' attention takes chunks, too, beside a window."""
    n, dk = 90, pad_head(D)
    cache = PagedKVCache(1, G, dk, v_head_dim=pad_head(V), max_tokens=128,
                         device=dev, dtype=dt)
    k, v, q = rnd(n, G, D, seed=1), rnd(n, G, V, seed=2), rnd(n, H, D, seed=3)
    kp, vp = cache.k_pages(0), cache.v_pages(0)
    for p in range(n):
        kp[p // 16, :, p % 16, :D] = k[p].to(dev, dt)
        vp[p // 16, :, :V, p % 16] = v[p].to(dev, dt)
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = (j <= i) & (i // chunk == j // chunk)
    if window:
        seen &= i - j < window
    want = torch.stack([
        oracle.softmax((q[:, h].double() @ k[:, h * G // H].double().T * 0.3)
                       .masked_fill(~seen, -math.inf)) @ v[:, h * G // H].double()
        for h in range(H)], 1).flatten(1)
    got = []
    for a, e in ((0, 40), (40, 41), (41, 90)):
        b = build_batch(cache, [a], [e - a], [list(range(6))])
        out = torch.empty(e - a, H * V, dtype=dt, device=dev)
        qd = torch.zeros(e - a, H, dk)
        qd[..., :D] = q[a:e]
        ragged.attn_ragged(qd.to(dev, dt), kp, vp, b, out, D, V, 0.3, window,
                           chunk=chunk)
        got.append(out.cpu().double())
    torch.testing.assert_close(torch.cat(got), want, **ATOL[dt])


# ---------------------------------------------------------------------------
# latent attention with a factor on the rotated part
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("H,D,E,V,R", [(6, 32, 16, 80, 64), (3, 18, 6, 21, 30),
                                       (2, 64, 64, 128, 128)])
@pytest.mark.parametrize("amp", [1.0, 1.35])
def test_latent_rotation_factor(dev, dt, H, D, E, V, R, amp):
    """The rotated part of queries and keys is scaled, the rest is not, in
    prompts and in decoding; no window and no sink."""
    Q, n = 40, 75
    s = LatentSpec(heads=H, dim=D, rot=E, rot_dims=E, vdim=V, q_rank=Q, rank=R,
                   scale=0.6 * (D + E) ** -0.5, window=0, eps=1e-3, amp=amp)
    s.c_off, s.g_off = round_up(Q, 8), round_up(Q, 8) + round_up(R + E, 8)
    s.q_cols, s.out_cols = round_up(Q, 64), round_up(H * V, 64)
    turns = mixers.rotary_turns(500.0, E)
    freqs = oracle.plain_frequencies(500.0, E)
    y = rnd(n, round_up(s.g_off + H * V, 64), seed=1)
    qn, cn = 1 + rnd(Q, seed=2, scale=0.3), 1 + rnd(R, seed=3, scale=0.3)
    uk, uv = (rnd(H * d, R, seed=4, scale=R ** -0.5) for d in (D, V))
    uq = rnd(H * (D + E), Q, seed=6, scale=2 * Q ** -0.5)
    order = half_order(E, E)
    yd = y.double()
    cq = oracle.rms(yd[:, :Q], s.eps) * qn.double()
    c = oracle.rms(yd[:, s.c_off:s.c_off + R], s.eps) * cn.double()
    r = oracle.rotate(yd[:, s.c_off + R:s.c_off + R + E], freqs, amp)
    q = (cq @ uq.double().T).view(n, H, D + E)
    q = torch.cat([q[..., :D], oracle.rotate(q[..., D:], freqs, amp)], -1)
    k = torch.cat([(c @ uk.double().T).view(n, H, D),
                   r[:, None].expand(n, H, E)], -1)
    o = oracle.attend(q, k, (c @ uv.double().T).view(n, H, V), s.scale)
    want = o.flatten(1) * oracle.sigmoid(yd[:, s.g_off:s.g_off + H * V])

    ukt, uvp = torch.zeros(H, s.rp, round_up(D, 32)), torch.zeros(
        H, round_up(V, 64), s.rp)
    ukv = torch.zeros(round_up(H * (D + V), 64), s.ck)
    ukt[:, :R, :D] = uk.view(H, D, R).transpose(1, 2)
    uvp[:, :V, :R] = uv.view(H, V, R)
    ukv[:H * (D + V), :R] = torch.cat([uk, uv])
    w = LatentWeights(*(t.to(dev, dt) for t in (ukt, uvp, ukv)), None)
    uqp = torch.zeros(round_up(H * (D + E), 64), s.q_cols)
    uqh = uq.view(H, D + E, Q)
    uqp[:H * (D + E), :Q] = torch.cat([uqh[:, :D], uqh[:, D:][:, order]], 1
                                      ).reshape(-1, Q)
    yh = y.clone()
    yh[:, s.c_off + R:s.c_off + R + E] = \
        y[:, s.c_off + R:s.c_off + R + E][:, order]
    cache = PagedKVCache(1, 1, s.ck, layout=["k"], max_tokens=128, device=dev,
                         dtype=dt)
    got = []
    for a, e in ((0, 40), (40, 41), (41, 43), (43, 75)):
        b = build_batch(cache, [a], [e - a], [[3, 1, 0, 5, 2]])
        cqd, gate = mixers.latent_post(
            as_parts(yh[a:e], dev, dt, 1), s, qn.to(dev), cn.to(dev),
            turns.to(dev), b, cache.k_pages(0), dt)
        out = mixers.latent_attention(
            ragged.linear_parts(cqd, uqp.to(dev, dt)), s, w, turns.to(dev), b,
            gate, cache.k_pages(0), dt)
        got.append(out[:, :H * V].cpu().double())
    torch.testing.assert_close(torch.cat(got), want, **ATOL[dt])


# ---------------------------------------------------------------------------
# recurrence
# ---------------------------------------------------------------------------

class Hgrn:
    """A recurrent layer's inputs for a step, given as projection outputs."""

    def __init__(self, dev, dt, H, D, V, slots=6, eps=1e-3, seed=0, bias=2.0,
                 lower=None):
        self.dev, self.dt = dev, dt
        s = self.s = HgrnSpec(heads=H, dim=D, vdim=V, eps=eps, router_n=H * D)
        s.v_off = round_up(H * D, 8)
        s.out_cols = round_up(H * V, 64) + 64
        self.cols = round_up(s.v_off + H * V, 64)
        self.fb = bias + rnd(H * D, seed=seed + 1)
        g = torch.Generator().manual_seed(seed + 2)
        self.lower = (torch.rand(H * D, generator=g) if lower is None
                      else torch.full((H * D,), float(lower)))
        self.nw = 1 + rnd(V, seed=seed + 3, scale=0.3)
        self.cache = PagedKVCache(1, 0, 0, layout=["none"], max_tokens=4096,
                                  state_shapes=[(H, D, V)], max_seqs=slots,
                                  device=dev, dtype=dt)
        self.cache.state(0).fill_(float("nan"))       # what earlier owners left

    def inputs(self, n, seed):
        return (rnd(n, self.cols, seed=seed),
                rnd(n, self.s.heads * self.s.dim, seed=seed + 1))

    def run(self, ys, zs, starts, slots, splits=1, pad=8):
        s = self.s
        counts = [y.shape[0] for y in ys]
        pages = [list(range(st + n)) for st, n in zip(starts, counts)]
        b = build_batch(self.cache, starts, counts, pages, slots)
        z = torch.zeros(1, b.n_tokens, pad + round_up(s.router_n, 8))
        z[0, :, pad:pad + s.router_n] = torch.cat(zs)
        out = mixers.hgrn_mix(
            as_parts(torch.cat(ys), self.dev, self.dt, splits), z.to(self.dev),
            pad, s, self.fb.to(self.dev), self.lower.to(self.dev),
            self.nw.to(self.dev), self.cache.state(0), b, self.dt)
        used = s.heads * s.vdim
        assert (out[:, used:] == 0).all()
        return list(out[:, :used].cpu().double().split(counts))

    def want(self, y, z):
        """(output before W_o, last state) of a whole sequence."""
        s, T = self.s, y.shape[0]
        H, D, V = s.heads, s.dim, s.vdim
        y = y.double()
        q = oracle.silu(y[:, :H * D]).view(T, H, D)
        f = oracle.forget(z.double() + self.fb.double(), self.lower.double())
        o, S = oracle.scan(q, f.view(T, H, D),
                           y[:, s.v_off:s.v_off + H * V].reshape(T, H, V))
        return (oracle.rms(o, s.eps) * self.nw.double()).reshape(T, H * V), S


GTOL = {torch.float32: dict(rtol=1e-4, atol=1e-4),
        torch.bfloat16: dict(rtol=3e-2, atol=3e-2)}


def state_close(got, want, dt):
    scale = want.abs().max()
    assert (got.cpu().double() - want).abs().max() < \
        (1e-5 if dt == torch.float32 else 3e-4) * scale


@kinds
@pytest.mark.parametrize("H,D,V", [
    (2, 40, 56), (3, 32, 48), (2, 18, 21), (1, 64, 64), (2, 128, 256),
    (2, 96, 100), (1, 256, 32), (1, 260, 30), (1, 40, 400), (1, 128, 512),
    (5, 8, 530), (1, 200, 320)])
def test_recurrence_portions(dev, dt, H, D, V):
    """Whole prompts, portions around chunk borders, pairs and single tokens,
    three sequences side by side, on slots full of garbage."""
    m = Hgrn(dev, dt, H, D, V)
    cuts = {4: [150], 0: [1, 2, 3, 5, 68, 69, 70, 134, 150],
            2: [63, 65, 128, 129, 149, 150]}
    data = {slot: m.inputs(150, seed=slot) for slot in cuts}
    got, at = {slot: [] for slot in cuts}, dict.fromkeys(cuts, 0)
    for step in range(9):
        live = [slot for slot in cuts if step < len(cuts[slot])]
        ends = [cuts[slot][step] for slot in live]
        outs = m.run([data[s][0][at[s]:e] for s, e in zip(live, ends)],
                     [data[s][1][at[s]:e] for s, e in zip(live, ends)],
                     [at[s] for s in live], live, pad=5 if step % 2 else 0)
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
@pytest.mark.parametrize("bias,lower", [
    (-40.0, 0.0), (-6.0, 0.0), (-200.0, 0.0), (-2.0, 0.5), (12.0, 0.0),
    (0.0, 0.996), (-40.0, 0.9)])
def test_recurrence_gates(dev, dt, bias, lower):
    """From channels that forget within a token to ones that hardly ever do, and
    lower bounds that keep them from forgetting: no overflow, no lost tokens."""
    m = Hgrn(dev, dt, 2, 48, 40, bias=bias, lower=lower, eps=1e-6)
    m.fb[::3] = 3.0                      # channels of very different memory
    y, z = m.inputs(140, seed=5)
    o, S = m.want(y, z)
    assert torch.isfinite(o).all()
    torch.testing.assert_close(m.run([y], [z], [0], [1])[0], o, **GTOL[dt])
    state_close(m.cache.state(0)[1], S, dt)
    a = m.run([y[:100]], [z[:100]], [0], [3])[0]
    b = [m.run([y[t:t + 1]], [z[t:t + 1]], [t], [3])[0] for t in range(100, 140)]
    torch.testing.assert_close(torch.cat([a] + b), o, **GTOL[dt])


@kinds
def test_gates_that_jump(dev, dt):
    """A token that wipes a state that was kept for long, in the middle of a
    chunk, at its border and alone."""
    m = Hgrn(dev, dt, 1, 32, 32, bias=6.0, lower=0.0)
    y, z = m.inputs(200, seed=3)
    z *= 0.3
    for t in (20, 63, 64, 130, 190):
        z[t] = -30.0
    o, S = m.want(y, z)
    got = [m.run([y[:170]], [z[:170]], [0], [0])[0]]
    got += [m.run([y[t:t + 1]], [z[t:t + 1]], [t], [0])[0] for t in range(170, 200)]
    torch.testing.assert_close(torch.cat(got), o, **GTOL[dt])
    state_close(m.cache.state(0)[0], S, dt)


@kinds
def test_recurrence_remembers_a_far_token(dev, dt):
    """One token writes into a channel that then keeps everything out, and is
    asked for hundreds of tokens later."""
    m = Hgrn(dev, dt, 1, 32, 32, bias=0.0, lower=0.0)
    n, c = 400, 7
    y, z = m.inputs(n, seed=2)
    z[:, c] = 14.0
    z[3, c] = -14.0                           # ... but for this one
    y[n - 1, :32] = -30.0                     # silu: nothing
    y[n - 1, c] = 20.0
    o, _ = m.want(y, z)
    v = y[3, m.s.v_off:m.s.v_off + 32].double()
    assert torch.cosine_similarity(o[-1] / m.nw.double(), v, 0) > 0.99
    whole = m.run([y], [z], [0], [0])[0]
    torch.testing.assert_close(whole, o, **GTOL[dt])
    part = m.run([y[:390]], [z[:390]], [0], [3])[0]
    for t in range(390, n):
        part = m.run([y[t:t + 1]], [z[t:t + 1]], [t], [3])[0]
    torch.testing.assert_close(part, o[-1:], **GTOL[dt])


@kinds
@pytest.mark.parametrize("splits", [1, 3])
def test_recurrence_splits_and_empty_slots(dev, dt, splits):
    m = Hgrn(dev, dt, 3, 24, 40)
    y, z = m.inputs(30, seed=8)
    a = m.run([y[:20], y[:1]], [z[:20], z[:1]], [0, 0], [0, 1], splits)[0]
    b = m.run([y[20:21], y[1:30]], [z[20:21], z[1:30]], [20, 1], [0, 1], splits)
    o, _ = m.want(y, z)
    torch.testing.assert_close(torch.cat([a, b[0]]), o[:21], **GTOL[dt])
    torch.testing.assert_close(b[1], o[1:], **GTOL[dt])
    slots = DecodeSlots(m.cache, 4, 64)
    slots.fill([1], [0], [[0]], [2])
    m.cache.state(0).fill_(5.0)
    out = mixers.hgrn_mix(
        as_parts(y[:4], dev, dt, splits), z[None, :4].to(dev).contiguous(), 0, m.s,
        m.fb.to(dev), m.lower.to(dev), m.nw.to(dev), m.cache.state(0),
        slots.batch, dt)
    torch.testing.assert_close(out[0, :120].cpu().double(),
                               m.want(y[:1], z[:1])[0][0], **GTOL[dt])
    assert (m.cache.state(0)[[0, 1, 3, 4, 5]] == 5).all()


# ---------------------------------------------------------------------------
# experts
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("N,E,top,scale", [(5, 13, 4, 1.0), (40, 7, 7, 1.0),
                                           (33, 100, 1, 2.5), (3, 90, 70, 1.0)])
def test_routing_over_the_chosen(dev, dt, N, E, top, scale):
    """Weights are a softmax over the chosen logits alone, also where those are
    far below nothing."""
    K = 128
    h, w = rnd(N, K, seed=1), rnd(round_up(E, 64), K, seed=2, scale=0.5)
    h[1] *= 8
    rt = ragged.route(h.to(dev, dt), w.to(dev, dt),
                      FfSpec(router_off=0, router_n=E, top=top, renorm=True,
                             scale=scale))
    ids, share = oracle.choose(h.double() @ w[:E].double().T, top)
    assert all(len(set(row)) == top for row in rt.ids.tolist())
    full = lambda i, p: torch.zeros(N, E, dtype=torch.double).scatter(1, i, p)
    torch.testing.assert_close(
        full(rt.ids.cpu().long(), rt.wts.cpu().double()), full(ids, share * scale),
        rtol=1e-4, atol=1e-6)


@kinds
@pytest.mark.parametrize("N,E,top,F,W,limit", [
    (6, 5, 2, 64, 128, 0.8), (50, 11, 3, 40, 192, 1.25), (3, 4, 4, 200, 64, 7.0),
    (300, 3, 2, 96, 256, 0.3), (32, 6, 1, 256, 256, 2.0)])
def test_clamped_experts(dev, dt, N, E, top, F, W, limit):
    """Gates and ups on both sides of the limits, in the weight stream, the tiles
    and the plain kernel."""
    Fp = round_up(F, 64)
    h = rnd(N, W, seed=1)
    w = {}
    up, down = torch.zeros(E, 2, Fp, W), torch.zeros(E, W, Fp)
    for e in range(E):
        for i, n in enumerate(("gate", "up", "down")):
            t = rnd(*((F, W) if i < 2 else (W, F)), seed=10 * e + i,
                    scale=2 * (W if i < 2 else F) ** -0.5)
            w[f"e{e}.{n}"] = t.double()
            if i < 2:
                up[e, i, :F] = t
            else:
                down[e, :, :F] = t
    g = torch.Generator().manual_seed(3)
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(N)])
    wts = torch.rand(N, top, generator=g)
    y = ragged.moe_experts(h.to(dev, dt), up.to(dev, dt), down.to(dev, dt),
                           Routing(ids.int().to(dev), wts.to(dev), None),
                           act=GluSpec(limit, 1.702, 1.0))
    want = torch.stack([torch.stack([
        wts[t, k].double() * oracle.expert(h[t].double(), w, f"e{ids[t, k]}.", limit)
        for k in range(top)]) for t in range(N)])
    torch.testing.assert_close(y.cpu().double(), want, **ATOL[dt])
    if dt == torch.float32:
        wrong = oracle.expert(h[0].double(), w, f"e{ids[0, 0]}.", 10 * limit)
        right = want[0, 0] / wts[0, 0].double()
        assert limit > 3 or (wrong - right).abs().max() > 1e-2
