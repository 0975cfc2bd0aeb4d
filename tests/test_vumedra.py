"""Vumedra models end to end: engine, cache and state slots, scheduler, trace
replay and swarm against the plain oracle, on small random models of several
shapes. CPU forms run here, the HIP kernels under -m gpu."""
import copy
import io
import json
import os

import pytest
import torch
from safetensors.torch import save_file

import vumedra_oracle as oracle
from bloombee_amd.engine import BlockStack, LocalEngine
from bloombee_amd.kv.paged import AllocationFailed, PagedKVError
from bloombee_amd.models.base import resolve_config
from bloombee_amd.models.vumedra import VumedraConfig
from bloombee_amd.scheduler import BatchScheduler

GPU = pytest.mark.gpu
KINDS = [pytest.param("cpu", "float32", id="cpu-f32"),
         pytest.param("cuda:0", "float32", id="gpu-f32", marks=GPU),
         pytest.param("cuda:0", "bfloat16", id="gpu-bf16", marks=GPU)]
kinds = pytest.mark.parametrize("dev,dt", KINDS)


def attention(heads, kv_heads, dim, vdim, scale=None, coef=0.5, every=16):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "scale": scale or dim ** -0.5}
    if coef is not None:
        m["q_temp"] = {"coef": coef, "every": every}
    return "attention", m


def mlstm(heads, dim, vdim, cap=15.0):
    return "mlstm", {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def rglru(width, blocks, conv):
    return "rglru", {"width": width, "blocks": blocks, "conv": conv}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    f = {"kind": "moe", "router": {"experts": experts, "top": top},
         "expert": {"ff": ff}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def model(width, vocab, layers, eps=1e-5, buckets=211, prev=19, cur=5):
    return {"architecture": "Vumedra", "width": width, "vocab": vocab,
            "norm": {"eps": eps},
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": prev,
                                     "mul_cur": cur}},
            "layers": [{"type": t, "mixer": m, "mlp": f}
                       for (t, m), f in layers]}


CONFIGS = {
    # all mechanisms, unlike sizes everywhere
    "full": model(192, 333, [
        (rglru(160, 5, 3), dense(200)),
        (mlstm(3, 32, 48), moe(7, 3, 72, 136)),
        (attention(6, 2, 48, 40), moe(5, 2, 64)),
        (mlstm(5, 24, 40, cap=4.0), None),
        (attention(4, 4, 32, 64, scale=0.3, coef=1.5, every=7), dense(96)),
        (rglru(256, 2, 6), moe(6, 1, 40, 48))]),
    # sizes that are no multiple of four, as few parts as there can be
    "odd": model(90, 101, [
        (attention(5, 1, 18, 21, coef=None), dense(77)),
        (mlstm(3, 18, 21, cap=1.5), moe(3, 3, 50, 30)),
        (rglru(77, 7, 1), None),
        (rglru(45, 1, 2), dense(31))], eps=1e-3, buckets=1, prev=3, cur=0),
    # the largest compiled sizes
    "wide": model(320, 517, [
        (attention(20, 4, 128, 128, coef=-0.2, every=1), dense(512)),
        (mlstm(2, 256, 128), None), (rglru(512, 2, 4), dense(320)),
        (mlstm(1, 128, 320, cap=30.0), moe(16, 4, 64, 64)),
        (attention(2, 1, 96, 256), None)], buckets=100003, prev=70001, cur=3001),
    # no recurrence
    "attentions": model(128, 97, [
        (attention(4, 2, 32, 32), None), (attention(4, 1, 32, 64), moe(4, 2, 32))]),
    # recurrence only
    "recurrent": model(128, 97, [(mlstm(2, 32, 64), dense(128)),
                                 (rglru(128, 4, 4), None)]),
}


def save(cfg, folder, weights):
    (folder / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.bfloat16() for k, v in weights.items()},
              str(folder / "model.safetensors"))
    return str(folder)


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (checkpoint folder, float64 weights, config)"""
    out = {}
    for i, (name, cfg) in enumerate(CONFIGS.items()):
        w = oracle.random_weights(cfg, seed=10 + i)
        out[name] = (save(cfg, tmp_path_factory.mktemp(name), w),
                     {k: v.double() for k, v in w.items()}, cfg)
    return out


def dirty(eng):
    """What earlier owners left."""
    for t in eng.kv_pool.states:
        for s in (t or {}).values():
            s.fill_(float("nan"))
    return eng


def engine(models, name, dev, dt, monkeypatch, tokens=1024, seqs=48):
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    return dirty(LocalEngine(models[name][0], device=dev, kv_max_tokens=tokens,
                             max_seqs=seqs))


def prompt(cfg, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def want_logits(models, name, toks):
    _, w, cfg = models[name]
    return oracle.forward(torch.tensor(toks), w, cfg)


def check(got, want, dt, what="", limit=None):
    """Root mean square over the vocabulary, mean taken off, against the
    spread of the logits. In 16 bits a close call of a router shows as a larger
    error at that position."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.std()
    if dt == "float32":
        assert err.max() < (limit or 5e-5), (what, err.max().item(),
                                             int(err.argmax()))
        return
    assert err.median() < 0.04, (what, err.median().item())
    # of few rows each may be one
    n = err.numel()
    assert (err < 0.1).sum() >= n - max(1, n // 5), (what, err.max().item())


def run(eng, toks, cuts):
    """All logits of one request fed in portions that end at `cuts`."""
    h = eng.kv_pool.open_elastic(eng.config.max_position_embeddings)
    out, at = [], 0
    for c in cuts:
        out.append(eng.step([(h, toks[at:c], list(range(c - at)))]).cpu())
        at = c
    h.close()
    return torch.cat(out)


# ---------------------------------------------------------------------------
# one request
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt(models, name, dev, dt, monkeypatch):
    eng = engine(models, name, dev, dt, monkeypatch)
    for n in (1, 2, 23, 130):
        toks = prompt(CONFIGS[name], n, seed=n)
        check(run(eng, toks, [n]), want_logits(models, name, toks), dt, n)
    assert eng.kv_pool.free_page_count() == eng.kv_pool.n_pages


@kinds
@pytest.mark.parametrize("name", list(CONFIGS))
def test_token_by_token(models, name, dev, dt, monkeypatch):
    """Decoding from the first token on."""
    eng = engine(models, name, dev, dt, monkeypatch)
    n = 120
    toks = prompt(CONFIGS[name], n, seed=3)
    check(run(eng, toks, list(range(1, n + 1))),
          want_logits(models, name, toks), dt)


@kinds
@pytest.mark.parametrize("size", [2, 3, 7, 16, 31, 50, 65])
def test_portions(models, size, dev, dt, monkeypatch):
    eng = engine(models, "full", dev, dt, monkeypatch)
    n = 131
    toks = prompt(CONFIGS["full"], n, seed=4)
    cuts = list(range(size, n, size)) + [n]
    check(run(eng, toks, cuts), want_logits(models, "full", toks), dt)


@kinds
def test_long_decoding(models, dev, dt, monkeypatch):
    eng = engine(models, "recurrent", dev, dt, monkeypatch)
    n = 600
    toks = prompt(CONFIGS["recurrent"], n, seed=5)
    check(run(eng, toks, [64] + list(range(65, n + 1))),
          want_logits(models, "recurrent", toks), dt, limit=2e-4)


@kinds
def test_residual_after_every_layer(models, dev, dt, monkeypatch):
    from bloombee_amd.kv.batch import session_batch
    eng = engine(models, "full", dev, dt, monkeypatch)
    toks = prompt(CONFIGS["full"], 40)
    _, w, cfg = models["full"]
    want = oracle.hidden_states(torch.tensor(toks), w, cfg)
    h = eng.kv_pool.open_elastic(64)
    h.extend(40)
    b = session_batch([(h, 40)])
    ids = torch.tensor(toks, device=dev)
    prev = torch.tensor([-1] + toks[:-1], device=dev)
    x = eng.head.embed(ids, b.tok_pos, prev)
    left = None
    for i, blk in enumerate(eng.stack.blocks):
        left = blk.forward_tokens(x, left, b)
        assert x.dtype == torch.float32
        full = x.clone()
        left.settle(full)
        err = (full.cpu() - want[i]).abs().amax(-1) / want[i].abs().max()
        if dt == "float32":
            assert err.max() < 1e-4, i
        else:
            assert err.median() < 0.03, i


@kinds
@pytest.mark.parametrize("change", [
    "sink", "temperature", "cap", "normalizer floor", "first pair",
    "decay", "weight on the output", "inner norm"])
def test_the_tests_can_see(tmp_path, change, dev, dt, monkeypatch):
    """An oracle with one planted mistake differs visibly, the engine does
    not."""
    cfg = model(128, 97, [
        (attention(4, 2, 32, 32, coef=1.0, every=9), None),
        (mlstm(2, 32, 48, cap=3.0), moe(4, 2, 64, 64)),
        (rglru(128, 4, 3), dense(96))],
        eps=0.2)        # else a norm hides the size of the memory's output
    w = oracle.random_weights(cfg, 5)
    wd = {k: v.double() for k, v in w.items()}
    path = save(cfg, tmp_path, w)
    toks = torch.tensor(prompt(cfg, 60, 6))
    want = oracle.forward(toks, wd, cfg)
    off, wo = copy.deepcopy(cfg), dict(wd)
    with monkeypatch.context() as mp:
        if change == "sink":
            mp.setattr(oracle, "sink_softmax", lambda s: torch.softmax(s, -1))
        elif change == "temperature":
            off["layers"][0]["mixer"]["q_temp"]["every"] = 30
        elif change == "cap":
            off["layers"][1]["mixer"]["gate_cap"] = 6.0
        elif change == "normalizer floor":
            # all input gates raised alike lower it
            plain = oracle.memory
            mp.setattr(oracle, "memory", lambda q, k, v, i, f: plain(
                q, k, v, i + 2, f))
        elif change == "first pair":
            wo["bigram"] = torch.cat([wd["bigram"][:-1], wd["bigram"][:1]])
        elif change == "decay":
            wo["l2.mix.lam"] = wd["l2.mix.lam"] + 1.5
        elif change == "weight on the output":
            def late(h, w, pre, mlp):
                b = torch.topk(oracle.sigmoid(h @ w[pre + "router"].T), 2, -1)
                y = oracle.expert(h, w, pre + "shared.")
                for t in range(h.shape[0]):
                    for e, p in zip(b.indices[t].tolist(), b.values[t]):
                        y[t] += p * oracle.expert(h[t], w, f"{pre}e{e}.")
                return y
            mp.setattr(oracle, "moe", late)
        else:
            wo["l1.norm1b"] = wd["l1.norm1b"] * 1.5
        wrong = oracle.forward(toks, wo, off)
    d = (wrong - want).pow(2).mean(-1).sqrt() / want.std()
    if change == "first pair":
        assert d[0] > 0.1
    else:
        assert (d > 0.02).float().mean() > 0.02, d.max()
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    eng = dirty(LocalEngine(path, device=dev, kv_max_tokens=128))
    toks = toks.tolist()
    check(run(eng, toks, [60]), want, dt)
    check(run(eng, toks, [30] + list(range(31, 61))), want, dt)


# ---------------------------------------------------------------------------
# batches
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("name", ["full", "odd", "recurrent"])
def test_mixed_batch(models, name, dev, dt, monkeypatch):
    """Unequal requests, portions beside decoded tokens, requests that pause,
    pages and state slots that change hands: every logit as if the request ran
    alone."""
    cfg = CONFIGS[name]
    eng = engine(models, name, dev, dt, monkeypatch, tokens=320, seqs=3)
    for p in eng.kv_pool.pools:
        for t in p or ():
            t.fill_(1e3)                 # what earlier owners left
    lens = {"a": 97, "b": 30, "c": 64, "d": 5, "e": 81, "f": 16}
    toks = {r: prompt(cfg, n, seed=ord(r)) for r, n in lens.items()}
    want = {r: want_logits(models, name, t) for r, t in toks.items()}
    plan = [{"a": 64, "b": 29}, {"a": 1, "b": 1, "c": 17}, {"c": 2, "d": 2},
            {"a": 30, "c": 1, "d": 1}, {"d": 2, "c": 1, "a": 2},
            {"e": 80, "c": 42}, {"c": 1, "e": 1, "f": 3}, {"f": 13}]
    at, live, got = {}, {}, {r: [] for r in toks}
    slots = set()
    for step in plan:
        entries = []
        for r, n in step.items():
            if r not in live:
                live[r] = eng.kv_pool.open_elastic(400)
                slots.add(live[r].seqs[0].slot)
            i = at.get(r, 0)
            entries.append((live[r], toks[r][i:i + n], list(range(n))))
            at[r] = i + n
        lg = eng.step(entries).cpu()
        for (r, n), part in zip(step.items(), lg.split(list(step.values()))):
            got[r].append(part)
        for r in list(live):
            if at[r] == lens[r]:
                live.pop(r).close()
    assert not live and eng.kv_pool.free_page_count() == eng.kv_pool.n_pages
    assert slots <= {0, 1, 2}
    for r in toks:
        check(torch.cat(got[r]), want[r], dt, r)


@kinds
def test_many_rows(models, dev, dt, monkeypatch):
    """Beyond 32 rows the GEMMs take other kernels; 40 decoded sequences, then
    300 prompt tokens beside them."""
    eng = engine(models, "full", dev, dt, monkeypatch, tokens=40 * 32 + 400)
    cfg = CONFIGS["full"]
    toks = [prompt(cfg, 14, seed=i) for i in range(40)]
    hs = [eng.kv_pool.open_elastic(32) for _ in toks]
    eng.step([(h, t[:12], []) for h, t in zip(hs, toks)])
    one = eng.step([(h, t[12:13], [0]) for h, t in zip(hs, toks)])
    long = prompt(cfg, 300, seed=99)
    hl = eng.kv_pool.open_elastic(400)
    two = eng.step([(h, t[13:], [0]) for h, t in zip(hs, toks)]
                   + [(hl, long, list(range(300)))])
    w = torch.stack([want_logits(models, "full", t)[12:] for t in toks])
    check(one, w[:, 0], dt)
    check(two[:40], w[:, 1], dt)
    check(two[40:], want_logits(models, "full", long), dt)


# ---------------------------------------------------------------------------
# cache and states
# ---------------------------------------------------------------------------

def test_layout_of_the_cache(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64, seqs=2)
    c = eng.kv_pool
    assert c.own_layers == [2, 4]
    assert c.pools[0] is None and c.pools[1] is None
    assert c.k_pages(2).shape == (4, 2, 16, 64)
    assert c.v_pages(2).shape == (4, 2, 64, 16)
    assert {n: tuple(t.shape) for n, t in c.state(1).items()} == {
        "S": (2, 3, 32, 48), "n": (2, 3, 32), "m": (2, 3)}
    assert {n: tuple(t.shape) for n, t in c.state(0).items()} == {
        "S": (2, 160), "conv": (2, 2, 160)}
    assert c.state(2) is None
    assert all(t.dtype == torch.float32 for s in c.states for t in (s or {}).values())


def test_state_slots_are_admission(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=256, seqs=2)
    c = eng.kv_pool
    a, b = c.open_elastic(64), c.allocate(1, 32)
    assert {a.seqs[0].slot, b.seqs[0].slot} == {0, 1}
    with pytest.raises(AllocationFailed):
        c.open_elastic(64)
    a.close()
    d = c.open_elastic(64)
    assert d.seqs[0].slot != b.seqs[0].slot


def test_recurrent_sessions_do_not_go_back(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=256)
    toks = prompt(CONFIGS["full"], 30, 8)
    h = eng.kv_pool.open_elastic(400)
    eng.step([(h, prompt(CONFIGS["full"], 20, 1), [])])
    with pytest.raises(PagedKVError):
        h.truncate([10])
    with pytest.raises(PagedKVError):
        h.extend(2, speculative=True)
    assert h.lengths == [20]
    h.truncate([0])                      # from the start is a new sequence
    check(eng.step([(h, toks, list(range(30)))]),
          want_logits(models, "full", toks), "float32")


def test_pairs_do_not_go_back(models, monkeypatch):
    """After tokens are taken back the one before the next is not known."""
    eng = engine(models, "attentions", "cpu", "float32", monkeypatch, tokens=256)
    toks = prompt(CONFIGS["attentions"], 30, 8)
    h = eng.kv_pool.open_elastic(400)
    eng.step([(h, toks[:20], [])])
    h.truncate([10])
    with pytest.raises(PagedKVError):
        eng.step([(h, toks[10:], [])])
    h.close()
    g = eng.kv_pool.open_elastic(400)
    eng.step([(g, toks[5:], [])])
    g.truncate([0])
    check(eng.step([(g, toks, list(range(30)))]),
          want_logits(models, "attentions", toks), "float32")


def test_swap_round_trip(models, monkeypatch):
    """Pages leave the device and come back elsewhere; the state stays."""
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=160)
    toks = prompt(CONFIGS["full"], 60, 8)
    want = want_logits(models, "full", toks)
    h = eng.kv_pool.allocate(1, 64)
    eng.step([(h, toks[:50], [])])
    h.swap_out()
    other = eng.kv_pool.open_elastic(400)
    eng.step([(other, prompt(CONFIGS["full"], 90, 9), [])])
    h.swap_in()
    check(eng.step([(h, toks[50:], list(range(10)))]), want[50:], "float32")


def test_step_refuses(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    toks = prompt(CONFIGS["full"], 20, 1)
    h = eng.kv_pool.open_elastic(400)
    eng.step([(h, toks[:7], [])])
    for bad in ([(h, [CONFIGS["full"]["vocab"]], [0])], [(h, [1], [1])],
                [(h, [], [])], [(h, [1], [0]), (h, [2], [0])]):
        with pytest.raises(ValueError):
            eng.step(bad)
    g = eng.kv_pool.open_elastic(400)
    with pytest.raises(AllocationFailed):
        eng.step([(h, [1] * 30, []), (g, [1] * 40, [])])
    # what was refused left no trace
    check(eng.step([(h, toks[7:], [12])]),
          want_logits(models, "full", toks)[19:], "float32")


# ---------------------------------------------------------------------------
# generation
# ---------------------------------------------------------------------------

def agree(got, models, name, p, dt):
    """Greedy continuation by the oracle, up to a close call."""
    toks, tol = list(p), 1e-3 if dt == "float32" else 0.4
    for g in got:
        lg = want_logits(models, name, toks)[-1]
        top = lg.topk(2).values
        if (top[0] - top[1]) / lg.std() < tol:
            return          # both continuations are right
        assert g == int(lg.argmax())
        toks.append(g)


@kinds
@pytest.mark.parametrize("name", ["full", "recurrent"])
def test_generate_greedy(models, name, dev, dt, monkeypatch):
    eng = engine(models, name, dev, dt, monkeypatch)
    ps = [prompt(CONFIGS[name], 21, s) for s in range(3)]
    out = eng.generate_greedy(torch.tensor(ps), 40)
    assert out.shape == (3, 40)
    for p, o in zip(ps, out.tolist()):
        agree(o, models, name, p, dt)
    assert eng.kv_pool.free_page_count() == eng.kv_pool.n_pages


@kinds
@pytest.mark.parametrize("seqs", [2, 8])
def test_scheduler(models, seqs, dev, dt, monkeypatch):
    """More requests than places, pages and state slots, prompts longer than a
    step."""
    eng = engine(models, "full", dev, dt, monkeypatch, tokens=240, seqs=seqs)
    s = BatchScheduler(eng, max_batch=3, chunk_tokens=24)
    lens = [(50, 20), (3, 30), (75, 5), (1, 12), (20, 33), (31, 1)]
    ps = [prompt(CONFIGS["full"], n, seed=n) for n, _ in lens]
    reqs = [s.submit(p, m) for p, (_, m) in zip(ps, lens)]
    peak = 0
    while s.step():
        peak = max(peak, len(s.running))
    assert peak == min(3, seqs) and all(r.done for r in reqs)
    for p, r, (_, m) in zip(ps, reqs, lens):
        assert len(r.output) == m
        agree(r.output, models, "full", p, dt)
    assert eng.kv_pool.free_page_count() == eng.kv_pool.n_pages
    assert len(eng.kv_pool._free_slots) == seqs


def test_sampling(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    s = BatchScheduler(eng)
    first = int(want_logits(models, "full", [5, 6, 7])[-1].argmax())
    r = s.submit([5, 6, 7], 10, eos_token_id=first)
    q = s.submit([5, 6, 7], 4, do_sample=True, top_k=1,
                 generator=torch.Generator().manual_seed(1))
    s.run()
    assert r.output == [first] and q.output[0] == first and len(q.output) == 4


@GPU
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_graph_replays_equal_eager_steps(models, dt, monkeypatch):
    """Many replays of a captured decode step, with eager steps and new
    sequences in between, each against the eager step."""
    eng = engine(models, "full", "cuda:0", dt, monkeypatch)
    ref = engine(models, "full", "cuda:0", dt, monkeypatch)
    cfg = CONFIGS["full"]
    toks = [prompt(cfg, 60, s) for s in range(6)]
    hs, rs, at = {}, {}, {}
    order = [[0, 1, 2], [0, 1, 2, 3], [1, 3], [0, 1, 2, 4], [5, 4, 3, 2]]
    for rnd_ in order * 4:
        for i in rnd_:
            if i not in hs:
                hs[i], rs[i] = (e.kv_pool.open_elastic(400) for e in (eng, ref))
                n = 5 + 7 * i
                for e, h in ((eng, hs[i]), (ref, rs[i])):
                    e.step([(h, toks[i][:n], [])])
                at[i] = n
        got = eng.decode([(hs[i], toks[i][at[i]]) for i in rnd_]).clone()
        want = ref.step([(rs[i], [toks[i][at[i]]], [0]) for i in rnd_])
        torch.cuda.synchronize()
        torch.testing.assert_close(got, want, rtol=1e-4, atol=1e-4)
        for i in rnd_:
            at[i] += 1
            if at[i] == 60:
                hs.pop(i).close()
                rs.pop(i).close()
    assert any(g.graph is not None for g in eng._decode_graphs.values())


@GPU
@pytest.mark.parametrize("B", [3, 40])
def test_lockstep_session_graph(models, B, monkeypatch):
    """A server session's captured decode step (vendor GEMMs beyond 32 rows)."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "bfloat16")
    from bloombee_amd.server.backend import StackBackend
    from bloombee_amd.server.from_pretrained import load_block_weights
    path, _, cfg = models["full"]
    n = len(cfg["layers"])
    be = StackBackend(resolve_config(path), 0, n, device="cuda:0",
                      checkpoint_dir=path, kv_max_tokens=8192)
    ref = BlockStack(resolve_config(path), 0, n, device="cuda:0")
    for i, blk in enumerate(ref.blocks):
        load_block_weights(blk, path, i)
    kv = ref.make_kv(8192).allocate(B, 64)
    be.open_session("s", B, 64)
    g = torch.Generator().manual_seed(0)
    for pos, T in [(0, 9)] + [(9 + i, 1) for i in range(12)]:
        x = torch.randn(B, T, cfg["width"], generator=g)
        out = be.inference_step("s", x, pos).clone()
        kv.extend(T)
        want = ref.forward_inference(
            x.cuda(), kv, torch.full((B,), pos, dtype=torch.int32, device="cuda"))
        torch.testing.assert_close(out, want, rtol=1e-3, atol=1e-3)
    assert be.graphs_captured == 1
    be.shutdown()


# ---------------------------------------------------------------------------
# command line, swarm, offload, training
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("name", ["full", "odd"])
def test_trace_replay(models, name, dev, dt, tmp_path, monkeypatch, capsys):
    from bloombee_amd.cli import trace_run
    cfg = CONFIGS[name]
    a, b = prompt(cfg, 40, 1), prompt(cfg, 20, 2)
    E = lambda r, t, w: {"id": r, "tokens": t, "want": w}
    steps = [
        {"step": 0, "entries": [E("a", a[:30], [0, 29])], "end": []},
        {"step": 1, "entries": [E("b", b[:2], []), E("a", a[30:31], [])], "end": []},
        {"step": 2, "entries": [E("a", a[31:32], [0]), E("b", b[2:3], [0])],
         "end": []},
        {"step": 3, "entries": [E("b", b[3:], [16]), E("a", a[32:], [7])],
         "end": ["a", "b"]},
        # the same names once more, on used pages and slots
        {"step": 4, "entries": [E("a", b, [19])], "end": ["a"]},
    ]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps))))
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    rc = trace_run.main(["--model", models[name][0], "--dtype", dt, "--out",
                         str(tmp_path), "--max-tokens", "128", "--max-requests",
                         "2", "--device", dev])
    assert rc == 0
    done = [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")]
    assert done == [f"done {i}" for i in range(5)]
    wa, wb = (want_logits(models, name, t) for t in (a, b))
    want = {0: wa[[0, 29]], 2: torch.stack([wa[31], wb[2]]),
            3: torch.stack([wb[19], wa[39]]), 4: wb[19:]}
    assert sorted(os.listdir(tmp_path)) == sorted(f"{k}.f32" for k in want)
    for k, w in want.items():
        raw = torch.frombuffer(bytearray((tmp_path / f"{k}.f32").read_bytes()),
                               dtype=torch.float32)
        check(raw.view(-1, cfg["vocab"]), w, dt, k)


@kinds
def test_swarm_generation(models, dev, dt, monkeypatch):
    """Two servers and a client on one checkpoint folder, hidden states in 32
    bits; the client follows the tokens for the pair embedding."""
    from bloombee_amd.client.config import ClientConfig
    from bloombee_amd.models import auto
    from bloombee_amd.net.dht import Dht
    from bloombee_amd.server import Server
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    path, _, cfg = models["wide"]
    boot = Dht()
    srvs = [Server(path, initial_peers=[boot.endpoint], block_indices=r,
                   update_period=5.0, device=dev, kv_max_tokens=4096)
            for r in ((0, 2), (2, 5))]
    for s in srvs:
        s.run_in_background()
    try:
        m = auto.AutoDistributedModelForCausalLM.from_pretrained(
            path, client_config=ClientConfig(initial_peers=[boot.endpoint]),
            device=dev)
        p = prompt(cfg, 12, 4)
        out = m.generate(torch.tensor([p], device=dev),
                         max_new_tokens=8)[0].tolist()
        assert out[:12] == p
        agree(out[12:], models, "wide", p, dt)
    finally:
        for s in srvs:
            s.shutdown()
        boot.shutdown()


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda:0", marks=GPU)])
def test_offloaded_blocks(models, dev, monkeypatch):
    """Blocks of unlike shapes stream through one arena."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    from bloombee_amd.offload import OffloadPolicy
    from bloombee_amd.offload.weights import OffloadedBlockStack
    from bloombee_amd.server.from_pretrained import load_block_weights
    path, w, cfg = models["full"]
    stack = BlockStack(resolve_config(path), 0, 6, device=dev)
    for i, blk in enumerate(stack.blocks):
        load_block_weights(blk, path, i)
    off = OffloadedBlockStack(stack, OffloadPolicy(weight_gpu_percent=20.0))
    toks = torch.tensor(prompt(cfg, 50, 5))
    want = oracle.hidden_states(toks, w, cfg)[-1]
    x = oracle.embed(toks, w, cfg).float()[None].to(dev)
    kv = off.make_kv(128).allocate(1, 50)
    out = []
    for a, b in ((0, 31), (31, 49), (49, 50)):
        kv.extend(b - a)
        out.append(off.forward_inference(
            x[:, a:b], kv, torch.tensor([a], dtype=torch.int32, device=dev)))
    got = torch.cat(out, 1)[0].cpu().double()
    torch.testing.assert_close(got, want, rtol=1e-4, atol=2e-4)


@pytest.mark.parametrize("name", ["full", "odd"])
def test_training_path(models, name, monkeypatch):
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    path, w, cfg = models[name]
    eng = LocalEngine(path, kv_max_tokens=64)
    toks = torch.tensor(prompt(cfg, 45, 5))
    col = oracle.hidden_states(toks, w, cfg)
    x = oracle.embed(toks, w, cfg).float()[None].requires_grad_(True)
    y = eng.stack.forward_train(x)
    torch.testing.assert_close(y[0].double(), col[-1], rtol=1e-4, atol=2e-4)
    lg = eng.head.train_logits(eng.head.train_norm(y))
    check(lg[0].detach(), oracle.forward(toks, w, cfg), "float32")
    y.square().mean().backward()
    assert torch.isfinite(x.grad).all() and x.grad.abs().max() > 0


def test_deep_prompts(models, monkeypatch):
    """Per-layer prompt vectors are added to the residual before each block."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    eng = LocalEngine(models["full"][0], kv_max_tokens=64)
    x = torch.randn(1, 20, 192, generator=torch.Generator().manual_seed(0))
    dp = torch.randn(6, 6, 192, generator=torch.Generator().manual_seed(1))
    kv = eng.kv_pool.allocate(1, 20)
    kv.extend(20)
    keep = x.clone()
    got = eng.stack.forward_inference(x, kv, torch.zeros(1, dtype=torch.int32),
                                      deep_prompts=dp)
    torch.testing.assert_close(x, keep)     # the caller's tensor is its own
    want = eng.stack.forward_train(x, deep_prompts=dp)
    torch.testing.assert_close(got, want, rtol=1e-4, atol=2e-4)


def test_config_reader(models):
    cfg = VumedraConfig.from_dict(CONFIGS["odd"])
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers) == (90, 101, 4)
    assert cfg.hidden_dtype == torch.float32 and cfg.rms_norm_eps == 1e-3
    assert cfg.bigram == {"buckets": 1, "mul_prev": 3, "mul_cur": 0}
    s = cfg.recurrent_spec(1)
    assert (s.heads, s.dim, s.vdim, s.cap) == (3, 18, 21, 1.5)
    s = cfg.recurrent_spec(2)
    assert (s.width, s.blocks, s.taps, s.block_p) == (77, 7, 1, 64)
    assert cfg.recurrent_spec(0) is None
    assert resolve_config(models["full"][0]).model_type == "vumedra"
    for change in (lambda c: c["layers"][0].update(type="convolution"),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=2),
                   lambda c: c["layers"][1]["mixer"].update(gate_cap=0.0),
                   lambda c: c["layers"][1]["mlp"]["router"].update(top=4),
                   lambda c: c["layers"][2]["mixer"].update(blocks=3),
                   lambda c: c["layers"][2]["mixer"].update(conv=0),
                   lambda c: c["layers"][3]["mlp"].update(kind="glu"),
                   lambda c: c["embedding"]["bigram"].update(buckets=0)):
        bad = copy.deepcopy(CONFIGS["odd"])
        change(bad)
        with pytest.raises(ValueError):
            VumedraConfig.from_dict(bad)


def test_presets_resolve():
    for name in ("vumedra-8b-attn-4l", "vumedra-8b-mlstm-4l",
                 "vumedra-8b-rglru-4l", "vumedra-8x7b-4l"):
        assert resolve_config(name).model_type == "vumedra"
    eng = LocalEngine("vumedra-tiny", kv_max_tokens=256)
    out = eng.generate_greedy(torch.tensor([[1, 2, 3]]), 4)
    assert out.shape == (1, 4)


def test_wrong_shapes_are_refused(models, tmp_path, monkeypatch):
    path, w, cfg = models["odd"]
    bad = {k: v.float() for k, v in w.items()}
    bad["l0.mlp.up"] = bad["l0.mlp.up"][:-1].contiguous()
    save(cfg, tmp_path, bad)
    with pytest.raises(ValueError, match="mlp.up"):
        LocalEngine(str(tmp_path), kv_max_tokens=64)


def test_no_tree_steps(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    kv = eng.kv_pool.allocate(1, 8)
    kv.extend(1)
    with pytest.raises(NotImplementedError):
        eng.stack.forward_inference(
            torch.zeros(1, 1, 192), kv, torch.zeros(1, dtype=torch.int32),
            position_ids=torch.zeros(1, 1, dtype=torch.int32))
