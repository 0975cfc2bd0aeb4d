"""Zatusun models end to end: engine, cache and state slots, scheduler, trace
replay and swarm against the plain oracle, on small random models of several
shapes. CPU forms run here, the HIP kernels under -m gpu."""
import copy
import io
import json
import os

import pytest
import torch
from safetensors.torch import save_file

import zatusun_oracle as oracle
from bloombee_amd.engine import BlockStack, LocalEngine
from bloombee_amd.kv.paged import AllocationFailed, PagedKVError
from bloombee_amd.models.base import resolve_config
from bloombee_amd.models.zatusun import ZatusunConfig
from bloombee_amd.scheduler import BatchScheduler

GPU = pytest.mark.gpu
KINDS = [pytest.param("cpu", "float32", id="cpu-f32"),
         pytest.param("cuda:0", "float32", id="gpu-f32", marks=GPU),
         pytest.param("cuda:0", "bfloat16", id="gpu-bf16", marks=GPU)]
kinds = pytest.mark.parametrize("dev,dt", KINDS)


def latent(heads, dim, rot, vdim, rank, q_rank, base=1e4, scale=None, factor=4.0,
           original=64, fast=8.0, slow=0.5):
    return "latent_attention", {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
        "kv_rank": rank, "q_rank": q_rank, "scale": scale or (dim + rot) ** -0.5,
        "rot": {"base": base, "dims": rot, "scaling": {
            "factor": factor, "original": original, "fast": fast,
            "slow": slow}}}


def diff(heads, kv_heads, dim, vdim, chunk, rot, base=5e4, scale=None, d=0.3,
         factor=8.0, low=1.0, high=4.0, original=128):
    return "attention", {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "diff": d,
        "mask": {"size": chunk}, "scale": scale or dim ** -0.5,
        "rot": {"base": base, "dims": rot, "scaling": {
            "factor": factor, "low": low, "high": high, "original": original}}}


def hgrn(heads, dim, vdim):
    return "hgrn2", {"heads": heads, "dim": dim, "vdim": vdim}


def moe(experts, top, ff, limit=1.0):
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff, "limit": limit}}


def model(width, vocab, layers, loop=None, eps=1e-5, scale=5.0, cap=20.0,
          positions=700):
    cfg = {"architecture": "Zatusun", "width": width, "vocab": vocab,
           "norm": {"eps": eps}, "embedding": {"scale": scale},
           "max_positions": positions, "logit_softcap": cap,
           "layers": [{"type": t, "mixer": m, "mlp": f} for (t, m), f in layers]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


CONFIGS = {
    # all mechanisms, layers before, in and behind a loop of three passes
    "full": model(192, 333, [
        (diff(6, 2, 24, 40, 50, 12), moe(7, 3, 72)),
        (hgrn(3, 32, 48), moe(5, 2, 64, limit=0.5)),
        (latent(5, 24, 16, 40, 80, 72), None),
        (diff(4, 4, 40, 64, 33, 40, d=0.7), moe(4, 4, 40, limit=3.0)),
        (hgrn(5, 24, 40), None)], loop=(1, 4, 3), scale=3.0),
    # sizes that are no multiple of four, as few parts as there can be
    "odd": model(90, 101, [
        (latent(3, 18, 6, 21, 30, 27, scale=0.3), moe(3, 3, 50)),
        (hgrn(3, 18, 21), moe(1, 1, 30)),
        (diff(5, 1, 18, 21, 7, 2), None)],
        loop=(1, 2, 2), eps=1e-3, scale=1.0, cap=3.0),
    # the largest compiled sizes, the whole model looped
    "wide": model(320, 517, [
        (diff(20, 4, 128, 128, 64, 128), moe(16, 4, 64)),
        (hgrn(2, 128, 256), None),
        (latent(18, 128, 64, 128, 128, 192), moe(6, 1, 320)),
        (diff(2, 1, 96, 256, 400, 64), None)], loop=(0, 4, 2), scale=8.0),
    # no loop, no recurrence
    "attentions": model(128, 97, [
        (latent(4, 32, 32, 32, 64, 64), None),
        (diff(4, 2, 32, 40, 24, 10), moe(4, 2, 32))], cap=None),
    # recurrence only, one pass
    "recurrent": model(128, 97, [(hgrn(2, 32, 64), moe(3, 2, 64)),
                                 (hgrn(4, 32, 32), None)], loop=(1, 2, 1)),
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
        if t is not None:
            t.fill_(float("nan"))
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
    hidden = eng.head.embed(torch.tensor(toks, device=dev), b.tok_pos)
    assert hidden.shape == (40, 2 * cfg["width"])
    x = b.split_hidden(hidden, cfg["width"])
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
    assert torch.equal(hidden[:, cfg["width"]:], eng.head.embed(
        torch.tensor(toks, device=dev), b.tok_pos)[:, :cfg["width"]])


@kinds
@pytest.mark.parametrize("change", [
    "chunk", "difference", "inner norm", "half pairs", "yarn factor", "bands",
    "output gate", "lower bound", "step", "embedding read again",
    "embedding output", "all scores", "limit", "norm weight", "softcap"])
def test_the_tests_can_see(tmp_path, change, dev, dt, monkeypatch):
    """An oracle with one planted mistake differs visibly, the engine does
    not."""
    cfg = model(128, 97, [
        (hgrn(2, 32, 48), moe(4, 2, 64, limit=0.7)),
        (latent(4, 32, 32, 40, 64, 64, scale=0.3, factor=9.0), None),
        (diff(4, 2, 32, 48, 13, 16, scale=0.4, original=40), moe(4, 2, 64))],
        loop=(0, 2, 2), cap=2.0)
    w = oracle.random_weights(cfg, 5)
    wd = {k: v.double() for k, v in w.items()}
    path = save(cfg, tmp_path, w)
    toks = torch.tensor(prompt(cfg, 60, 6))
    want = oracle.forward(toks, wd, cfg)
    off, wo = copy.deepcopy(cfg), dict(wd)
    with monkeypatch.context() as mp:
        if change == "chunk":
            off["layers"][2]["mixer"]["mask"]["size"] = 14
        elif change == "difference":
            wo["l2.mix.lq1"] = -wd["l2.mix.lq1"]
        elif change == "inner norm":
            off["layers"][2]["mixer"]["diff"] = 0.35
            plain = oracle.mix_factor
            mp.setattr(oracle, "mix_factor", lambda w, pre, d: plain(w, pre, 0.3))
        elif change == "half pairs":
            def halves(x, freqs, factor=1.0, first=0):
                n = len(freqs)
                order = torch.stack([torch.arange(n), torch.arange(n) + n],
                                    1).flatten()
                y = x.clone()
                y[..., order] = plain_rotate(x[..., order], freqs, factor, first)
                return y
            plain_rotate = oracle.rotate
            mp.setattr(oracle, "rotate", halves)
        elif change == "yarn factor":
            plain = oracle.yarn
            mp.setattr(oracle, "yarn", lambda rot: (plain(rot)[0], 1.0))
        elif change == "bands":
            off["layers"][2]["mixer"]["rot"]["scaling"]["high"] = 1.5
        elif change == "output gate":
            wo["l1.mix.g"] = wd["l1.mix.g"] * 0.5
        elif change == "lower bound":
            wo["l0.mix.lower"] = wd["l0.mix.lower"] * 0.9
        elif change == "step":
            wo["loop.step"] = wd["loop.step"].flip(0)
        elif change == "embedding read again":
            mp.setattr(oracle, "enter_pass", lambda x, x0, t, w: torch.cat(
                [x, x], -1) @ w["loop.in"].T + w["loop.step"][t])
        elif change == "embedding output":
            plain = oracle.embed
            mp.setattr(oracle, "embed", lambda ids, w, cfg: plain(ids, w, {
                **cfg, "embedding": {"scale": 4.0}}))
        elif change == "all scores":
            mp.setattr(oracle, "choose", lambda z, top: (
                torch.topk(z, top, -1).indices,
                torch.topk(oracle.softmax(z), top, -1).values))
        elif change == "limit":
            off["layers"][0]["mlp"]["expert"]["limit"] = 0.9
        elif change == "norm weight":
            wo["l2.norm1"] = wd["l2.norm1"] * 0
        else:
            off["logit_softcap"] = 2.2
        wrong = oracle.forward(toks, wo, off)
    d = (wrong - want).pow(2).mean(-1).sqrt() / want.std()
    assert (d > 0.01).double().mean() > 0.1, d.max()
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
    # three passes over layers 1 .. 3, each with its own
    assert [c.layout[i] for i in range(11)] == \
        ["kv"] + ["none", "k", "kv"] * 3 + ["none"]
    assert len({c.k_pages(i).data_ptr() for i in (2, 5, 8)}) == 3
    assert c.k_pages(0).shape == (4, 2, 16, 64)
    assert c.v_pages(0).shape == (4, 2, 64, 16)
    assert c.k_pages(3).shape == (4, 4, 16, 128)
    assert c.k_pages(2).shape == (4, 1, 16, 160)
    assert c.state(1).shape == c.state(7).shape == (2, 3, 32, 48)
    assert c.state(10).shape == (2, 5, 24, 40) and c.state(2) is None
    assert all(t.dtype == torch.float32 for t in c.states if t is not None)
    # ... and the weights in common
    b = eng.stack.blocks
    assert b[1].in_w is b[4].in_w is b[7].in_w and b[3].out_w is b[9].out_w
    assert [x.enters for x in b[1:8:3]] == [0, 1, 2]
    assert b[2].enters is None and b[10].enters is None


def test_random_weights_do_not_depend_on_the_block_range(monkeypatch):
    """A server that starts in the middle of the loop draws what one that holds
    everything draws."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    cfg = resolve_config("zatusun-tiny")
    whole, part = BlockStack(cfg, 0, 6), BlockStack(cfg, 2, 6)
    for i, blk in enumerate(part.blocks):
        other = dict(whole.blocks[i + 2].named_parameters())
        for name, w in blk.named_parameters():
            assert torch.equal(w, other.pop(name)), (i, name)
        assert not other


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
    tol = 1e-3 if dt == "float32" else 0.4
    all_lg = want_logits(models, name, list(p) + list(got[:-1]))
    for g, lg in zip(got, all_lg[len(p) - 1:]):
        top = lg.topk(2).values
        if (top[0] - top[1]) / lg.std() < tol:
            return          # both continuations are right
        assert g == int(lg.argmax())


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
    n = resolve_config(path).num_hidden_layers
    be = StackBackend(resolve_config(path), 0, n, device="cuda:0",
                      checkpoint_dir=path, kv_max_tokens=8192)
    ref = BlockStack(resolve_config(path), 0, n, device="cuda:0")
    for i, blk in enumerate(ref.blocks):
        load_block_weights(blk, path, i)
    kv = ref.make_kv(8192).allocate(B, 64)
    be.open_session("s", B, 64)
    g = torch.Generator().manual_seed(0)
    for pos, T in [(0, 9)] + [(9 + i, 1) for i in range(12)]:
        x = torch.randn(B, T, 2 * cfg["width"], generator=g)
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
    """Two servers and a client on one checkpoint folder; the second server starts
    within the first pass and runs the whole second one."""
    from bloombee_amd.client.config import ClientConfig
    from bloombee_amd.models import auto
    from bloombee_amd.net.dht import Dht
    from bloombee_amd.server import Server
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    path, _, cfg = models["wide"]
    boot = Dht()
    srvs = [Server(path, initial_peers=[boot.endpoint], block_indices=r,
                   update_period=5.0, device=dev, kv_max_tokens=4096)
            for r in ((0, 3), (3, 8))]
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
    """Blocks of unlike shapes stream through one arena, runs of one layer each
    with what they need."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    from bloombee_amd.offload import OffloadPolicy
    from bloombee_amd.offload.weights import OffloadedBlockStack
    from bloombee_amd.server.from_pretrained import load_block_weights
    path, w, cfg = models["full"]
    stack = BlockStack(resolve_config(path), 0, 11, device=dev)
    for i, blk in enumerate(stack.blocks):
        load_block_weights(blk, path, i)
    off = OffloadedBlockStack(stack, OffloadPolicy(weight_gpu_percent=20.0))
    toks = torch.tensor(prompt(cfg, 50, 5))
    want = oracle.hidden_states(toks, w, cfg)[-1]
    x = oracle.embed(toks, w, cfg).float()[None].to(dev).repeat(1, 1, 2)
    kv = off.make_kv(128).allocate(1, 50)
    out = []
    for a, b in ((0, 31), (31, 49), (49, 50)):
        kv.extend(b - a)
        out.append(off.forward_inference(
            x[:, a:b], kv, torch.tensor([a], dtype=torch.int32, device=dev)))
    got = torch.cat(out, 1)[0, :, :cfg["width"]].cpu().double()
    torch.testing.assert_close(got, want, rtol=1e-4, atol=2e-4)


@pytest.mark.parametrize("name", ["full", "odd", "attentions"])
def test_training_path(models, name, monkeypatch):
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    path, w, cfg = models[name]
    eng = LocalEngine(path, kv_max_tokens=64)
    toks = torch.tensor(prompt(cfg, 45, 5))
    col = oracle.hidden_states(toks, w, cfg)
    x = oracle.embed(toks, w, cfg).float()[None].repeat(
        1, 1, eng.head.copies).requires_grad_(True)
    y = eng.stack.forward_train(x)
    torch.testing.assert_close(y[0, :, :cfg["width"]].double(), col[-1], rtol=1e-4,
                               atol=2e-4)
    lg = eng.head.train_logits(eng.head.train_norm(y))
    check(lg[0].detach(), oracle.forward(toks, w, cfg), "float32")
    y.square().mean().backward()
    assert torch.isfinite(x.grad).all() and x.grad.abs().max() > 0
    if cfg.get("loop"):          # the embedding output is read in every pass
        assert x.grad[..., cfg["width"]:].abs().max() > 0


def test_deep_prompts(models, monkeypatch):
    """Per-layer prompt vectors are added to the residual before each block."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    eng = LocalEngine(models["full"][0], kv_max_tokens=64)
    x = torch.randn(1, 20, 384, generator=torch.Generator().manual_seed(0))
    dp = torch.randn(11, 6, 192, generator=torch.Generator().manual_seed(1))
    kv = eng.kv_pool.allocate(1, 20)
    kv.extend(20)
    keep = x.clone()
    got = eng.stack.forward_inference(x, kv, torch.zeros(1, dtype=torch.int32),
                                      deep_prompts=dp)
    torch.testing.assert_close(x, keep)     # the caller's tensor is its own
    want = eng.stack.forward_train(x, deep_prompts=dp)
    torch.testing.assert_close(got, want, rtol=1e-4, atol=2e-4)


def test_prompt_tuning_client(models, monkeypatch):
    """A trained prompt goes ahead of the embedded tokens, in both halves of what
    travels."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    from bloombee_amd.client.config import ClientConfig
    from bloombee_amd.models.zatusun import DistributedZatusunModel
    m = DistributedZatusunModel(resolve_config(models["odd"][0]), ClientConfig(
        initial_peers=[]), "m", manager=object(), pre_seq_len=3,
        checkpoint_dir=models["odd"][0])
    h = m.embed(torch.tensor([[1, 2], [3, 4]]), 3)
    p = m.prompt_hidden(h)
    assert h.shape == (2, 2, 180) and p.shape == (2, 3, 180)
    assert torch.equal(p[..., :90], p[..., 90:])
    assert torch.equal(p[0, :, :90], m.prompt_embeds)


def test_config_reader(models):
    cfg = ZatusunConfig.from_dict(CONFIGS["full"])
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers) == (192, 333, 11)
    assert cfg.hidden_columns == 384 and cfg.hidden_dtype == torch.float32
    assert cfg.max_position_embeddings == 700 and cfg.embedding_scale == 3.0
    runs = [(r.layer, r.enters, r.first) for r in cfg.runs]
    assert runs == [(0, None, 0), (1, 0, 1), (2, None, 2), (3, None, 3),
                    (1, 1, 1), (2, None, 2), (3, None, 3),
                    (1, 2, 1), (2, None, 2), (3, None, 3), (4, None, 10)]
    s = cfg.mixer_spec(3)
    assert (s.rope.heads, s.rope.kv_heads, s.rope.dim, s.chunk) == (4, 4, 40, 33)
    assert s.factor == pytest.approx(0.3)
    assert cfg.mixer_spec(2).amp == pytest.approx(1 + 0.1 * 1.3862943611)
    assert cfg.glu_spec(1).limit == 0.5
    plain = ZatusunConfig.from_dict(CONFIGS["attentions"])
    assert plain.hidden_columns == 128 and plain.num_hidden_layers == 2
    assert plain.logit_softcap == 0.0
    assert resolve_config(models["full"][0]).model_type == "zatusun"
    for change in (lambda c: c["layers"][0].update(type="convolution"),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
                   lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26),
                   lambda c: c["layers"][2]["mixer"]["rot"].update(dims=7),
                   lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
                   lambda c: c["layers"][1]["mlp"]["router"].update(top=6),
                   lambda c: c["layers"][1]["mlp"].update(kind="dense"),
                   lambda c: c["loop"].update(stop=6),
                   lambda c: c["loop"].update(times=0)):
        bad = copy.deepcopy(CONFIGS["full"])
        change(bad)
        with pytest.raises(ValueError):
            ZatusunConfig.from_dict(bad)


def test_presets_resolve():
    for name in ("zatusun-8b-latent-4l", "zatusun-8b-diff-4l",
                 "zatusun-8b-hgrn2-4l", "zatusun-8x7b-4l"):
        cfg = resolve_config(name)
        assert cfg.model_type == "zatusun" and cfg.num_hidden_layers == 4
    eng = LocalEngine("zatusun-tiny", kv_max_tokens=256)
    out = eng.generate_greedy(torch.tensor([[1, 2, 3]]), 4)
    assert out.shape == (1, 4)


def test_wrong_shapes_are_refused(models, tmp_path, monkeypatch):
    path, w, cfg = models["odd"]
    bad = {k: v.float() for k, v in w.items()}
    bad["l0.mlp.e1.up"] = bad["l0.mlp.e1.up"][:-1].contiguous()
    save(cfg, tmp_path, bad)
    with pytest.raises(ValueError, match="mlp.e1.up"):
        LocalEngine(str(tmp_path), kv_max_tokens=64)


def test_no_tree_steps(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    kv = eng.kv_pool.allocate(1, 8)
    kv.extend(1)
    with pytest.raises(NotImplementedError):
        eng.stack.forward_inference(
            torch.zeros(1, 1, 384), kv, torch.zeros(1, dtype=torch.int32),
            position_ids=torch.zeros(1, 1, dtype=torch.int32))
