"""Mubasun models end to end: engine, cache, scheduler, trace replay and swarm
against the plain oracle, on small random models of several shapes. CPU forms
run here, the HIP kernels under -m gpu."""
import copy
import io
import json
import os

import pytest
import torch
from safetensors.torch import save_file

import mubasun_oracle as oracle
from bloombee_amd.engine import BlockStack, LocalEngine
from bloombee_amd.kv.paged import AllocationFailed, PagedKVError
from bloombee_amd.models.base import resolve_config
from bloombee_amd.models.mubasun import MubasunConfig
from bloombee_amd.scheduler import BatchScheduler

GPU = pytest.mark.gpu
KINDS = [pytest.param("cpu", "float32", id="cpu-f32"),
         pytest.param("cuda:0", "float32", id="gpu-f32", marks=GPU),
         pytest.param("cuda:0", "bfloat16", id="gpu-bf16", marks=GPU)]
kinds = pytest.mark.parametrize("dev,dt", KINDS)


def attn(heads, kv, dim, vdim, window, scale=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
         "scale": scale or dim ** -0.5, "mask": {"size": window}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def moe(E, ff, top, identity=0, scale=1.0, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff},
         "router": {"experts": E, "identity": identity, "scale": scale,
                    "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def model(width, vocab, groups, layers, eps=1e-5, max_positions=400):
    return {"architecture": "Mubasun", "width": width, "vocab": vocab,
            "max_positions": max_positions,
            "norm": {"eps": eps, "groups": groups},
            "layers": [{"type": "attention", "mixer": m, "mlp": f}
                       for m, f in layers]}


CONFIGS = {
    # all mechanisms, unlike sizes everywhere
    "full": model(192, 333, 3, [
        (attn(6, 2, 48, 40, 24), dense(200)),
        (attn(6, 2, 48, 40, 33, scale=0.2), moe(6, 80, 3, 2, 1.7, shared=112)),
        (attn(6, 2, 48, 40, 17, kv_from=1), moe(6, 80, 2, 3, 0.6)),
        (attn(6, 2, 48, 40, 50, kv_from=0), None),
        (attn(4, 4, 64, 32, 1), moe(3, 96, 3, 0, 1.0, shared=64))]),
    # sizes that are no multiple of four, layers that differ in heads
    "odd": model(90, 101, 5, [
        (attn(3, 1, 30, 21, 19), moe(5, 33, 2, 1, 2.0, shared=27)),
        (attn(5, 5, 18, 18, 31), dense(77)),
        (attn(3, 1, 30, 21, 40, kv_from=0), dense(50))], eps=1e-3),
    # windows beyond the context, many heads on one key head, one group
    "wide": model(320, 517, 1, [
        (attn(20, 1, 32, 64, 5000), dense(512)),
        (attn(2, 1, 128, 128, 96), moe(16, 64, 4, 0, 1.0))]),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    """name -> (checkpoint folder, float64 weights, config)"""
    out = {}
    for i, (name, cfg) in enumerate(CONFIGS.items()):
        d = tmp_path_factory.mktemp(name)
        w = oracle.random_weights(cfg, seed=10 + i)
        (d / "config.json").write_text(json.dumps(cfg))
        save_file({k: v.bfloat16() for k, v in w.items()},
                  str(d / "model.safetensors"))
        out[name] = (str(d), {k: v.double() for k, v in w.items()}, cfg)
    return out


def engine(models, name, dev, dt, monkeypatch, tokens=1024):
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    return LocalEngine(models[name][0], device=dev, kv_max_tokens=tokens)


def prompt(cfg, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def want_logits(models, name, toks):
    _, w, cfg = models[name]
    return oracle.forward(torch.tensor(toks), w, cfg)


def check(got, want, dt, what=""):
    """Root mean square over the vocabulary, mean taken off, against the
    spread of the logits."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.std()
    limit = 1e-5 if dt == "float32" else 0.04
    assert err.max() < limit, (what, err.max().item(), int(err.argmax()))


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
    """Decoding from the first token on, far past every window."""
    eng = engine(models, name, dev, dt, monkeypatch)
    n = 120
    toks = prompt(CONFIGS[name], n, seed=3)
    check(run(eng, toks, list(range(1, n + 1))),
          want_logits(models, name, toks), dt)


@kinds
@pytest.mark.parametrize("size", [2, 3, 7, 16, 31, 50])
def test_portions(models, size, dev, dt, monkeypatch):
    eng = engine(models, "full", dev, dt, monkeypatch)
    n = 111
    toks = prompt(CONFIGS["full"], n, seed=4)
    cuts = list(range(size, n, size)) + [n]
    check(run(eng, toks, cuts), want_logits(models, "full", toks), dt)


@kinds
def test_residual_after_every_layer(models, dev, dt, monkeypatch):
    from bloombee_amd.kv.batch import session_batch
    from bloombee_amd.ops import ragged
    eng = engine(models, "full", dev, dt, monkeypatch)
    toks = prompt(CONFIGS["full"], 40)
    col = []
    _, w, cfg = models["full"]
    oracle.forward(torch.tensor(toks), w, cfg, col)
    h = eng.kv_pool.open_elastic(64)
    h.extend(40)
    b = session_batch([(h, 40)])
    x = eng.head.embed(torch.tensor(toks, device=dev), b.tok_pos)
    for blk, want in zip(eng.stack.blocks, col):
        ragged.residual_norm(x, blk.forward_tokens(x, None, b))
        tol = 1e-4 if dt == "float32" else 0.05
        assert x.dtype == torch.float32
        assert (x.cpu() - want).abs().max() < tol * want.abs().max()


def bend(w, layer, boost):
    """Make layer `layer`'s scores sharp so that single keys decide."""
    w = dict(w)
    for n in ("q.norm", "k.norm"):
        key = f"l{layer}.mix.{n}"
        if key in w:
            w[key] = (w[key] * boost).bfloat16().to(w[key].dtype)
    return w


@kinds
def test_sharp_scores_near_the_window_edge(tmp_path, dev, dt, monkeypatch):
    """Scores so far apart that a window off by one changes the logits."""
    cfg = model(128, 97, 8, [(attn(4, 2, 32, 32, 21), dense(96))])
    w = bend(oracle.random_weights(cfg, 5), 0, 3.0)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.bfloat16() for k, v in w.items()},
              str(tmp_path / "model.safetensors"))
    wd = {k: v.double() for k, v in w.items()}
    toks = prompt(cfg, 90, 6)
    want = oracle.forward(torch.tensor(toks), wd, cfg)
    off = copy.deepcopy(cfg)
    off["layers"][0]["mixer"]["mask"]["size"] = 20
    wrong = oracle.forward(torch.tensor(toks), wd, off)
    d = (wrong - want).pow(2).mean(-1).sqrt() / want.std()
    assert (d[30:] > 0.04).float().mean() > 0.1      # the test can see it
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    eng = LocalEngine(str(tmp_path), device=dev, kv_max_tokens=128)
    check(run(eng, toks, [90]), want, dt)
    check(run(eng, toks, [40] + list(range(41, 91))), want, dt)


# ---------------------------------------------------------------------------
# batches
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("name", ["full", "odd"])
def test_mixed_batch(models, name, dev, dt, monkeypatch):
    """Unequal requests, portions beside decoded tokens, requests that pause,
    pages that change hands: every logit as if the request ran alone."""
    cfg = CONFIGS[name]
    eng = engine(models, name, dev, dt, monkeypatch, tokens=320)
    for t in {id(t): t for p in eng.kv_pool.pools for t in p}.values():
        t.fill_(1e3)                 # what earlier owners left
    lens = {"a": 97, "b": 30, "c": 64, "d": 5, "e": 81, "f": 16}
    toks = {r: prompt(cfg, n, seed=ord(r)) for r, n in lens.items()}
    want = {r: want_logits(models, name, t) for r, t in toks.items()}
    plan = [{"a": 64, "b": 29}, {"a": 1, "b": 1, "c": 17}, {"c": 2, "d": 2},
            {"a": 30, "c": 1, "d": 1}, {"d": 2, "c": 1, "a": 2},
            {"e": 80, "c": 42}, {"c": 1, "e": 1, "f": 3}, {"f": 13}]
    at, live, got = {}, {}, {r: [] for r in toks}
    for step in plan:
        entries = []
        for r, n in step.items():
            if r not in live:
                live[r] = eng.kv_pool.open_elastic(400)
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
    for r in toks:
        check(torch.cat(got[r]), want[r], dt, r)


@kinds
def test_many_rows(models, dev, dt, monkeypatch):
    """Beyond 32 rows the GEMMs, the router and the experts take other
    kernels; 40 decoded sequences, then 300 prompt tokens beside them."""
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
    for i in (0, 17, 39):
        w = want_logits(models, "full", toks[i])
        check(one[i:i + 1], w[12:13], dt, i)
        check(two[i:i + 1], w[13:14], dt, i)
    check(two[40:], want_logits(models, "full", long), dt)


def test_step_refuses(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    h = eng.kv_pool.open_elastic(400)
    with pytest.raises(ValueError):
        eng.step([(h, [CONFIGS["full"]["vocab"]], [0])])
    with pytest.raises(ValueError):
        eng.step([(h, [1], [1])])
    with pytest.raises(ValueError):
        eng.step([(h, [], [])])
    with pytest.raises(ValueError):
        eng.step([(h, [1], [0]), (h, [2], [0])])
    g = eng.kv_pool.open_elastic(400)
    with pytest.raises(AllocationFailed):
        eng.step([(h, [1] * 40, []), (g, [1] * 40, [])])
    # nothing was taken by the refused step
    assert h.lengths == [0] and g.lengths == [0]
    assert eng.kv_pool.free_page_count() == 4
    eng.step([(h, [1] * 64, [])])
    with pytest.raises(ValueError):
        eng.step([(h, [1] * 400, [])])


# ---------------------------------------------------------------------------
# cache
# ---------------------------------------------------------------------------

def test_shared_layers_own_no_pages(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    c = eng.kv_pool
    assert c.own_layers == [0, 1, 4]
    assert c.k_pages(2) is c.k_pages(1) and c.pools[3][1] is c.pools[0][1]
    assert c.k_pages(0).shape[3] == 64 and c.v_pages(0).shape[2] == 64
    assert c.k_pages(4).shape[3] == 64 and c.v_pages(4).shape[2] == 32


def test_swap_round_trip_with_shared_layers(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=256)
    toks = prompt(CONFIGS["full"], 60, 8)
    want = want_logits(models, "full", toks)
    h = eng.kv_pool.allocate(1, 64)
    eng.step([(h, toks[:50], [])])
    h.swap_out()
    other = eng.kv_pool.open_elastic(400)
    eng.step([(other, prompt(CONFIGS["full"], 100, 9), [])])
    h.swap_in()
    check(eng.step([(h, toks[50:], list(range(10)))]), want[50:], "float32")
    h.swap_out_rows(0, 1)
    h.swap_in_rows(0, 1)
    h.close()


def test_rollback_of_speculative_tokens(models, monkeypatch):
    """Cut a sequence back and go on otherwise."""
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=256)
    toks = prompt(CONFIGS["full"], 60, 8)
    h = eng.kv_pool.open_elastic(400)
    eng.step([(h, toks[:40], [])])
    eng.step([(h, prompt(CONFIGS["full"], 9, 77), [])])
    h.truncate([40])
    check(eng.step([(h, toks[40:], list(range(20)))]),
          want_logits(models, "full", toks)[40:], "float32")


# ---------------------------------------------------------------------------
# generation
# ---------------------------------------------------------------------------

def greedy(models, name, toks, n):
    """Greedy continuation by the oracle, and the smallest lead a chosen token
    had over the runner-up, in spreads of the logits."""
    toks, lead = list(toks), []
    for _ in range(n):
        lg = want_logits(models, name, toks)[-1]
        top = lg.topk(2).values
        lead.append(float((top[0] - top[1]) / lg.std()))
        toks.append(int(lg.argmax()))
    return toks[-n:], lead


def agree(got, models, name, p, dt):
    want, lead = greedy(models, name, p, len(got))
    tol = 1e-3 if dt == "float32" else 0.2
    for g, w, l in zip(got, want, lead):
        if l < tol:
            return          # a close call: both continuations are right
        assert g == w


@kinds
def test_generate_greedy(models, dev, dt, monkeypatch):
    eng = engine(models, "full", dev, dt, monkeypatch)
    ps = [prompt(CONFIGS["full"], 21, s) for s in range(3)]
    out = eng.generate_greedy(torch.tensor(ps), 40)
    assert out.shape == (3, 40)
    for p, o in zip(ps, out.tolist()):
        agree(o, models, "full", p, dt)
    assert eng.kv_pool.free_page_count() == eng.kv_pool.n_pages


@kinds
def test_scheduler(models, dev, dt, monkeypatch):
    """More requests than places and pages, prompts longer than a step."""
    eng = engine(models, "full", dev, dt, monkeypatch, tokens=240)
    s = BatchScheduler(eng, max_batch=3, chunk_tokens=24)
    lens = [(50, 20), (3, 30), (75, 5), (1, 12), (20, 33), (31, 1)]
    ps = [prompt(CONFIGS["full"], n, seed=n) for n, _ in lens]
    reqs = [s.submit(p, m) for p, (_, m) in zip(ps, lens)]
    peak = 0
    while s.step():
        peak = max(peak, len(s.running))
    assert peak == 3 and all(r.done for r in reqs)
    for p, r, (_, m) in zip(ps, reqs, lens):
        assert len(r.output) == m
        agree(r.output, models, "full", p, dt)
    assert eng.kv_pool.free_page_count() == eng.kv_pool.n_pages
    assert eng.kv_pool.tokens_left == eng.kv_pool.max_tokens


def test_scheduler_limits(models, monkeypatch):
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    s = BatchScheduler(eng)
    with pytest.raises(ValueError):
        s.submit([], 4)
    with pytest.raises(ValueError):
        s.submit([1] * 60, 10)
    first = want_logits(models, "full", [5, 6, 7])[-1].argmax()
    r = s.submit([5, 6, 7], 10, eos_token_id=int(first))
    g = torch.Generator().manual_seed(1)
    q = s.submit([5, 6, 7], 4, do_sample=True, top_k=1, generator=g)
    s.run()
    assert r.output == [int(first)]
    assert q.output[0] == int(first) and len(q.output) == 4


def test_scheduler_runs_other_families():
    eng = LocalEngine("llama-tiny", kv_max_tokens=512)
    ids = torch.randint(0, 1000, (1, 9), generator=torch.Generator().manual_seed(2))
    want = eng.generate_greedy(ids, 5)[0].tolist()
    s = BatchScheduler(eng, chunk_tokens=4)
    r = s.submit(ids[0].tolist(), 5)
    other = s.submit([3, 4], 3)
    s.run()
    assert r.output == want and len(other.output) == 3


@GPU
@pytest.mark.parametrize("dt", ["float32", "bfloat16"])
def test_graph_replays_equal_eager_steps(models, dt, monkeypatch):
    """Many replays of a captured decode step, with eager steps and new
    sequences in between, each against the eager step."""
    eng = engine(models, "full", "cuda:0", dt, monkeypatch, tokens=1024)
    ref = engine(models, "full", "cuda:0", dt, monkeypatch, tokens=1024)
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
        torch.testing.assert_close(got, want, rtol=1e-5, atol=1e-5)
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
    path, _, cfg = models["full"]
    be = StackBackend(resolve_config(path), 0, len(cfg["layers"]),
                      device="cuda:0", checkpoint_dir=path, kv_max_tokens=8192)
    ref = BlockStack(resolve_config(path), 0, len(cfg["layers"]), device="cuda:0")
    from bloombee_amd.server.from_pretrained import load_block_weights
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
# command line, swarm, training
# ---------------------------------------------------------------------------

@kinds
@pytest.mark.parametrize("name", ["full", "odd"])
def test_trace_replay(models, name, dev, dt, tmp_path, monkeypatch, capsys):
    from bloombee_amd.cli import trace_run
    cfg = CONFIGS[name]
    a, b = prompt(cfg, 40, 1), prompt(cfg, 20, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 29]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:2], "want": []},
                                {"id": "a", "tokens": a[30:31], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[31:32], "want": [0]},
                                {"id": "b", "tokens": b[2:3], "want": [0]}], "end": []},
        {"step": 3, "entries": [{"id": "b", "tokens": b[3:], "want": [16]},
                                {"id": "a", "tokens": a[32:], "want": [7]}],
         "end": ["a", "b"]},
        # the same names once more, on used pages
        {"step": 4, "entries": [{"id": "a", "tokens": b, "want": [19]}], "end": ["a"]},
    ]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps))))
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    rc = trace_run.main(["--model", models[name][0], "--dtype", dt, "--out",
                         str(tmp_path), "--max-tokens", "128", "--device", dev])
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
    """A server and a client on one checkpoint folder, hidden states in 32 bits."""
    from bloombee_amd.client.config import ClientConfig
    from bloombee_amd.models import auto
    from bloombee_amd.net.dht import Dht
    from bloombee_amd.server import Server
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", dt)
    path, _, cfg = models["odd"]
    boot = Dht()
    srv = Server(path, initial_peers=[boot.endpoint], block_indices=(0, 3),
                 update_period=5.0, device=dev)
    srv.run_in_background()
    try:
        m = auto.AutoDistributedModelForCausalLM.from_pretrained(
            path, client_config=ClientConfig(initial_peers=[boot.endpoint]),
            device=dev)
        p = prompt(cfg, 12, 4)
        out = m.generate(torch.tensor([p], device=dev),
                         max_new_tokens=8)[0].tolist()
        assert out[:12] == p
        agree(out[12:], models, "odd", p, dt)
    finally:
        srv.shutdown()
        boot.shutdown()


def test_block_range_must_hold_the_shared_layer(models, monkeypatch):
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    cfg = resolve_config(models["full"][0])
    BlockStack(cfg, 1, 3).make_kv(64)
    with pytest.raises(RuntimeError, match="KV of layer 1"):
        BlockStack(cfg, 2, 4).make_kv(64)


@pytest.mark.parametrize("dev", ["cpu", pytest.param("cuda:0", marks=GPU)])
def test_offloaded_blocks(models, dev, monkeypatch):
    """Blocks of unlike shapes stream through one arena."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    from bloombee_amd.offload import OffloadPolicy
    from bloombee_amd.offload.weights import OffloadedBlockStack
    from bloombee_amd.server.from_pretrained import load_block_weights
    path, w, cfg = models["full"]
    stack = BlockStack(resolve_config(path), 0, 5, device=dev)
    for i, blk in enumerate(stack.blocks):
        load_block_weights(blk, path, i)
    off = OffloadedBlockStack(stack, OffloadPolicy(weight_gpu_percent=20.0))
    toks = prompt(cfg, 50, 5)
    col = []
    oracle.forward(torch.tensor(toks), w, cfg, col)
    x = (w["embed"][toks] + w["pos"][:50]).float()[None].to(dev)
    kv = off.make_kv(128).allocate(1, 50)
    out = []
    for a, b in ((0, 31), (31, 49), (49, 50)):
        kv.extend(b - a)
        out.append(off.forward_inference(
            x[:, a:b], kv, torch.tensor([a], dtype=torch.int32, device=dev)))
    got = torch.cat(out, 1)[0].cpu().double()
    torch.testing.assert_close(got, col[-1], rtol=1e-4, atol=1e-4)


def test_training_path(models, monkeypatch):
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    path, w, cfg = models["full"]
    eng = LocalEngine(path, kv_max_tokens=64)
    toks = prompt(cfg, 45, 5)
    col = []
    oracle.forward(torch.tensor(toks), w, cfg, col)
    x = (w["embed"][toks] + w["pos"][:45]).float()[None].requires_grad_(True)
    y = eng.stack.forward_train(x)
    torch.testing.assert_close(y[0].double(), col[-1], rtol=1e-4, atol=1e-4)
    y.square().mean().backward()
    assert torch.isfinite(x.grad).all() and x.grad.abs().max() > 0


def test_deep_prompts(models, monkeypatch):
    """Per-layer prompt vectors are added to the residual before each block."""
    monkeypatch.setenv("BBAMD_TORCH_DTYPE", "float32")
    eng = LocalEngine(models["full"][0], kv_max_tokens=64)
    x = torch.randn(1, 20, 192, generator=torch.Generator().manual_seed(0))
    dp = torch.randn(5, 6, 192, generator=torch.Generator().manual_seed(1))
    kv = eng.kv_pool.allocate(1, 20)
    kv.extend(20)
    keep = x.clone()
    got = eng.stack.forward_inference(x, kv, torch.zeros(1, dtype=torch.int32),
                                      deep_prompts=dp)
    torch.testing.assert_close(x, keep)     # the caller's tensor is its own
    want = eng.stack.forward_train(x, deep_prompts=dp)
    torch.testing.assert_close(got, want, rtol=1e-4, atol=1e-4)


def test_config_reader():
    cfg = MubasunConfig.from_dict(CONFIGS["odd"])
    assert (cfg.hidden_size, cfg.vocab_size, cfg.num_hidden_layers) == (90, 101, 3)
    assert cfg.hidden_dtype == torch.float32 and cfg.norm_groups == 5
    for change in (lambda c: c["norm"].update(groups=7),
                   lambda c: c["layers"][0].update(type="recurrent"),
                   lambda c: c["layers"][0]["mixer"].update(kv_heads=2),
                   lambda c: c["layers"][1]["mixer"].update(kv_from=2),
                   lambda c: c["layers"][2]["mixer"].update(kv_from=1),
                   lambda c: c["layers"][1]["mlp"].update(kind="sparse"),
                   lambda c: c["layers"][0]["mlp"]["router"].update(top=9)):
        bad = copy.deepcopy(CONFIGS["odd"])
        change(bad)
        with pytest.raises(ValueError):
            MubasunConfig.from_dict(bad)
    with pytest.raises(KeyError):
        from bloombee_amd.models.base import model_type_of
        model_type_of({"architecture": "Nothing"})


def test_presets_resolve():
    for name in ("mubasun-tiny", "mubasun-64e-4l", "mubasun-8b-4l"):
        assert resolve_config(name).model_type == "mubasun"
    eng = LocalEngine("mubasun-tiny", kv_max_tokens=256)
    out = eng.generate_greedy(torch.tensor([[1, 2, 3]]), 4)
    assert out.shape == (1, 4)


def test_wrong_shapes_are_refused(models, tmp_path, monkeypatch):
    path, w, cfg = models["odd"]
    bad = {k: v.bfloat16() for k, v in w.items()}
    bad["l1.mlp.up"] = bad["l1.mlp.up"][:-1].contiguous()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(bad, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l.*mlp.up"):
        LocalEngine(str(tmp_path), kv_max_tokens=64)


def test_no_lockstep_step_on_host_prefix_sessions(models, monkeypatch):
    from bloombee_amd.kv.batch import lockstep_batch
    eng = engine(models, "full", "cpu", "float32", monkeypatch, tokens=64)
    h = eng.kv_pool.allocate(1, 32)
    h._pos_offset = 4
    with pytest.raises(PagedKVError):
        lockstep_batch(h, torch.zeros(1, dtype=torch.int32), 1, 1)
