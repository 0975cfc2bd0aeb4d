"""Driver benchmark contract: flagship decode throughput.

Measures BASELINE.json's metric — decode tokens/sec (+ p50 step latency) for
Llama-3-8B greedy decode, sharded over N MI355X workers as a micro-batched
pipeline over RCCL/xGMI (bloombee_amd/parallel/pipeline.py). Synthetic data,
random-init weights (no network in this environment), bf16.

Weak scaling: global_batch = batch_per_gpu * N (per-GPU work fixed as N grows).

  python bench.py --gpus N --steps K --warmup W
  (N>1 is launched by the driver via torch.distributed.run, one rank per GPU)
"""
from __future__ import annotations

import argparse
import json
import os
import time

import torch


def stage_max_pos(model: str) -> int:
    from bloombee_amd.models.base import resolve_config

    return resolve_config(model).max_position_embeddings


def run_swarm(args):
    """The REAL decentralized serving stack under the bench contract: one
    Server (DHT + rpc_inference handler + paged-KV backend) per rank/GPU,
    the client on rank 0, every activation hop on the RCCL/xGMI device
    plane (net/channels.py) — VERDICT r01 item 1's "bench mode that runs
    the real Server/session stack"."""
    import torch.distributed as dist
    import torch.nn.functional as F

    from bloombee_amd import ops
    from bloombee_amd.client.config import ClientConfig
    from bloombee_amd.client.routing import RemoteSequenceManager
    from bloombee_amd.client.session import InferenceSession
    from bloombee_amd.models.base import resolve_config
    from bloombee_amd.net.channels import channels
    from bloombee_amd.net.dht import Dht
    from bloombee_amd.parallel.pipeline import init_distributed, layer_range
    from bloombee_amd.server import Server

    device = init_distributed("cpu" if args.device == "cpu" else "auto")
    if args.device:
        device = args.device
    rank = dist.get_rank() if dist.is_initialized() else 0
    world = dist.get_world_size() if dist.is_initialized() else 1
    on_gpu = device.startswith("cuda")
    channels.enable(device)  # collective when dist is initialized

    cfg = resolve_config(args.model)
    global_batch = args.batch_per_gpu * world
    session_len = args.prompt + args.steps + args.warmup + 8
    kv_tokens = global_batch * ((session_len + 15) // 16 + 1) * 16 + 1024

    # micro-batch policy for the GPU swarm: decode kernels lose ~2x below 8
    # rows (bench_kernels), so slices are per-GPU-batch sized; single-stage
    # worlds never split
    os.environ.setdefault("BBAMD_MICRO_BATCH_SIZE", str(args.batch_per_gpu))
    os.environ.setdefault("BBAMD_MIN_BATCH_TO_SPLIT",
                          str(2 * args.batch_per_gpu))

    # loopback DHT bootstrap: rank 0 owns it and shares the endpoint
    if dist.is_initialized():
        boot_ep = [None]
        boot = None
        if rank == 0:
            boot = Dht()
            boot_ep = [boot.endpoint]
        dist.broadcast_object_list(boot_ep, src=0)
        boot_ep = boot_ep[0]
    else:
        boot = Dht()
        boot_ep = boot.endpoint

    start, end = layer_range(cfg.num_hidden_layers, rank, world)
    server = Server(args.model, initial_peers=[boot_ep],
                    block_indices=(start, end), device=device, seed=0,
                    kv_max_tokens=kv_tokens, update_period=10.0,
                    max_batch_size=max(2048, global_batch))
    server.run_in_background()

    def _wait_done(dht):
        while not dht.get("bench_done"):
            time.sleep(0.5)

    if rank != 0:
        # workers serve until the client posts the done flag (no dist
        # collectives during decode: the data plane owns the comm)
        local_dht = server.dht
        _wait_done(local_dht)
        server.shutdown()
        channels.disable()
        if dist.is_initialized():
            dist.destroy_process_group()
        return

    # ---- rank 0: the client -------------------------------------------
    ccfg = ClientConfig(initial_peers=[boot_ep], keep_history=False,
                        update_period=10.0)
    manager = RemoteSequenceManager(ccfg, args.model, cfg.num_hidden_layers)
    deadline = time.monotonic() + 120
    while True:
        try:
            manager.update()
            route = manager.make_sequence(0, cfg.num_hidden_layers)
            if len(route) == world:
                break
        except Exception:
            pass
        if time.monotonic() > deadline:
            raise RuntimeError("swarm did not converge to a full route")
        time.sleep(0.5)

    gen = torch.Generator().manual_seed(0)
    dt = cfg.dtype
    dev = torch.device(device)
    embed = (torch.randn(cfg.vocab_size, cfg.hidden_size, generator=gen)
             .mul_(0.02).to(dt).to(dev))
    norm_w = torch.ones(cfg.hidden_size, dtype=dt, device=dev)
    lm_head_w = embed if cfg.tie_word_embeddings else (
        torch.randn(cfg.vocab_size, cfg.hidden_size, generator=gen)
        .mul_(0.02).to(dt).to(dev))

    session = InferenceSession(manager, max_length=session_len, config=ccfg)
    prompt = torch.randint(0, cfg.vocab_size, (global_batch, args.prompt),
                           generator=gen)
    CH = 512
    out = None
    for c0 in range(0, args.prompt, CH):
        chunk = prompt[:, c0:c0 + CH].to(dev)
        out = session.step(F.embedding(chunk, embed))

    def _lm_head(hidden_last):
        y = ops.rms_norm(hidden_last, norm_w, cfg.rms_norm_eps)
        return F.linear(y, lm_head_w).float().argmax(-1)

    ids = _lm_head(out[:, -1])
    for _ in range(args.warmup):
        out = session.step(F.embedding(ids.view(-1, 1), embed))
        ids = _lm_head(out[:, -1])
    if on_gpu:
        torch.cuda.synchronize()
    t0 = time.monotonic()
    step_ms = []
    for _ in range(args.steps):
        s0 = time.monotonic()
        out = session.step(F.embedding(ids.view(-1, 1), embed))
        ids = _lm_head(out[:, -1])
        if on_gpu:
            torch.cuda.synchronize()
        step_ms.append((time.monotonic() - s0) * 1e3)
    if on_gpu:
        torch.cuda.synchronize()
    elapsed = time.monotonic() - t0

    session.close()
    manager.shutdown()
    # release the workers, then spin down
    boot.store("bench_done", "client", True, time.time() + 600)
    p50 = sorted(step_ms)[len(step_ms) // 2]
    result = {
        "metric": f"decode tokens/sec, {args.model} greedy, serving stack over RCCL/xGMI",
        "value": round(global_batch * args.steps / elapsed, 2),
        "unit": "tokens/s",
        "n_gpus": world,
        "steps": args.steps,
        "warmup": args.warmup,
        "ms_per_step": round(elapsed * 1000 / args.steps, 3),
        "higher_is_better": True,
        "scaling": "weak",
        "vs_baseline": None,
        "dtype": "bfloat16" if cfg.torch_dtype == "bfloat16" else cfg.torch_dtype,
        "data": "synthetic",
        "config": {
            "model": args.model,
            "global_batch": global_batch,
            "seq_len": args.prompt,
            "parallelism": f"swarm-pp{world}",
            "p50_step_ms": round(p50, 3),
        },
    }
    print(json.dumps(result))
    time.sleep(1.0)
    server.shutdown()
    boot.shutdown()
    channels.disable()
    if dist.is_initialized():
        dist.destroy_process_group()


# (model, closest family of equal layer size); both run LAYERS blocks
LAYER_PAIRS = [("mubasun-8b-4l", "llama-3-8b"),
               ("mubasun-8x7b-4l", "mixtral-8x7b-4l"),
               ("mubasun-64e-4l", None),
               ("risepel-8b-latent-4l", "mubasun-8b-4l"),
               ("risepel-8b-gla-4l", "mubasun-8b-4l"),
               ("risepel-8b-4l", "llama-3-8b"),
               ("vumedra-8b-attn-4l", "llama-3-8b"),
               ("vumedra-8b-mlstm-4l", "risepel-8b-gla-4l"),
               ("vumedra-8b-rglru-4l", "risepel-8b-gla-4l"),
               ("vumedra-8x7b-4l", "mubasun-8x7b-4l"),
               ("zatusun-8b-latent-4l", "risepel-8b-latent-mixer-4l"),
               ("zatusun-8b-diff-4l", "vumedra-8b-attn-mixer-4l"),
               ("zatusun-8b-hgrn2-4l", "risepel-8b-gla-mixer-4l"),
               ("zatusun-8x7b-4l", "mubasun-8x7b-4l")]
LAYERS = 4


def _layer_numbers(model: str, args) -> dict:
    """Prefill and decode throughput of LAYERS blocks of `model` (random
    weights, lockstep sessions, decode replayed from a captured graph where the
    family's step can be captured)."""
    from bloombee_amd.engine import BlockStack
    from bloombee_amd.models.base import resolve_config

    cfg = resolve_config(model)
    dev = args.device or ("cuda:0" if torch.cuda.is_available() else "cpu")
    on_gpu = dev.startswith("cuda")
    stack = BlockStack(cfg, 0, LAYERS, device=dev, seed=0)
    W = cfg.hidden_columns
    gen = torch.Generator().manual_seed(1)
    sync = torch.cuda.synchronize if on_gpu else (lambda: None)
    out = {}

    def timed(fn):
        for _ in range(args.warmup):
            fn()
        sync()
        t0 = time.monotonic()
        for _ in range(args.steps):
            fn()
        sync()
        return (time.monotonic() - t0) / args.steps

    for B, T in ((1, 512), (1, 2048), (8, 512)):
        kv = stack.make_kv(B * T).allocate(B, T)
        x = (torch.randn(B, T, W, generator=gen).to(cfg.hidden_dtype).to(dev))
        pos = torch.zeros(B, dtype=torch.int32, device=dev)
        kv.extend(T)
        t = timed(lambda: stack.forward_inference(x, kv, pos))
        out[f"prefill {B}x{T}"] = round(B * T / t, 1)
        kv.close()

    for B, ctx in ((1, 1024), (32, 1024), (32, 4096), (128, 1024)):
        kv = stack.make_kv(B * (ctx + 16)).allocate(B, ctx + 16)
        kv.extend(ctx)
        x = torch.randn(B, 1, W, generator=gen).to(cfg.hidden_dtype).to(dev)
        pos = torch.full((B,), ctx - 1, dtype=torch.int32, device=dev)
        kv.page_table()
        step = lambda: stack.forward_inference(x, kv, pos)
        step()
        # mixtral's routing (bincount) cannot be captured: it runs eagerly
        if on_gpu and cfg.model_type != "mixtral":
            step()
            sync()
            graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(graph):
                step()
            step = graph.replay
        t = timed(step)
        out[f"decode B{B} ctx{ctx}"] = round(B / t, 1)
        kv.close()
    return out


def run_layers(args):
    """Tokens/s through LAYERS blocks: a model beside its closest relative of
    equal layer size, on the same inputs."""
    rows = {}
    for model, like in LAYER_PAIRS:
        if args.pair and args.pair not in model:
            continue
        rows[model] = _layer_numbers(model, args)
        if like and like not in rows:
            rows[like] = _layer_numbers(like, args)
        if like:
            rows[f"{model} / {like}"] = {
                k: round(rows[model][k] / rows[like][k], 3)
                for k in rows[model]}
        if torch.cuda.is_available():
            torch.cuda.empty_cache()
    first = next(iter(rows.values()))
    print(json.dumps({
        "metric": f"decode tokens/sec through {LAYERS} layers, B32 ctx1024",
        "value": first["decode B32 ctx1024"], "unit": "tokens/s",
        "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "higher_is_better": True, "vs_baseline": None, "dtype": "bf16",
        "data": "synthetic", "config": {"mode": "layers", "layers": LAYERS},
        "rows": rows}))


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--model", default="llama-3-8b")
    ap.add_argument("--batch-per-gpu", type=int, default=32)
    ap.add_argument("--prompt", type=int, default=2048,
                    help="prompt length prefillled before the timed decode steps")
    ap.add_argument("--device", default=None, help="override (e.g. cpu for tests)")
    ap.add_argument("--micro-batches", type=int, default=0)
    ap.add_argument("--tp", type=int, default=1,
                    help="tensor-parallel degree within the pipeline (world %% tp == 0)")
    ap.add_argument("--tp-mode", default="tensor", choices=["tensor", "expert"],
                    help="what the intra-stage group shards: tensor dims "
                         "(llama TP) or MoE experts (mixtral EP)")
    ap.add_argument("--mode", default="pipeline", choices=["pipeline", "swarm", "layers"],
                    help="pipeline = raw RCCL pipeline stages (flagship); "
                         "swarm = the full decentralized serving stack "
                         "(DHT + sessions + handler) over the same device plane; "
                         "layers = mubasun, risepel and vumedra layers "
                         "beside the closest family's")
    ap.add_argument("--pair", default=None,
                    help="layers mode: only pairs whose model name contains this")
    args = ap.parse_args()

    if args.mode == "swarm":
        run_swarm(args)
        return

    if args.mode == "layers":
        run_layers(args)
        return

    import torch.distributed as dist
    from bloombee_amd.parallel.pipeline import PipelineStage, init_distributed

    device = init_distributed("cpu" if args.device == "cpu" else "auto")
    if args.device:
        device = args.device
    rank = dist.get_rank() if dist.is_initialized() else 0
    world = dist.get_world_size() if dist.is_initialized() else 1
    assert world == args.gpus or not dist.is_initialized(), \
        f"world {world} != --gpus {args.gpus}"
    on_gpu = device.startswith("cuda")

    global_batch = args.batch_per_gpu * world
    session_len = args.prompt + args.steps + args.warmup + 8
    assert session_len <= stage_max_pos(args.model), (
        f"prompt+steps {session_len} exceeds the model's "
        f"max_position_embeddings — shorten --prompt or --steps")
    # KV budget: whole session for every sequence on every rank (page-rounded)
    kv_tokens = global_batch * ((session_len + 15) // 16 + 1) * 16 + 1024

    stage = PipelineStage(args.model, device, global_batch,
                          micro_batches=args.micro_batches,
                          kv_max_tokens=kv_tokens, max_session_len=session_len,
                          tp=args.tp, tp_mode=args.tp_mode)

    gen = torch.Generator().manual_seed(42)
    V = stage.config.vocab_size
    ids = None
    if rank == 0:
        prompt = torch.randint(0, V, (global_batch, args.prompt), generator=gen)
    # ---- prefill (untimed setup; chunked to bound activation memory) ----
    CH = 512
    for c0 in range(0, args.prompt, CH):
        chunk = None
        if rank == 0:
            chunk = prompt[:, c0:c0 + CH]
        ids = stage.prefill_round(chunk, min(CH, args.prompt - c0))

    # ---- warmup ----
    for _ in range(args.warmup):
        ids = stage.decode_round(ids if rank == 0 else None)

    if dist.is_initialized():
        dist.barrier()
    if on_gpu:
        torch.cuda.synchronize()

    step_ms = []
    t0 = time.monotonic()
    if on_gpu and rank == 0:
        ev = [torch.cuda.Event(enable_timing=True) for _ in range(args.steps + 1)]
        ev[0].record()
    for s in range(args.steps):
        ids = stage.decode_round(ids if rank == 0 else None)
        if on_gpu and rank == 0:
            ev[s + 1].record()
    if on_gpu:
        torch.cuda.synchronize()
    if dist.is_initialized():
        dist.barrier()
    if on_gpu:
        torch.cuda.synchronize()
    t1 = time.monotonic()
    elapsed = t1 - t0
    if dist.is_initialized():
        e = torch.tensor([elapsed])
        dist.all_reduce(e, op=dist.ReduceOp.MAX)
        elapsed = float(e)

    if rank == 0:
        if on_gpu:
            step_ms = [ev[i].elapsed_time(ev[i + 1]) for i in range(args.steps)]
        else:
            step_ms = [elapsed / args.steps * 1000] * args.steps
        p50 = sorted(step_ms)[len(step_ms) // 2]
        tokens_per_s = global_batch * args.steps / elapsed
        result = {
            "metric": f"decode tokens/sec, {args.model} greedy, pipeline over RCCL/xGMI",
            "value": round(tokens_per_s, 2),
            "unit": "tokens/s",
            "n_gpus": world,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(elapsed * 1000 / args.steps, 3),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "bfloat16" if stage.config.torch_dtype == "bfloat16" else stage.config.torch_dtype,
            "data": "synthetic",
            "config": {
                "model": args.model,
                "global_batch": global_batch,
                "seq_len": args.prompt,
                "parallelism": (f"pp{world // args.tp}x"
                                f"{'ep' if args.tp_mode == 'expert' else 'tp'}"
                                f"{args.tp}" if args.tp > 1 else f"pp{world}"),
                "micro_batches": stage.M,
                "p50_step_ms": round(p50, 3),
            },
        }
        print(json.dumps(result))
    if dist.is_initialized():
        dist.destroy_process_group()


if __name__ == "__main__":
    main()
