"""Replay a trace of token ids through a model, step by step, and write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": []}

All entries of a step run as one ragged batch on LocalEngine.step, the step
function of the batch scheduler: portions of prompts beside single tokens, each
continuing from its request's cache. `want` names the places whose logits go
to OUT/<step>.f32 (32-bit floats, [wanted, vocab], entry order); `end` frees
requests. After every step a line "done <step>" is printed. Nothing is sampled.

The KV pool holds --max-tokens and state slots for --max-requests, so pages and
slots of ended requests are used again.
Steps in which every entry brings one token and wants its logits replay the
engine's captured decode graph, as generation does.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

def ensure_built(block_cls) -> None:
    """Compile the extension modules this model's blocks run on, if they are
    missing: hip_modules of ragged-batch blocks, _hip_ops for the others. A
    lock file lets concurrent first calls share one compilation."""
    import fcntl

    from bloombee_amd import ops as _ops

    ops_dir = os.path.dirname(os.path.abspath(_ops.__file__))
    root = os.path.dirname(os.path.dirname(ops_dir))
    need = getattr(block_cls, "hip_modules", ("_hip_ops",))
    path = lambda m: os.path.join(ops_dir, m + ".so")
    if all(os.path.exists(path(m)) for m in need):
        return
    with open(os.path.join(ops_dir, ".build.lock"), "w") as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        missing = [m for m in need if not os.path.exists(path(m))]
        if missing:
            import importlib.util
            spec = importlib.util.spec_from_file_location(
                "bbamd_setup", os.path.join(root, "setup.py"))
            mod = importlib.util.module_from_spec(spec)
            spec.loader.exec_module(mod)
            mod.build(missing, verbose=False)
    if "_hip_ops" in need:
        # this module was looked for when its dispatch layer was imported
        import importlib

        from bloombee_amd.ops import interface
        importlib.reload(interface)
        importlib.reload(_ops)


class TraceReplay:
    """Requests by name over one LocalEngine."""

    def __init__(self, engine):
        self.engine = engine
        self.live = {}

    def step(self, line: dict):
        """Runs one step; returns its wanted logits, (wanted, V)."""
        entries = []
        for e in line["entries"]:
            h = self.live.get(e["id"])
            if h is None:
                h = self.live[e["id"]] = self.engine.kv_pool.open_elastic(
                    self.engine.config.max_position_embeddings)
            entries.append((h, e["tokens"], e.get("want") or []))
        logits = None
        if entries:
            if all(len(t) == 1 and list(w) == [0] for _, t, w in entries):
                logits = self.engine.decode([(h, t[0]) for h, t, _ in entries])
            else:
                logits = self.engine.step(entries)
        for rid in line.get("end") or []:
            self.live.pop(rid).close()
        return logits


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=["bfloat16", "float32"])
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="KV tokens that live requests hold at any time")
    ap.add_argument("--max-requests", type=int, default=4,
                    help="requests live at any time (state slots of models "
                         "with recurrent layers)")
    ap.add_argument("--device", default="cuda:0")
    args = ap.parse_args(argv)

    os.environ["BBAMD_TORCH_DTYPE"] = args.dtype
    import torch

    from bloombee_amd.models.auto import get_block_class
    from bloombee_amd.models.base import resolve_config

    cfg = resolve_config(args.model)
    if args.device.startswith("cuda"):
        if not torch.cuda.is_available():
            print("trace_run: no GPU", file=sys.stderr)
            return 2
        ensure_built(get_block_class(cfg.model_type))
    # 32-bit products stay 32-bit
    torch.backends.cuda.matmul.allow_tf32 = False
    torch.set_float32_matmul_precision("highest")

    from bloombee_amd.engine import LocalEngine

    replay = TraceReplay(LocalEngine(args.model, device=args.device,
                                     kv_max_tokens=args.max_tokens,
                                     max_seqs=args.max_requests))
    for text in sys.stdin:
        if not text.strip():
            continue
        line = json.loads(text)
        logits = replay.step(line)
        if logits is not None and logits.shape[0]:
            data = logits.float().cpu().contiguous().numpy().astype("<f4")
            with open(os.path.join(args.out, f"{line['step']}.f32"), "wb") as f:
                f.write(data.tobytes())
        elif args.device.startswith("cuda"):
            torch.cuda.synchronize()
        print(f"done {line['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
