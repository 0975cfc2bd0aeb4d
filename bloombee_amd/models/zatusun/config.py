"""Zatusun family config.

Native config.json keys: `width`, `vocab`, `max_positions`, `norm` (eps),
`embedding` (scale), `logit_softcap`, `layers`, one entry per layer with its
mixer's type and sizes and its feed-forward (moe or none), and `loop`: the layers
start .. stop - 1 run `times` times in a row. They map onto the common
ModelConfig fields; what differs per layer stays in `layers`.

To the rest of the framework a layer run is a layer: num_hidden_layers counts
runs, and the runs of a looped layer have caches and states of their own and
weights in common (`weights_of`).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import List, NamedTuple, Optional

import torch

from bloombee_amd.models.base import ModelConfig
from bloombee_amd.ops import mixers
from bloombee_amd.ops.mixers import DiffSpec, HgrnSpec, LatentSpec
from bloombee_amd.ops.ragged import GluSpec, RopeSpec, pad_head

GLU_SLOPE, GLU_SHIFT = 1.702, 1.0   # of the experts' activation


class Run(NamedTuple):
    """One run of a layer."""
    layer: int
    enters: Optional[int]   # the pass that begins with this run
    first: int              # the first run of the same layer


def _latent(heads, dim, rot, vdim, rank, q_rank, mlp, base=10000.0,
            scale=None, scaling=None) -> dict:
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
        "kv_rank": rank, "q_rank": q_rank, "scale": scale or (dim + rot) ** -0.5,
        "rot": {"base": base, "dims": rot, "scaling": scaling or {
            "factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}}


def _diff(heads, kv_heads, dim, vdim, mlp, chunk, rot=None, base=500000.0,
          diff=0.5, scaling=None) -> dict:
    return {"type": "attention", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "scale": dim ** -0.5, "diff": diff, "mask": {"size": chunk},
        "rot": {"base": base, "dims": rot or dim, "scaling": scaling or {
            "factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}}


def _hgrn2(heads, dim, vdim, mlp) -> dict:
    return {"type": "hgrn2", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim}}


def _moe(experts, top, ff, limit=7.0) -> dict:
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff, "limit": limit}}


def _preset(width, vocab, layers, loop=None, positions=8192, scale=8.0,
            cap=30.0, eps=1e-5) -> dict:
    return dict(width=width, vocab=vocab, norm={"eps": eps}, layers=layers,
                loop=loop, max_positions=positions, logit_softcap=cap,
                embedding={"scale": scale})


ZATUSUN_PRESETS = {
    # mixers of llama-3-8b's width beside their like kinds in other families,
    # without feed-forward: 32 latent heads of 128
    "zatusun-8b-latent-4l": _preset(4096, 32000, [
        _latent(32, 128, 64, 128, 512, 1536, None) for _ in range(4)]),
    # 16 heads of two maps of 128, 4 key/value heads: as many queries, keys and
    # values as 32 heads of 128 with 8 key/value heads
    "zatusun-8b-diff-4l": _preset(4096, 32000, [
        _diff(16, 4, 128, 256, None, 8192) for _ in range(4)]),
    # 16 recurrent heads of 128 channels and 256 values
    "zatusun-8b-hgrn2-4l": _preset(4096, 32000, [
        _hgrn2(16, 128, 256, None) for _ in range(4)]),
    # all kinds with mixtral's experts; two layers run twice
    "zatusun-8x7b-4l": _preset(4096, 32000, [
        _hgrn2(16, 128, 256, _moe(8, 2, 14336)),
        _diff(16, 4, 128, 256, _moe(8, 2, 14336), 2048),
        _latent(32, 128, 64, 128, 512, 1536, _moe(8, 2, 14336))],
        loop={"start": 0, "stop": 1, "times": 2}),
    "zatusun-tiny": _preset(192, 320, [
        _latent(4, 32, 16, 40, 80, 96, _moe(5, 2, 64)),
        _hgrn2(3, 32, 40, _moe(6, 3, 64)),
        _diff(4, 2, 24, 40, None, 16, rot=12), _hgrn2(2, 40, 56, None)],
        loop={"start": 1, "stop": 3, "times": 2}, positions=512),
}


@dataclass
class ZatusunConfig(ModelConfig):
    model_type: str = "zatusun"

    @classmethod
    def from_dict(cls, d: dict) -> "ZatusunConfig":
        d = copy.deepcopy(d)
        layers = d["layers"]
        first = layers[0]["mixer"]
        mapped = {
            "hidden_size": int(d["width"]),
            "vocab_size": int(d["vocab"]),
            "max_position_embeddings": int(d["max_positions"]),
            "rms_norm_eps": float(d["norm"]["eps"]),
            "num_attention_heads": int(first["heads"]),
            "num_key_value_heads": int(first.get("kv_heads", first["heads"])),
            "head_dim": int(first["dim"]),
        }
        cfg = super().from_dict({**d, **mapped})
        cfg._check()
        cfg.num_hidden_layers = len(cfg.runs)
        return cfg

    def _check(self) -> None:
        loop = self.loop
        if loop is not None and not (
                0 <= loop["start"] < loop["stop"] <= len(self.layers)
                and loop["times"] >= 1):
            raise ValueError(f"cannot loop over layers {loop} of "
                             f"{len(self.layers)}")
        for i, layer in enumerate(self.layers):
            mx, mlp = layer["mixer"], layer.get("mlp")
            if layer["type"] not in ("latent_attention", "attention", "hgrn2"):
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer["type"] != "hgrn2":
                size = (mx["rot_dim"] if layer["type"] == "latent_attention"
                        else mx["dim"])
                dims = mx["rot"]["dims"]
                if dims % 2 or not 0 < dims <= size:
                    raise ValueError(f"layer {i}: cannot rotate {dims} of "
                                     f"{size} dimensions")
            if layer["type"] == "attention":
                if mx["heads"] % mx["kv_heads"]:
                    raise ValueError(f"layer {i}: {mx['heads']} heads do not "
                                     f"share {mx['kv_heads']} key heads evenly")
                if (mx.get("mask") or {}).get("size", 1) < 1:
                    raise ValueError(f"layer {i}: empty chunks")
            if mlp is None:
                continue
            if mlp["kind"] != "moe":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")
            rt = mlp["router"]
            if not 1 <= rt["top"] <= rt["experts"] <= 1024:
                raise ValueError(f"layer {i}: cannot choose {rt['top']} of "
                                 f"{rt['experts']} experts")

    @property
    def layers(self) -> list:
        return self.extras["layers"]

    @property
    def loop(self) -> Optional[dict]:
        return self.extras.get("loop")

    @property
    def runs(self) -> List[Run]:
        """The layer runs in order."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return [Run(i, None, i) for i in range(n)]
        a, b, times = loop["start"], loop["stop"], loop["times"]
        out = [Run(i, None, i) for i in range(a)]
        for t in range(times):
            out += [Run(i, t if i == a else None, i) for i in range(a, b)]
        return out + [Run(i, None, i + (times - 1) * (b - a))
                      for i in range(b, n)]

    def weights_of(self, layer: int) -> int:
        return self.runs[layer].first

    @property
    def hidden_columns(self) -> int:
        """A pass reads the embedding output again, so it travels along:
        [residual | embedding output]."""
        return self.hidden_size * (1 if self.loop is None else 2)

    @property
    def embedding_scale(self) -> float:
        return float(self.extras["embedding"]["scale"])

    @property
    def learned_positions(self) -> bool:
        return True

    @property
    def logit_softcap(self) -> float:
        return float(self.extras.get("logit_softcap") or 0.0)

    @property
    def norm_offset(self) -> float:
        """Layer and final norms scale by one plus their stored weight."""
        return 1.0

    @property
    def hidden_dtype(self) -> torch.dtype:
        """The residual is 32-bit whatever the compute type."""
        return torch.float32

    def rotation(self, layer: int):
        """(turns per position, factor of cosine and sine) of a layer."""
        kind, rot = self.layers[layer]["type"], self.layers[layer]["mixer"]["rot"]
        base, dims, s = float(rot["base"]), int(rot["dims"]), rot.get("scaling")
        if s is None:
            return mixers.rotary_turns(base, dims), 1.0
        if kind == "latent_attention":
            return mixers.yarn_turns(base, dims, s["factor"], s["original"],
                                     s["fast"], s["slow"])
        return mixers.banded_turns(base, dims, s["factor"], s["low"], s["high"],
                                   s["original"]), 1.0

    def mixer_spec(self, layer: int):
        """Sizes and constants of a layer's mixer."""
        kind, mx = self.layers[layer]["type"], self.layers[layer]["mixer"]
        heads, dim, vdim = (int(mx[k]) for k in ("heads", "dim", "vdim"))
        if kind == "latent_attention":
            return LatentSpec(
                heads=heads, dim=dim, rot=int(mx["rot_dim"]),
                rot_dims=int(mx["rot"]["dims"]), vdim=vdim,
                q_rank=int(mx["q_rank"]), rank=int(mx["kv_rank"]),
                scale=float(mx["scale"]), window=0, eps=self.rms_norm_eps,
                amp=self.rotation(layer)[1])
        if kind == "attention":
            diff = float(mx["diff"])
            return DiffSpec(
                RopeSpec(heads=heads, kv_heads=int(mx["kv_heads"]), maps=2,
                         dim=dim, vdim=vdim, rot_dims=int(mx["rot"]["dims"])),
                scale=float(mx["scale"]), lam=diff, factor=1 - diff,
                eps=self.rms_norm_eps,
                chunk=int((mx.get("mask") or {}).get("size") or 0))
        return HgrnSpec(heads=heads, dim=dim, vdim=vdim, eps=self.rms_norm_eps,
                        router_n=heads * dim)

    def glu_spec(self, layer: int) -> GluSpec:
        limit = self.layers[layer]["mlp"]["expert"]["limit"]
        return GluSpec(limit=float(limit), slope=GLU_SLOPE, shift=GLU_SHIFT)

    def kv_layout(self, start: int, end: int) -> dict:
        """PagedKVCache geometry of the runs [start, end): a plane of [latent |
        rotated part], planes of keys (two maps a head) and values, or a state."""
        heads, dims, vdims, layout, states = [], [], [], [], []
        for run in self.runs[start:end]:
            s = self.mixer_spec(run.layer)
            kind = self.layers[run.layer]["type"]
            if kind == "latent_attention":
                row = (1, s.ck, 0, "k", None)
            elif kind == "attention":
                r = s.rope
                row = (r.kv_heads, r.maps * r.dk, pad_head(r.vdim), "kv", None)
            else:
                row = (0, 0, 0, "none", (s.heads, s.dim, s.vdim))
            for out, v in zip((heads, dims, vdims, layout, states), row):
                out.append(v)
        return dict(num_kv_heads=heads, head_dim=dims, v_head_dim=vdims,
                    layout=layout, state_shapes=states)
