"""Risepel family config.

Native config.json keys: `width`, `vocab`, `norm` (eps), `postln_alpha`,
`logit_softcap` and `layers`, one entry per layer with its mixer's type and
sizes and its feed-forward (dense or none). They map onto the common
ModelConfig fields; what differs per layer stays in `layers`. The rank of the
decay projection of gated linear attention layers is no config key: a
checkpoint's tensors give it (`decay_rank` of the mixer for random weights).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Callable, Optional

import torch

from bloombee_amd.models.base import ModelConfig, kv_shares
from bloombee_amd.ops.mixers import LatentSpec

MAX_POSITIONS = 1 << 20   # positions are rotary: the design has no limit
DECAY_RANK = 16


def _latent(heads, dim, rot, vdim, rank, q_rank, window, ff=None, base=10000.0,
            scale=None, kv_from=None, limit=7.0) -> dict:
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
             "kv_rank": rank, "q_rank": q_rank,
             "rot": {"base": base, "dims": rot},
             "scale": scale or (dim + rot) ** -0.5, "mask": {"size": window}}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mixer, "mlp": _mlp(ff, limit)}


def _gla(heads, dim, vdim, ff=None, tau=16.0, limit=7.0) -> dict:
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                     "tau": tau}, "mlp": _mlp(ff, limit)}


def _mlp(ff, limit) -> Optional[dict]:
    return {"kind": "dense", "ff": ff, "limit": limit} if ff else None


def _preset(width, vocab, layers, alpha=2.0, cap=30.0, eps=1e-5) -> dict:
    return dict(width=width, vocab=vocab, norm={"eps": eps}, layers=layers,
                postln_alpha=alpha, logit_softcap=cap)


RISEPEL_PRESETS = {
    # layers of llama-3-8b's width and feed-forward, 32 latent heads of 128,
    # 1k window
    "risepel-8b-latent-4l": _preset(4096, 32000, [
        _latent(32, 128, 64, 128, 512, 1536, 1024, ff=14336) for _ in range(4)]),
    # the same with 16 recurrent heads of 128 keys and 256 values
    "risepel-8b-gla-4l": _preset(4096, 32000, [
        _gla(16, 128, 256, ff=14336) for _ in range(4)]),
    # the mixers of both without feed-forward
    "risepel-8b-latent-mixer-4l": _preset(4096, 32000, [
        _latent(32, 128, 64, 128, 512, 1536, 0) for _ in range(4)]),
    "risepel-8b-gla-mixer-4l": _preset(4096, 32000, [
        _gla(16, 128, 256) for _ in range(4)]),
    # both kinds, a shared latent
    "risepel-8b-4l": _preset(4096, 32000, [
        _latent(32, 128, 64, 128, 512, 1536, 1024, ff=14336),
        _gla(16, 128, 256, ff=14336), _gla(16, 128, 256, ff=14336),
        _latent(32, 128, 64, 128, 512, 1536, 1024, ff=14336, kv_from=0)]),
    "risepel-tiny": _preset(192, 320, [
        _gla(3, 32, 48, ff=256), _latent(6, 32, 16, 48, 80, 96, 24),
        _latent(6, 32, 16, 48, 80, 96, 40),
        _latent(4, 32, 16, 48, 80, 96, 33, ff=256, kv_from=2)]),
}


@dataclass
class RisepelConfig(ModelConfig):
    model_type: str = "risepel"

    @classmethod
    def from_dict(cls, d: dict) -> "RisepelConfig":
        d = copy.deepcopy(d)
        layers = d["layers"]
        first = layers[0]["mixer"]
        mapped = {
            "hidden_size": int(d["width"]),
            "num_hidden_layers": len(layers),
            "vocab_size": int(d["vocab"]),
            "max_position_embeddings": int(d.get("max_positions", MAX_POSITIONS)),
            "rms_norm_eps": float(d["norm"]["eps"]),
            "num_attention_heads": int(first["heads"]),
            "num_key_value_heads": int(first["heads"]),
            "head_dim": int(first["dim"]),
        }
        cfg = super().from_dict({**d, **mapped})
        cfg._check()
        return cfg

    def _check(self) -> None:
        for i, layer in enumerate(self.layers):
            mx, mlp = layer["mixer"], layer.get("mlp")
            if layer["type"] == "gla":
                mx.setdefault("decay_rank", DECAY_RANK)
                if mx["tau"] <= 0:
                    raise ValueError(f"layer {i}: tau must be positive")
            elif layer["type"] == "latent_attention":
                dims = mx["rot"]["dims"]
                if dims % 2 or not 0 < dims <= mx["rot_dim"]:
                    raise ValueError(f"layer {i}: cannot rotate {dims} of "
                                     f"{mx['rot_dim']} dimensions")
                self._check_source(i, mx)
            else:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")

    def _check_source(self, i: int, mx: dict) -> None:
        j = mx.get("kv_from")
        if j is None:
            return
        src = self.layers[j] if 0 <= j < i else None
        if (src is None or src["type"] != "latent_attention"
                or src["mixer"].get("kv_from") is not None):
            raise ValueError(f"layer {i}: kv_from must name an earlier layer "
                             f"with latents of its own")
        if any(src["mixer"][k] != mx[k] for k in ("kv_rank", "rot_dim", "rot")):
            raise ValueError(f"layer {i}: latent sizes or rotation differ from "
                             f"those of layer {j}")

    def adopt_shapes(self, shape_of: Callable[[str], tuple]) -> None:
        for i, layer in enumerate(self.layers):
            if layer["type"] == "gla":
                layer["mixer"]["decay_rank"] = int(shape_of(f"l{i}.mix.a1")[0])

    @property
    def layers(self) -> list:
        return self.extras["layers"]

    @property
    def alpha(self) -> float:
        """Factor of the residual in every sum."""
        return float(self.extras["postln_alpha"])

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

    def kv_source(self, layer: int) -> Optional[int]:
        """Layer whose latents `layer` reads, None = its own (or none)."""
        return self.layers[layer]["mixer"].get("kv_from")

    def latent_spec(self, layer: int) -> LatentSpec:
        mx = self.layers[layer]["mixer"]
        return LatentSpec(
            heads=int(mx["heads"]), dim=int(mx["dim"]), rot=int(mx["rot_dim"]),
            rot_dims=int(mx["rot"]["dims"]), vdim=int(mx["vdim"]),
            q_rank=int(mx["q_rank"]), rank=int(mx["kv_rank"]),
            scale=float(mx["scale"]),
            window=int((mx.get("mask") or {}).get("size") or 0),
            eps=self.rms_norm_eps)

    def kv_layout(self, start: int, end: int) -> dict:
        """PagedKVCache geometry of layers [start, end): one key plane of
        [latent | rotated part] for attention, a state for recurrence."""
        heads, sizes, layout, states = [], [], [], []
        for i in range(start, end):
            mx = self.layers[i]["mixer"]
            gla = self.layers[i]["type"] == "gla"
            heads.append(0 if gla else 1)
            sizes.append(0 if gla else self.latent_spec(i).ck)
            layout.append("none" if gla else "k")
            states.append((mx["heads"], mx["dim"], mx["vdim"]) if gla else None)
        return dict(num_kv_heads=heads, head_dim=sizes, layout=layout,
                    shares=kv_shares(self.kv_source, start, end),
                    state_shapes=states)
