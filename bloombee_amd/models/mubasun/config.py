"""Mubasun family config.

Native config.json keys: `width`, `vocab`, `max_positions`, `norm` (eps,
groups) and `layers`, one entry per layer with its own mixer (head counts, key
and value sizes, score scale, window, whose keys/values it reads) and its own
feed-forward (dense, routed or none). They map onto the common ModelConfig
fields; what differs per layer stays in `layers`.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional

import torch

from bloombee_amd.models.base import ModelConfig, kv_shares
from bloombee_amd.ops.ragged import pad_head


def _layer(heads, kv_heads, dim, window, vdim=None, scale=None, dense=None,
           experts=0, top=0, ff=0, identity=0, shared=0, router_scale=1.0,
           kv_from=None) -> dict:
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim,
             "vdim": vdim or dim, "scale": scale or dim ** -0.5,
             "mask": {"size": window}}
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    mlp = None
    if dense:
        mlp = {"kind": "dense", "ff": dense}
    elif experts:
        mlp = {"kind": "moe", "expert": {"ff": ff},
               "router": {"experts": experts, "identity": identity,
                          "scale": router_scale, "top": top}}
        if shared:
            mlp["shared"] = {"ff": shared}
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


MUBASUN_PRESETS = {
    # layer sizes of llama-3-8b, dense feed-forwards, 1k window
    "mubasun-8b-4l": dict(
        width=4096, vocab=32000, max_positions=32768,
        norm={"eps": 1e-5, "groups": 8},
        layers=[_layer(32, 8, 128, 1024, dense=14336) for _ in range(4)]),
    # layer sizes of mixtral-8x7b: 8 experts, 2 of them per token
    "mubasun-8x7b-4l": dict(
        width=4096, vocab=32000, max_positions=32768,
        norm={"eps": 1e-5, "groups": 8},
        layers=[_layer(32, 8, 128, 1024, experts=8, top=2, ff=14336)
                for _ in range(4)]),
    # many small experts, a shared one, identity experts, a shared KV tail
    "mubasun-64e-4l": dict(
        width=4096, vocab=32000, max_positions=32768,
        norm={"eps": 1e-5, "groups": 8},
        layers=[_layer(32, 8, 128, 1024, experts=64, top=6, ff=1408,
                       identity=4, shared=2816, router_scale=2.0,
                       kv_from=1 if i > 1 else None) for i in range(4)]),
    "mubasun-tiny": dict(
        width=192, vocab=320, max_positions=512,
        norm={"eps": 1e-5, "groups": 3},
        layers=[_layer(6, 2, 32, 24, vdim=48, dense=320),
                _layer(6, 2, 32, 33, vdim=48, experts=6, top=3, ff=80,
                       identity=2, shared=112, router_scale=1.5),
                _layer(6, 2, 32, 24, vdim=48),
                _layer(6, 2, 32, 24, vdim=48, experts=6, top=3, ff=80,
                       identity=2, kv_from=2)]),
}


@dataclass
class MubasunConfig(ModelConfig):
    model_type: str = "mubasun"

    @classmethod
    def from_dict(cls, d: dict) -> "MubasunConfig":
        d = copy.deepcopy(d)
        layers = d["layers"]
        first = layers[0]["mixer"]
        mapped = {
            "hidden_size": int(d["width"]),
            "num_hidden_layers": len(layers),
            "vocab_size": int(d["vocab"]),
            "max_position_embeddings": int(d["max_positions"]),
            "rms_norm_eps": float(d["norm"]["eps"]),
            "num_attention_heads": int(first["heads"]),
            "num_key_value_heads": int(first["kv_heads"]),
            "head_dim": int(first["dim"]),
        }
        cfg = super().from_dict({**d, **mapped})
        cfg._check()
        return cfg

    def _check(self) -> None:
        if self.hidden_size % self.norm_groups:
            raise ValueError("norm groups must divide the width")
        for i, layer in enumerate(self.layers):
            if layer["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            mx, mlp = layer["mixer"], layer.get("mlp")
            if mx["heads"] % mx["kv_heads"]:
                raise ValueError(f"layer {i}: kv_heads must divide heads")
            j = mx.get("kv_from")
            if j is not None:
                src = self.layers[j]["mixer"] if 0 <= j < i else None
                if src is None or src.get("kv_from") is not None:
                    raise ValueError(f"layer {i}: kv_from must name an earlier "
                                     f"layer with keys of its own")
                if any(src[k] != mx[k] for k in ("kv_heads", "dim", "vdim")):
                    raise ValueError(f"layer {i}: key/value sizes differ from "
                                     f"those of layer {j}")
            if mlp is None:
                continue
            if mlp["kind"] not in ("dense", "moe"):
                raise ValueError(f"layer {i}: unknown feed-forward "
                                 f"{mlp['kind']!r}")
            if mlp["kind"] == "moe":
                rt = mlp["router"]
                if not 1 <= rt["top"] <= rt["experts"] + rt["identity"]:
                    raise ValueError(f"layer {i}: cannot choose {rt['top']} "
                                     f"experts")

    @property
    def layers(self) -> list:
        return self.extras["layers"]

    @property
    def learned_positions(self) -> bool:
        return True

    @property
    def norm_groups(self) -> int:
        return int(self.extras["norm"]["groups"])

    @property
    def hidden_dtype(self) -> torch.dtype:
        """The residual is 32-bit whatever the compute type."""
        return torch.float32

    def kv_source(self, layer: int) -> Optional[int]:
        """Layer whose keys and values `layer` reads, None = its own."""
        return self.layers[layer]["mixer"].get("kv_from")

    def kv_layout(self, start: int, end: int) -> dict:
        """PagedKVCache geometry of layers [start, end)."""
        mixers = [self.layers[i]["mixer"] for i in range(start, end)]
        return dict(
            num_kv_heads=[m["kv_heads"] for m in mixers],
            head_dim=[pad_head(m["dim"]) for m in mixers],
            v_head_dim=[pad_head(m["vdim"]) for m in mixers],
            shares=kv_shares(self.kv_source, start, end))
