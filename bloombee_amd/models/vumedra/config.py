"""Vumedra family config.

Native config.json keys: `width`, `vocab`, `norm` (eps), `embedding` (bigram:
buckets and the two multipliers of its hash) and `layers`, one entry per layer
with its mixer's type and sizes and its feed-forward (dense, moe or none). They
map onto the common ModelConfig fields; what differs per layer stays in `layers`.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional

import torch

from bloombee_amd.models.base import ModelConfig
from bloombee_amd.ops.ragged import pad_head
from bloombee_amd.ops.recurrent import MlstmSpec, RglruSpec

MAX_POSITIONS = 1 << 20   # positions are sinusoidal: the design has no limit


def _attention(heads, kv_heads, dim, vdim, mlp, scale=None, coef=0.5,
               every=1024) -> dict:
    return {"type": "attention", "mlp": mlp, "mixer": {
        "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
        "scale": scale or dim ** -0.5,
        "q_temp": {"coef": coef, "every": every}}}


def _mlstm(heads, dim, vdim, mlp, cap=15.0) -> dict:
    return {"type": "mlstm", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _rglru(width, blocks, mlp, conv=4) -> dict:
    return {"type": "rglru", "mlp": mlp,
            "mixer": {"width": width, "blocks": blocks, "conv": conv}}


def _dense(ff) -> dict:
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, shared) -> dict:
    return {"kind": "moe", "router": {"experts": experts, "top": top},
            "expert": {"ff": ff}, "shared": {"ff": shared}}


def _preset(width, vocab, layers, buckets, eps=1e-6) -> dict:
    return dict(width=width, vocab=vocab, norm={"eps": eps}, layers=layers,
                embedding={"bigram": {"buckets": buckets, "mul_prev": 8191,
                                      "mul_cur": 31}})


VUMEDRA_PRESETS = {
    # layers of llama-3-8b's width, heads and feed-forward
    "vumedra-8b-attn-4l": _preset(4096, 32000, [
        _attention(32, 8, 128, 128, _dense(14336)) for _ in range(4)], 65521),
    # the same without feed-forward
    "vumedra-8b-attn-mixer-4l": _preset(4096, 32000, [
        _attention(32, 8, 128, 128, None) for _ in range(4)], 65521),
    # 16 memory heads of 128 keys and 256 values
    "vumedra-8b-mlstm-4l": _preset(4096, 32000, [
        _mlstm(16, 128, 256, _dense(14336)) for _ in range(4)], 65521),
    # a recurrent unit as wide as the model
    "vumedra-8b-rglru-4l": _preset(4096, 32000, [
        _rglru(4096, 16, _dense(14336)) for _ in range(4)], 65521),
    # all three; routed feed-forwards
    "vumedra-8x7b-4l": _preset(4096, 32000, [
        _mlstm(16, 128, 256, _moe(8, 2, 14336, 4096)),
        _mlstm(16, 128, 256, _moe(8, 2, 14336, 4096)),
        _rglru(4096, 16, _moe(8, 2, 14336, 4096)),
        _attention(32, 8, 128, 128, _moe(8, 2, 14336, 4096))], 65521),
    "vumedra-tiny": _preset(192, 320, [
        _mlstm(3, 32, 40, _dense(256)), _rglru(192, 4, _moe(6, 2, 64, 128)),
        _attention(6, 2, 48, 32, _moe(6, 2, 64, 128), every=16),
        _mlstm(3, 32, 40, None)], 509),
}


@dataclass
class VumedraConfig(ModelConfig):
    model_type: str = "vumedra"

    @classmethod
    def from_dict(cls, d: dict) -> "VumedraConfig":
        d = copy.deepcopy(d)
        layers = d["layers"]
        # the common head fields describe the first layer that has heads
        first = next((l["mixer"] for l in layers if "heads" in l["mixer"]),
                     {"heads": 1, "dim": int(d["width"])})
        mapped = {
            "hidden_size": int(d["width"]),
            "num_hidden_layers": len(layers),
            "vocab_size": int(d["vocab"]),
            "max_position_embeddings": int(d.get("max_positions", MAX_POSITIONS)),
            "rms_norm_eps": float(d["norm"]["eps"]),
            "num_attention_heads": int(first["heads"]),
            "num_key_value_heads": int(first.get("kv_heads", first["heads"])),
            "head_dim": int(first["dim"]),
        }
        cfg = super().from_dict({**d, **mapped})
        cfg._check()
        return cfg

    def _check(self) -> None:
        pair = self.bigram
        if pair["buckets"] < 1 or min(pair["mul_prev"], pair["mul_cur"]) < 0:
            raise ValueError("token pairs need buckets and factors >= 0")
        for i, layer in enumerate(self.layers):
            mx, mlp = layer["mixer"], layer.get("mlp")
            if layer["type"] == "attention":
                if mx["heads"] % mx["kv_heads"]:
                    raise ValueError(f"layer {i}: {mx['heads']} heads do not share "
                                     f"{mx['kv_heads']} key heads evenly")
                if mx.get("q_temp") and mx["q_temp"]["every"] <= 0:
                    raise ValueError(f"layer {i}: q_temp.every must be positive")
            elif layer["type"] == "mlstm":
                if mx["gate_cap"] <= 0:
                    raise ValueError(f"layer {i}: gate_cap must be positive")
            elif layer["type"] == "rglru":
                if mx["width"] % mx["blocks"] or mx["conv"] < 1:
                    raise ValueError(f"layer {i}: {mx['width']} channels in "
                                     f"{mx['blocks']} blocks, {mx['conv']} taps")
            else:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if mlp is None or mlp["kind"] == "dense":
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
    def bigram(self) -> dict:
        return self.extras["embedding"]["bigram"]

    @property
    def sinusoidal_positions(self) -> bool:
        return True

    @property
    def scalar_norm(self) -> bool:
        """Layer and final norms have one weight for all coordinates."""
        return True

    @property
    def hidden_dtype(self) -> torch.dtype:
        """The residual is 32-bit whatever the compute type."""
        return torch.float32

    def recurrent_spec(self, layer: int):
        """Sizes of a recurrent mixer, None for attention."""
        mx, kind = self.layers[layer]["mixer"], self.layers[layer]["type"]
        if kind == "mlstm":
            return MlstmSpec(heads=int(mx["heads"]), dim=int(mx["dim"]),
                             vdim=int(mx["vdim"]), cap=float(mx["gate_cap"]),
                             eps=self.rms_norm_eps)
        if kind == "rglru":
            return RglruSpec(width=int(mx["width"]), blocks=int(mx["blocks"]),
                             taps=int(mx["conv"]))
        return None

    def kv_layout(self, start: int, end: int) -> dict:
        """PagedKVCache geometry of layers [start, end): pages for attention,
        states for recurrence."""
        heads, dims, vdims, layout, states = [], [], [], [], []
        for i in range(start, end):
            spec, mx = self.recurrent_spec(i), self.layers[i]["mixer"]
            rec = spec is not None
            heads.append(0 if rec else mx["kv_heads"])
            dims.append(0 if rec else pad_head(mx["dim"]))
            vdims.append(0 if rec else pad_head(mx["vdim"]))
            layout.append("none" if rec else "kv")
            states.append(spec.state_shapes() if rec else None)
        return dict(num_kv_heads=heads, head_dim=dims, v_head_dim=vdims,
                    layout=layout, state_shapes=states)
