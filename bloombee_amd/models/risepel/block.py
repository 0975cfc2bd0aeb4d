"""Risepel decoder block on the ragged-batch ops.

Norms come after the sums: x <- norm1(alpha x + mixer(x)), then
x <- norm2(alpha x + ff(x)). Nothing is normed ahead of a sublayer: a layer hands the
next one its rows in the activation type (Carried) and owes it nothing.

Latent attention, one GEMM for everything that reads x:
    in_w  [query latent | latent, rotated part | gate]
then norms and page slots, the query GEMM, attention with sink and gate
(ops/mixers.py), W_o.

Gated linear attention:
    in_w  [q | k | v | gate | decay rank (computed in f32)]
then the recurrence with its norm and gate, W_o.

Feed-forward: mlp_w [gate | up], clamped product, down_w. Every sum, with the
GEMM's split-K partials and bias, ends in one launch of sum_norm.
"""
from __future__ import annotations

import math
from typing import Callable, Dict, Optional, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.kv.batch import TokenBatch, lockstep_batch
from bloombee_amd.models.risepel.config import RisepelConfig
from bloombee_amd.ops import mixers, ragged
from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.mixers import GlaSpec, LatentWeights
from bloombee_amd.ops.ragged import Carried, pad_k, round_up

GLU_SLOPE = 1.702   # of the feed-forward's sigmoid


class RisepelBlock(torch.nn.Module):
    token_batched = True   # BlockStack hands whole steps to forward_tokens
    hip_modules = ("_hip_ragged", "_hip_mixers")

    def __init__(self, config: RisepelConfig, layer_index: int = 0, rope=None):
        super().__init__()
        self.config = config
        self.layer_index = layer_index     # BlockStack rebases it to its pool
        self.global_index = layer_index
        layer = config.layers[layer_index]
        mx, self.mlp = layer["mixer"], layer.get("mlp")
        self.is_gla = layer["type"] == "gla"
        W = config.hidden_size
        self.kv_source = config.kv_source(layer_index)
        self.K = pad_k(W)                  # stored inner size of x
        # tensor name -> (first row, rows) of in_w
        self._in_rows: Dict[str, Tuple[int, int]] = {}
        at = 0

        def section(name: str, rows: int) -> int:
            nonlocal at
            off = at
            self._in_rows[name] = (off, rows)
            at = round_up(off + rows, 8)
            return off

        dt, f32 = config.dtype, torch.float32

        def p(*shape, dtype=dt):
            return torch.nn.Parameter(torch.zeros(*shape, dtype=dtype),
                                      requires_grad=False)

        H, D, V = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"])
        if self.is_gla:
            s = GlaSpec(heads=H, dim=D, vdim=V, tau=float(mx["tau"]),
                        eps=config.rms_norm_eps)
            s.q_off = section("mix.q", H * D)
            s.k_off = section("mix.k", H * D)
            s.v_off = section("mix.v", H * V)
            s.g_off = section("mix.g", H * V)
            # the decay rows start a 64-row block: the rows before it are a
            # GEMM of their own where they are computed apart
            at = round_up(at, 64)
            s.router_n = int(mx["decay_rank"])
            s.router_off = section("mix.a1", s.router_n)
            self.a2_w = p(s.router_n, H * D, dtype=f32)    # transposed
            self.a2_b = p(H * D, dtype=f32)
            self.o_norm_w = p(V, dtype=f32)
        else:
            s = config.latent_spec(layer_index)
            s.q_off = section("mix.dq", s.q_rank)
            if self.kv_source is None:
                s.c_off = section("mix.dkv", s.rank + s.rot)
                self.c_norm_w = p(s.rank, dtype=f32)
            s.g_off = section("mix.g", H * V)
            s.q_cols = pad_k(s.q_rank)
            self.q_norm_w = p(s.q_rank, dtype=f32)
            self.uq_w = p(round_up(H * (D + s.rot), 64), s.q_cols)
            self.uk_w = p(H, s.rp, round_up(D, 32))        # transposed
            self.uv_w = p(H, round_up(V, 64), s.rp)
            self.ukv_w = p(round_up(H * (D + V), 64), s.ck)
            self.sink = p(H, dtype=f32)
            self.turns = torch.nn.Parameter(
                mixers.rotary_turns(float(mx["rot"]["base"]), s.rot_dims),
                requires_grad=False)
        s.out_cols = pad_k(H * V)
        self.spec = s
        self.heads, self.dim, self.vdim = H, D, V
        self.in_w = p(round_up(at, 64), self.K)
        self.out_w = p(round_up(W, 64), s.out_cols)
        self.norm1_w = p(W, dtype=f32)
        if self.mlp is not None:
            ff = self.ff = int(self.mlp["ff"])
            self.limit = float(self.mlp["limit"])
            self.up_off = round_up(ff, 8)
            self.mlp_w = p(round_up(self.up_off + ff, 64), self.K)
            self.gate_b, self.up_b = p(ff, dtype=f32), p(ff, dtype=f32)
            self.down_w = p(round_up(W, 64), pad_k(ff))
            self.down_b = p(W, dtype=f32)
            self.norm2_w = p(W, dtype=f32)

    # -- weights ----------------------------------------------------------
    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint tensors of this layer, without the layer prefix."""
        s, W = self.spec, self.config.hidden_size
        H, D, V = self.heads, self.dim, self.vdim
        out = {n: (rows, W) for n, (_, rows) in self._in_rows.items()}
        out["norm1"] = (W,)
        out["mix.o"] = (W, H * V)
        if self.is_gla:
            out["mix.norm"] = (V,)
            out["mix.a2"] = (H * D, s.router_n)
            out["mix.a2.b"] = (H * D,)
        else:
            out["mix.dq.norm"] = (s.q_rank,)
            out["mix.uq"] = (H * (D + s.rot), s.q_rank)
            out["mix.uk"] = (H * D, s.rank)
            out["mix.uv"] = (H * V, s.rank)
            out["mix.sink"] = (H,)
            if self.kv_source is None:
                out["mix.dkv.norm"] = (s.rank,)
        if self.mlp is not None:
            out["norm2"] = (W,)
            for n in ("gate", "up"):
                out[f"mlp.{n}"], out[f"mlp.{n}.b"] = (self.ff, W), (self.ff,)
            out["mlp.down"], out["mlp.down.b"] = (W, self.ff), (W,)
        return out

    @torch.no_grad()
    def load_tensors(self, get: Callable[[str], torch.Tensor]) -> int:
        """Fill the fused, padded weights from get(name); returns the number
        of tensors read."""
        s, W = self.spec, self.config.hidden_size
        H, D, V = self.heads, self.dim, self.vdim
        shapes = self.tensor_shapes()

        def take(name: str) -> torch.Tensor:
            t = get(name)
            if tuple(t.shape) != shapes[name]:
                raise ValueError(f"layer {self.global_index} {name}: shape "
                                 f"{tuple(t.shape)}, expected {shapes[name]}")
            return t

        for name, (off, rows) in self._in_rows.items():
            self.in_w[off:off + rows, :W].copy_(take(name))
        self.out_w[:W, :H * V].copy_(take("mix.o"))
        # layer norm weights are stored as their distance from one
        self.norm1_w.copy_(take("norm1")).add_(1.0)
        if self.is_gla:
            self.o_norm_w.copy_(take("mix.norm"))
            self.a2_w.copy_(take("mix.a2").t())
            self.a2_b.copy_(take("mix.a2.b"))
        else:
            self.q_norm_w.copy_(take("mix.dq.norm"))
            if self.kv_source is None:
                self.c_norm_w.copy_(take("mix.dkv.norm"))
            self.uq_w[:H * (D + s.rot), :s.q_rank].copy_(take("mix.uq"))
            uk, uv = take("mix.uk"), take("mix.uv")
            self.uk_w[:, :s.rank, :D].copy_(
                uk.view(H, D, s.rank).transpose(1, 2))
            self.uv_w[:, :V, :s.rank].copy_(uv.view(H, V, s.rank))
            self.ukv_w[:H * D, :s.rank].copy_(uk)
            self.ukv_w[H * D:H * (D + V), :s.rank].copy_(uv)
            self.sink.copy_(take("mix.sink"))
        if self.mlp is not None:
            ff, u = self.ff, self.up_off
            self.mlp_w[:ff, :W].copy_(take("mlp.gate"))
            self.mlp_w[u:u + ff, :W].copy_(take("mlp.up"))
            self.gate_b.copy_(take("mlp.gate.b"))
            self.up_b.copy_(take("mlp.up.b"))
            self.down_w[:W, :ff].copy_(take("mlp.down"))
            self.down_b.copy_(take("mlp.down.b"))
            self.norm2_w.copy_(take("norm2")).add_(1.0)
        return len(shapes)

    @torch.no_grad()
    def init_random(self, seed: Optional[int] = None):
        s = seed if seed is not None else 1234 + self.global_index
        dev = self.in_w.device
        gen = torch.Generator(device=dev).manual_seed(s)
        std = 0.02 / math.sqrt(2 * self.config.num_hidden_layers)
        shapes = self.tensor_shapes()

        def draw(name: str) -> torch.Tensor:
            shape = shapes[name]
            if name.startswith("norm") or name.endswith((".b", ".sink")):
                return torch.zeros(shape, device=dev)
            if name.endswith(".norm"):
                return torch.ones(shape, device=dev)
            return torch.randn(shape, generator=gen, dtype=torch.float32,
                               device=dev).mul_(std)

        self.load_tensors(draw)
        return self

    # -- inference --------------------------------------------------------
    def _kv_layer(self) -> int:
        """Index, in this stack's pool, of the pages this layer reads."""
        if self.kv_source is None:
            return self.layer_index
        at = self.layer_index - (self.global_index - self.kv_source)
        if at < 0:
            raise RuntimeError(
                f"layer {self.global_index} reads the KV of layer "
                f"{self.kv_source}, which is not in this block range")
        return at

    def _latent(self, h: torch.Tensor, batch: TokenBatch) -> torch.Tensor:
        s, dt = self.spec, self.in_w.dtype
        pages = batch.k_pages(self._kv_layer())
        cq, gate = mixers.latent_post(
            ragged.linear_parts(h, self.in_w), s, self.q_norm_w,
            self.c_norm_w if s.has_kv else None, self.turns, batch, pages, dt)
        w = LatentWeights(self.uk_w, self.uv_w, self.ukv_w, self.sink)
        return mixers.latent_attention(ragged.linear_parts(cq, self.uq_w), s, w,
                                       self.turns, batch, gate, pages, dt)

    def _gla(self, h: torch.Tensor, batch: TokenBatch) -> torch.Tensor:
        parts, aparts, a0 = ragged.input_projection(h, self.in_w, self.spec)
        return mixers.gla_mix(parts, aparts, a0, self.spec, self.a2_w, self.a2_b,
                              self.o_norm_w, batch.cache.state(self.layer_index),
                              batch, self.in_w.dtype)

    @torch.no_grad()
    def forward_tokens(self, x: torch.Tensor, left: Optional[Carried],
                       batch: TokenBatch) -> Carried:
        """x (N, W) f32: the residual, updated in place."""
        c, dt = self.config, self.in_w.dtype
        h = left.h if left is not None else ragged.input_rows(x, self.K, dt)

        def add(y, bias, norm_w):
            return ragged.sum_norm(x, y, bias, norm_w, c.alpha, c.rms_norm_eps,
                                   self.K, dt)

        y = self._gla(h, batch) if self.is_gla else self._latent(h, batch)
        h = add(ragged.linear_parts(y, self.out_w), None, self.norm1_w)
        if self.mlp is not None:
            a = ragged.clamped_glu(
                ragged.linear_parts(h, self.mlp_w), 0, self.up_off, self.ff,
                self.gate_b, self.up_b, self.limit, GLU_SLOPE,
                self.down_w.shape[1], dt)
            h = add(ragged.linear_parts(a, self.down_w), self.down_b,
                    self.norm2_w)
        return Carried(h)

    def forward_inference(self, hidden: torch.Tensor, kv, start_pos,
                          position_ids=None) -> torch.Tensor:
        """Lockstep step of one block (offloaded stacks call blocks singly)."""
        if position_ids is not None:
            raise NotImplementedError(
                "recurrent layers follow the sequence: no position_ids")
        B, T, W = hidden.shape
        x = hidden.reshape(B * T, W).to(torch.float32, copy=True)
        self.forward_tokens(x, None, lockstep_batch(kv, start_pos, B, T))
        return x.view(B, T, W)

    # -- training ---------------------------------------------------------
    def _train_mixer(self, x: torch.Tensor, start_pos: int) -> torch.Tensor:
        s, W, dt = self.spec, self.config.hidden_size, self.in_w.dtype
        H, D, V = self.heads, self.dim, self.vdim
        B, T, _ = x.shape
        h = x.to(dt)

        def rows(name):
            off, n = self._in_rows[name]
            return F.linear(h, self.in_w[off:off + n, :W])

        def rms(t, w):
            return ref.grouped_rms_norm(t, w, 1, s.eps)

        if self.is_gla:
            q = rows("mix.q").float().view(B, T, H, D) * D ** -0.5
            k = rows("mix.k").float().view(B, T, H, D)
            v = rows("mix.v").float().view(B, T, H, V)
            alpha = ref.channel_decays(rows("mix.a1").float(), self.a2_w,
                                       self.a2_b, s.tau).view(B, T, H, D)
            zero = torch.zeros(H, D, V, device=x.device)
            o = torch.stack([ref.gla_scan(q[b], k[b], v[b], alpha[b], zero)[0]
                             for b in range(B)])
            o = rms(o, self.o_norm_w).reshape(B, T, H * V)
            o = (o * F.silu(rows("mix.g").float())).to(dt)
            return F.linear(o, self.out_w[:W, :H * V])

        pos = torch.arange(start_pos, start_pos + T, device=x.device)

        def rotate(t):      # (B, T, ..., rot)
            return ref.rotate_half(t.transpose(0, 1), pos,
                                   self.turns).transpose(0, 1)

        if self.kv_source is None:
            y = rows("mix.dkv").float()
            self._train_kv = (rms(y[..., :s.rank], self.c_norm_w).to(dt),
                              rotate(y[..., s.rank:]).to(dt))
            lat, kr = self._train_kv
        else:
            src = getattr(self, "train_source", None)
            if src is None or getattr(src, "_train_kv", None) is None:
                raise RuntimeError(
                    f"layer {self.global_index} needs layer "
                    f"{self.kv_source} in the same training span")
            lat, kr = src._train_kv
        cq = rms(rows("mix.dq"), self.q_norm_w).to(dt)
        q = F.linear(cq, self.uq_w[:H * (D + s.rot), :s.q_rank])
        q = q.float().view(B, T, H, D + s.rot)
        q = torch.cat([q[..., :D], rotate(q[..., D:])], -1)
        kv = F.linear(lat, self.ukv_w[:H * (D + V), :s.rank]).float()
        k = torch.cat([kv[..., :H * D].view(B, T, H, D),
                       kr.float().unsqueeze(2).expand(B, T, H, s.rot)], -1)
        v = kv[..., H * D:].reshape(B, T, H, V).transpose(1, 2)
        sc = torch.matmul(q.transpose(1, 2).contiguous(),
                          k.permute(0, 2, 3, 1).contiguous()) * s.scale
        dist = pos.view(T, 1) - pos.view(1, T)
        seen = dist >= 0
        if s.window:
            seen &= dist < s.window
        sc = sc.masked_fill(~seen, float("-inf"))
        sc = torch.cat([sc, self.sink.view(1, H, 1, 1).expand(B, H, T, 1)], -1)
        o = torch.matmul(torch.softmax(sc, -1)[..., :T], v.contiguous())
        o = o.transpose(1, 2).reshape(B, T, H * V)
        o = (o * torch.sigmoid(rows("mix.g").float())).to(dt)
        return F.linear(o, self.out_w[:W, :H * V])

    def forward_train(self, hidden: torch.Tensor, start_pos: int = 0,
                      ) -> torch.Tensor:
        """Differentiable full-sequence path, no KV cache. A layer that reads
        another's latents takes them from the source block's last call, which
        BlockStack runs just before (`train_source`)."""
        c, W, dt = self.config, self.config.hidden_size, self.in_w.dtype
        x = hidden.float()
        x = ref.grouped_rms_norm(
            c.alpha * x + self._train_mixer(x, start_pos).float(), self.norm1_w,
            1, c.rms_norm_eps)
        if self.mlp is None:
            return x
        h, ff, u = x.to(dt), self.ff, self.up_off
        a = ref.clamped_glu(F.linear(h, self.mlp_w[:ff, :W]).float(),
                            F.linear(h, self.mlp_w[u:u + ff, :W]).float(),
                            self.gate_b, self.up_b, self.limit, GLU_SLOPE)
        y = F.linear(a.to(dt), self.down_w[:W, :ff]).float() + self.down_b
        return ref.grouped_rms_norm(c.alpha * x + y, self.norm2_w, 1,
                                    c.rms_norm_eps)

    def forward(self, *args, **kw):
        return self.forward_inference(*args, **kw)
