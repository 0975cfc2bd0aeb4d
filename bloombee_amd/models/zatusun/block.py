"""Zatusun decoder block (one run of a layer) on the ragged-batch ops.

Pre-norm: x <- x + mixer(norm1(x)), then x <- x + experts(norm2(x)); what a
sublayer adds is left Pending and the next norm's launch folds it. The run that
begins a pass of the loop first puts W_in [x | x0] + step in the residual's place,
with x0 the embedding output.

One GEMM reads the normed rows of a mixer:
    latent_attention  in_w [query latent | latent, rotated part | gate]
    attention         in_w [q | k | v]             two maps per head
    hgrn2             in_w [q | v | forget gate (computed in f32)]
and a small one, in f32, those of the router.

Rotary pairs lie side by side in the checkpoint; the kernels turn one half of a
vector with the other, so the rows of the projections are reordered when loaded.
"""
from __future__ import annotations

import math
from typing import Callable, Dict, Optional, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.kv.batch import TokenBatch, lockstep_batch
from bloombee_amd.models.zatusun.config import ZatusunConfig
from bloombee_amd.ops import mixers, ragged
from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.mixers import LatentWeights, half_order
from bloombee_amd.ops.ragged import FfSpec, Pending, pad_k, round_up


class ZatusunBlock(torch.nn.Module):
    token_batched = True   # BlockStack hands whole steps to forward_tokens
    hip_modules = ("_hip_ragged", "_hip_mixers", "_hip_differential",
                   "_hip_hgrn")
    model_tensors = ("loop.in", "loop.step")   # checkpoint names without layer

    def __init__(self, config: ZatusunConfig, layer_index: int = 0, rope=None):
        super().__init__()
        self.config = config
        self.layer_index = layer_index     # BlockStack rebases it to its pool
        self.global_index = layer_index
        run = config.runs[layer_index]
        self.checkpoint_index, self.enters = run.layer, run.enters
        layer = config.layers[run.layer]
        self.kind, self.mlp = layer["type"], layer.get("mlp")
        W = config.hidden_size
        self.K = pad_k(W)                  # stored inner size of h
        dt, f32 = config.dtype, torch.float32

        def p(*shape, dtype=f32):
            return torch.nn.Parameter(torch.zeros(*shape, dtype=dtype),
                                      requires_grad=False)

        # tensor name -> (first row, rows) of in_w
        self._in_rows: Dict[str, Tuple[int, int]] = {}
        at = 0

        def section(name: str, rows: int, align: int = 8) -> int:
            nonlocal at
            off = round_up(at, align)
            self._in_rows[name] = (off, rows)
            at = off + rows
            return off

        # plain f32 parameters: tensor name -> attribute, shape
        self._vectors: Dict[str, Tuple[str, Tuple[int, ...]]] = {}

        def vector(name: str, attr: str, *shape: int) -> None:
            self._vectors[name] = (attr, shape)
            setattr(self, attr, p(*shape))

        s = config.mixer_spec(run.layer)
        if self.kind == "latent_attention":
            H, D, V = s.heads, s.dim, s.vdim
            s.q_off = section("mix.dq", s.q_rank)
            s.c_off = section("mix.dkv", s.rank + s.rot)
            s.g_off = section("mix.g", H * V)
            s.q_cols = pad_k(s.q_rank)
            vector("mix.dq.norm", "q_norm_w", s.q_rank)
            vector("mix.dkv.norm", "c_norm_w", s.rank)
            self.uq_w = p(round_up(H * (D + s.rot), 64), s.q_cols, dtype=dt)
            self.uk_w = p(H, s.rp, round_up(D, 32), dtype=dt)   # transposed
            self.uv_w = p(H, round_up(V, 64), s.rp, dtype=dt)
            self.ukv_w = p(round_up(H * (D + V), 64), s.ck, dtype=dt)
        elif self.kind == "attention":
            r = s.rope
            H, D, V = r.heads, r.dim, r.vdim
            r.q_off = section("mix.q", H * r.maps * D)
            r.k_off = section("mix.k", r.kv_heads * r.maps * D)
            r.v_off = section("mix.v", r.kv_heads * V)
            self.diff = float(layer["mixer"]["diff"])
        else:
            H, D, V = s.heads, s.dim, s.vdim
            s.q_off = section("mix.q", H * D)
            s.v_off = section("mix.v", H * V)
            # the gate rows start a 64-row block: the rows before them are a
            # GEMM of their own where they are computed apart
            s.router_off = section("mix.f", H * D, 64)
            vector("mix.f.b", "f_b", H * D)
            vector("mix.lower", "lower", H * D)
            vector("mix.norm", "o_norm_w", V)
        if self.kind != "hgrn2":
            self.turns = torch.nn.Parameter(config.rotation(run.layer)[0],
                                            requires_grad=False)
        self.inner = H * V
        s.out_cols = pad_k(self.inner)
        self.heads, self.dim, self.vdim, self.spec = H, D, V, s
        self.in_w = p(round_up(at, 64), self.K, dtype=dt)
        self.out_w = p(round_up(W, 64), s.out_cols, dtype=dt)
        self.norms = ["norm1"] if self.mlp is None else ["norm1", "norm2"]
        for n in self.norms:
            setattr(self, n + "_w", p(W))
        if self.mlp is not None:
            self.E, self.Fe = (int(self.mlp["router"]["experts"]),
                               int(self.mlp["expert"]["ff"]))
            self.glu = config.glu_spec(run.layer)
            self.ff_spec = FfSpec(router_off=0, router_n=self.E, renorm=True,
                                  top=int(self.mlp["router"]["top"]))
            self.router_w = p(round_up(self.E, 64), self.K, dtype=dt)
            self.expert_up_w = p(self.E, 2, round_up(self.Fe, 64), self.K,
                                 dtype=dt)
            self.expert_down_w = p(self.E, round_up(W, 64),
                                   round_up(self.Fe, 64), dtype=dt)
        if self.enters is not None:
            self.loop_w = p(round_up(W, 64), pad_k(2 * W), dtype=dt)
            self.steps = p(int(config.loop["times"]), W)

    # -- weights ----------------------------------------------------------
    def share_weights(self, other: "ZatusunBlock") -> None:
        """Use the weights of another run of the same layer."""
        for name, w in other.named_parameters():
            setattr(self, name, w)
        self.spec = other.spec

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint tensors of this run, without the layer prefix."""
        s, W = self.spec, self.config.hidden_size
        H, D, V = self.heads, self.dim, self.vdim
        out = {n: (rows, W) for n, (_, rows) in self._in_rows.items()}
        out.update({n: shape for n, (_, shape) in self._vectors.items()})
        out.update({n: (W,) for n in self.norms})
        out["mix.o"] = (W, self.inner)
        if self.kind == "latent_attention":
            out["mix.uq"] = (H * (D + s.rot), s.q_rank)
            out["mix.uk"] = (H * D, s.rank)
            out["mix.uv"] = (H * V, s.rank)
        elif self.kind == "attention":
            for n in ("lq1", "lk1", "lq2", "lk2"):
                out[f"mix.{n}"] = (D,)
        if self.mlp is not None:
            out["mlp.router"] = (self.E, W)
            for e in range(self.E):
                for n in ("gate", "up"):
                    out[f"mlp.e{e}.{n}"] = (self.Fe, W)
                out[f"mlp.e{e}.down"] = (W, self.Fe)
        if self.enters is not None:
            out["loop.in"] = (W, 2 * W)
            out["loop.step"] = tuple(self.steps.shape)
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
                raise ValueError(f"layer {self.checkpoint_index} {name}: shape "
                                 f"{tuple(t.shape)}, expected {shapes[name]}")
            return t

        def halves(t: torch.Tensor, dims: int, size: int,
                   skip: int = 0) -> torch.Tensor:
            """Rows of vectors of `size` elements, after `skip` that pass, with
            their rotary pairs apart."""
            v = t.view(-1, skip + size, t.shape[1])
            order = half_order(dims, size).to(t.device)
            return torch.cat([v[:, :skip], v[:, skip:][:, order]], 1).view_as(t)

        for name, (off, rows) in self._in_rows.items():
            t = take(name)
            if name == "mix.dkv":
                t = halves(t, s.rot_dims, s.rot, s.rank)
            elif self.kind == "attention" and name != "mix.v":
                t = halves(t, s.rope.rot_dims, D)
            self.in_w[off:off + rows, :W].copy_(t)
        for name, (attr, _) in self._vectors.items():
            getattr(self, attr).copy_(take(name))
        for name in self.norms:
            # stored as their distance from one
            getattr(self, name + "_w").copy_(take(name)).add_(1.0)
        self.out_w[:W, :self.inner].copy_(take("mix.o"))
        if self.kind == "latent_attention":
            self.uq_w[:H * (D + s.rot), :s.q_rank].copy_(
                halves(take("mix.uq"), s.rot_dims, s.rot, D))
            uk, uv = take("mix.uk"), take("mix.uv")
            self.uk_w[:, :s.rank, :D].copy_(
                uk.view(H, D, s.rank).transpose(1, 2))
            self.uv_w[:, :V, :s.rank].copy_(uv.view(H, V, s.rank))
            self.ukv_w[:H * D, :s.rank].copy_(uk)
            self.ukv_w[H * D:H * (D + V), :s.rank].copy_(uv)
        elif self.kind == "attention":
            q1, k1, q2, k2 = (take(f"mix.{n}").double()
                              for n in ("lq1", "lk1", "lq2", "lk2"))
            s.lam = float(torch.exp((q1 * k1).sum())
                          - torch.exp((q2 * k2).sum())) + self.diff
        if self.mlp is not None:
            self.router_w[:self.E, :W].copy_(take("mlp.router"))
            for e in range(self.E):
                for i, n in enumerate(("gate", "up")):
                    self.expert_up_w[e, i, :self.Fe, :W].copy_(
                        take(f"mlp.e{e}.{n}"))
                self.expert_down_w[e, :W, :self.Fe].copy_(
                    take(f"mlp.e{e}.down"))
        if self.enters is not None:
            self.loop_w[:W, :2 * W].copy_(take("loop.in"))
            self.steps.copy_(take("loop.step"))
        return len(shapes)

    @torch.no_grad()
    def init_random(self, seed: Optional[int] = None):
        s = seed if seed is not None else 1234 + self.global_index
        dev = self.in_w.device
        gen = torch.Generator(device=dev).manual_seed(s)
        std = 0.02 / math.sqrt(2 * self.config.num_hidden_layers)
        shapes = self.tensor_shapes()
        # forgetting slowly
        const = {"mix.f.b": 3.0, "mix.lower": 0.5, "mix.norm": 1.0,
                 "mix.dq.norm": 1.0, "mix.dkv.norm": 1.0}

        def draw(name: str) -> torch.Tensor:
            shape = shapes[name]
            if name.startswith("norm") or name in const:
                return torch.full(shape, const.get(name, 0.0), device=dev)
            return torch.randn(shape, generator=gen, dtype=torch.float32,
                               device=dev).mul_(std)

        self.load_tensors(draw)
        return self

    # -- inference --------------------------------------------------------
    def _latent(self, h: torch.Tensor, batch: TokenBatch) -> torch.Tensor:
        s, dt = self.spec, self.in_w.dtype
        pages = batch.k_pages(self.layer_index)
        cq, gate = mixers.latent_post(
            ragged.linear_parts(h, self.in_w), s, self.q_norm_w, self.c_norm_w,
            self.turns, batch, pages, dt)
        w = LatentWeights(self.uk_w, self.uv_w, self.ukv_w, None)
        return mixers.latent_attention(ragged.linear_parts(cq, self.uq_w), s, w,
                                       self.turns, batch, gate, pages, dt)

    def _mix(self, h: torch.Tensor, batch: TokenBatch) -> torch.Tensor:
        i, dt = self.layer_index, self.in_w.dtype
        if self.kind == "latent_attention":
            return self._latent(h, batch)
        if self.kind == "attention":
            return mixers.differential_attention(
                ragged.linear_parts(h, self.in_w), self.spec, self.turns, batch,
                batch.k_pages(i), batch.v_pages(i), dt)
        parts, fparts, f0 = ragged.input_projection(h, self.in_w, self.spec)
        return mixers.hgrn_mix(parts, fparts, f0, self.spec, self.f_b, self.lower,
                               self.o_norm_w, batch.cache.state(i), batch, dt)

    @torch.no_grad()
    def forward_tokens(self, x: torch.Tensor, pending: Optional[Pending],
                       batch: TokenBatch) -> Pending:
        """x (N, W) f32: the residual before `pending`, updated in place."""
        eps, dt = self.config.rms_norm_eps, self.in_w.dtype
        if self.enters is not None:
            rows = ragged.join_rows(x, pending, batch.embedded,
                                    self.loop_w.shape[1], dt)
            pending = Pending(ragged.linear_sums(rows, self.loop_w),
                              bias=self.steps[self.enters], keep=0.0)
        h = ragged.residual_norm(x, pending, self.norm1_w, 1, eps, self.K, dt)
        left = Pending(ragged.linear_parts(self._mix(h, batch), self.out_w))
        if self.mlp is None:
            return left
        h = ragged.residual_norm(x, left, self.norm2_w, 1, eps, self.K, dt)
        rt = ragged.route(h, self.router_w, self.ff_spec)
        return Pending(None, ragged.moe_experts(
            h, self.expert_up_w, self.expert_down_w, rt, act=self.glu), rt)

    def forward_inference(self, hidden: torch.Tensor, kv, start_pos,
                          position_ids=None) -> torch.Tensor:
        """Lockstep step of one block (offloaded stacks call blocks singly)."""
        if position_ids is not None:
            raise NotImplementedError(
                "recurrent layers follow the sequence: no position_ids")
        B, T, C = hidden.shape
        rows = hidden.reshape(B * T, C).to(torch.float32, copy=True)
        batch = lockstep_batch(kv, start_pos, B, T)
        x = batch.split_hidden(rows, self.config.hidden_size)
        self.forward_tokens(x, None, batch).settle(x)
        return rows.view(B, T, C)

    # -- training ---------------------------------------------------------
    def _train_mixer(self, h: torch.Tensor, start_pos: int) -> torch.Tensor:
        s, W, dt = self.spec, self.config.hidden_size, self.in_w.dtype
        H, D, V = self.heads, self.dim, self.vdim
        B, T, _ = h.shape

        def rows(name):
            off, n = self._in_rows[name]
            return F.linear(h, self.in_w[off:off + n, :W])

        def rms(t, w):
            return ref.grouped_rms_norm(t, w, 1, s.eps)

        if self.kind == "hgrn2":
            f, k = ref.forget_gates(rows("mix.f"), self.f_b, self.lower)
            q, k, f, v = (t.float().reshape(B, T, H, -1) for t in (
                F.silu(rows("mix.q").float()), k, f, rows("mix.v")))
            zero = torch.zeros(H, D, V, device=h.device)
            o = torch.stack([ref.gla_scan(q[b], k[b], v[b], f[b], zero)[0]
                             for b in range(B)])
            o = rms(o, self.o_norm_w).reshape(B, T, H * V).to(dt)
            return F.linear(o, self.out_w[:W, :self.inner])

        pos = torch.arange(start_pos, start_pos + T, device=h.device)

        def rotate(t, amp):      # (B, T, ..., rotated first)
            return ref.rotate_half(t.transpose(0, 1), pos, self.turns,
                                   amp).transpose(0, 1)

        def attend(q, k, v, chunk=0):    # (B, T, H, ...)
            sc = torch.matmul(q.transpose(1, 2).contiguous(),
                              k.permute(0, 2, 3, 1).contiguous()) * s.scale
            dist = pos.view(T, 1) - pos.view(1, T)
            seen = dist >= 0
            if chunk:
                seen &= dist <= pos.view(T, 1) % chunk
            p = torch.softmax(sc.masked_fill(~seen, float("-inf")), -1)
            return torch.matmul(p, v.transpose(1, 2).contiguous()).transpose(1, 2)

        if self.kind == "attention":
            r = s.rope
            G = r.kv_heads
            q = rotate(rows("mix.q").float().view(B, T, H, 2, D), r.amp)
            k = rotate(rows("mix.k").float().view(B, T, G, 2, D), r.amp)
            k = k.to(dt).float().repeat_interleave(H // G, 2)
            v = rows("mix.v").float().view(B, T, G, V).repeat_interleave(
                H // G, 2)
            a = [attend(q[..., m, :], k[..., m, :], v, s.chunk)
                 for m in range(2)]
            o = rms(a[0] - s.lam * a[1], torch.ones(V, device=h.device)) * s.factor
            return F.linear(o.reshape(B, T, H * V).to(dt),
                            self.out_w[:W, :self.inner])

        y = rows("mix.dkv").float()
        lat = rms(y[..., :s.rank], self.c_norm_w).to(dt)
        kr = rotate(y[..., s.rank:], s.amp).to(dt)
        cq = rms(rows("mix.dq"), self.q_norm_w).to(dt)
        q = F.linear(cq, self.uq_w[:H * (D + s.rot), :s.q_rank])
        q = q.float().view(B, T, H, D + s.rot)
        q = torch.cat([q[..., :D], rotate(q[..., D:], s.amp)], -1)
        kv = F.linear(lat, self.ukv_w[:H * (D + V), :s.rank]).float()
        k = torch.cat([kv[..., :H * D].view(B, T, H, D),
                       kr.float().unsqueeze(2).expand(B, T, H, s.rot)], -1)
        o = attend(q, k, kv[..., H * D:].reshape(B, T, H, V))
        o = o.reshape(B, T, H * V) * torch.sigmoid(rows("mix.g").float())
        return F.linear(o.to(dt), self.out_w[:W, :self.inner])

    def _train_ff(self, h: torch.Tensor) -> torch.Tensor:
        f, W, dt = self.ff_spec, self.config.hidden_size, self.in_w.dtype
        flat = h.reshape(-1, W)
        logits = flat.float() @ self.router_w[:self.E, :W].float().t()
        ids, wts, _ = ref.route_topk(logits, None, self.E, f.top, f.scale,
                                     f.sigmoid, f.renorm)
        out = torch.zeros_like(flat, dtype=torch.float32)
        for e in range(self.E):
            t, c = (ids == e).nonzero(as_tuple=True)
            if t.numel() == 0:
                continue
            g, u = (F.linear(flat[t], self.expert_up_w[e, i, :self.Fe, :W]).float()
                    for i in range(2))
            a = ref.clamped_glu(g, u, None, None, self.glu.limit, self.glu.slope)
            y = F.linear(a.to(dt), self.expert_down_w[e, :W, :self.Fe]).float()
            out = out.index_add(0, t, y * wts[t, c, None])
        return out.view(*h.shape[:-1], W)

    def forward_train(self, hidden: torch.Tensor, start_pos: int = 0,
                      ) -> torch.Tensor:
        """Differentiable full-sequence path, no KV cache and no state."""
        W, dt, eps = (self.config.hidden_size, self.in_w.dtype,
                      self.config.rms_norm_eps)

        def rms(t, w):
            return ref.grouped_rms_norm(t, w, 1, eps).to(dt)

        hidden = hidden.float()
        x = hidden[..., :W]
        if self.enters is not None:
            x = (F.linear(hidden.to(dt), self.loop_w[:W, :2 * W]).float()
                 + self.steps[self.enters])
        x = x + self._train_mixer(rms(x, self.norm1_w), start_pos).float()
        if self.mlp is not None:
            x = x + self._train_ff(rms(x, self.norm2_w))
        return torch.cat([x, hidden[..., W:]], -1)

    def forward(self, *args, **kw):
        return self.forward_inference(*args, **kw)
