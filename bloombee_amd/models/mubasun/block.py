"""Mubasun decoder block on the ragged-batch ops.

Parallel residual: h = norm(x), x += mixer(h) + ff(h). Both sublayers read the
same h, so their first projections are one GEMM and their last ones another:

    in_w  [q | k | v | gate | ff up (| gate) | router, shared gate]
    out_w [W_o | W_down]        inner size = attention columns + activations

Between them one fused row step (q/k norm, K/V pages, activation, routing),
attention with the output gate in its epilogue, and the routed experts. What
the layer adds to the residual is left Pending: the next layer's norm kernel
folds it in. Rows are tokens of a TokenBatch, so prompts, portions of prompts
and single decoded tokens take the same path.
"""
from __future__ import annotations

import math
from typing import Callable, Dict, Optional, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.kv.batch import TokenBatch, lockstep_batch
from bloombee_amd.models.mubasun.config import MubasunConfig
from bloombee_amd.ops import ragged
from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.ragged import Pending, ProjSpec, pad_k, round_up


class MubasunBlock(torch.nn.Module):
    token_batched = True   # BlockStack hands whole steps to forward_tokens
    hip_modules = ("_hip_ragged",)

    def __init__(self, config: MubasunConfig, layer_index: int = 0, rope=None):
        super().__init__()
        self.config = config
        self.layer_index = layer_index     # BlockStack rebases it to its pool
        self.global_index = layer_index
        layer = config.layers[layer_index]
        mx, mlp = layer["mixer"], layer.get("mlp")
        self.mixer, self.mlp = mx, mlp
        W = config.hidden_size
        H, G = int(mx["heads"]), int(mx["kv_heads"])
        D, V = int(mx["dim"]), int(mx["vdim"])
        self.scale = float(mx["scale"])
        self.window = int((mx.get("mask") or {}).get("size") or 0)
        self.kv_source = config.kv_source(layer_index)
        self.K = pad_k(W)                  # stored inner size of h

        spec = ProjSpec(heads=H, kv_heads=G, dim=D, vdim=V,
                        eps=config.rms_norm_eps)
        # tensor name -> (first row, rows) of in_w
        self._in_rows: Dict[str, Tuple[int, int]] = {}
        at = 0

        def section(name: str, rows: int) -> int:
            nonlocal at
            off = at
            self._in_rows[name] = (off, rows)
            at = round_up(off + rows, 8)
            return off

        spec.q_off = section("mix.q", H * D)
        if self.kv_source is None:
            spec.k_off = section("mix.k", G * D)
            spec.v_off = section("mix.v", G * V)
        spec.g_off = section("mix.g", H * V)
        spec.act_col = round_up(H * V, 8)
        inner = H * V
        E = 0
        if mlp is not None and mlp["kind"] == "dense":
            spec.act, spec.ff = 1, int(mlp["ff"])
            spec.u_off = section("mlp.up", spec.ff)
        elif mlp is not None:
            rt = mlp["router"]
            E = spec.experts = int(rt["experts"])
            spec.identity = int(rt["identity"])
            spec.top = int(rt["top"])
            spec.router_scale = float(rt["scale"])
            if mlp.get("shared"):
                spec.act, spec.ff = 2, int(mlp["shared"]["ff"])
                spec.u_off = section("mlp.shared.gate", spec.ff)
                spec.u2_off = section("mlp.shared.up", spec.ff)
            # the router starts a 64-row block: the rows before it are a GEMM
            # of their own where it is computed apart
            at = round_up(at, 64)
            spec.router_off = at
            n = E + spec.identity
            self._in_rows["mlp.router"] = (at, n)
            spec.router_n = n
            if spec.act == 2:
                self._in_rows["mlp.shared.sg"] = (at + n, 1)
                spec.router_n += 1
            at += spec.router_n
        if spec.act:
            inner = spec.act_col + spec.ff
        spec.a2_cols = pad_k(inner)
        self.spec = spec
        self.E = E

        dt = config.dtype

        def p(*shape, dtype=dt):
            return torch.nn.Parameter(torch.empty(*shape, dtype=dtype),
                                      requires_grad=False)

        f32 = torch.float32
        self.norm_w = p(W, dtype=f32)
        self.q_norm_w = p(H * D, dtype=f32)
        if self.kv_source is None:
            self.k_norm_w = p(G * D, dtype=f32)
        self.slopes = torch.nn.Parameter(ref.distance_slopes(H),
                                         requires_grad=False)
        self.in_w = p(round_up(at, 64), self.K)
        self.out_w = p(round_up(W, 64), spec.a2_cols)
        if spec.routed:
            self.correction = p(E + spec.identity, dtype=f32)
        if E:
            Fe = int(mlp["expert"]["ff"])
            self.expert_gate_up_w = p(E, 2, round_up(Fe, 64), self.K)
            self.expert_down_w = p(E, round_up(W, 64), round_up(Fe, 64))

    # -- weights ----------------------------------------------------------
    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint tensors of this layer, without the layer prefix."""
        s, W = self.spec, self.config.hidden_size
        out = {n: (rows, W) for n, (_, rows) in self._in_rows.items()}
        out["norm1"] = (W,)
        out["mix.q.norm"] = (s.heads * s.dim,)
        if self.kv_source is None:
            out["mix.k.norm"] = (s.kv_heads * s.dim,)
        out["mix.o"] = (W, s.heads * s.vdim)
        if s.act == 1:
            out["mlp.down"] = (W, s.ff)
            out["mlp.act"] = (2,)
        elif s.act == 2:
            out["mlp.shared.down"] = (W, s.ff)
        if s.routed:
            out["mlp.correction"] = (s.experts + s.identity,)
        for e in range(self.E):
            Fe = int(self.mlp["expert"]["ff"])
            out[f"mlp.e{e}.gate"] = out[f"mlp.e{e}.up"] = (Fe, W)
            out[f"mlp.e{e}.down"] = (W, Fe)
        return out

    @torch.no_grad()
    def load_tensors(self, get: Callable[[str], torch.Tensor]) -> int:
        """Fill the fused, padded weights from get(name); returns the number
        of tensors read."""
        s, W = self.spec, self.config.hidden_size
        shapes = self.tensor_shapes()

        def take(name: str) -> torch.Tensor:
            t = get(name)
            if tuple(t.shape) != shapes[name]:
                raise ValueError(f"layer {self.global_index} {name}: shape "
                                 f"{tuple(t.shape)}, expected {shapes[name]}")
            return t

        for w in (self.in_w, self.out_w):
            w.zero_()
        for name, (off, rows) in self._in_rows.items():
            self.in_w[off:off + rows, :W].copy_(take(name))
        self.norm_w.copy_(take("norm1"))
        self.q_norm_w.copy_(take("mix.q.norm"))
        if self.kv_source is None:
            self.k_norm_w.copy_(take("mix.k.norm"))
        self.out_w[:W, :s.heads * s.vdim].copy_(take("mix.o"))
        if s.act:
            down = "mlp.down" if s.act == 1 else "mlp.shared.down"
            self.out_w[:W, s.act_col:s.act_col + s.ff].copy_(take(down))
        if s.act == 1:
            # the two curvatures, softplus applied once here
            a, b = F.softplus(take("mlp.act").double().cpu()).tolist()
            s.xielu_pos, s.xielu_neg = a, 0.5 + b
        if s.routed:
            self.correction.copy_(take("mlp.correction"))
        if self.E:
            gu, dn = self.expert_gate_up_w, self.expert_down_w
            gu.zero_()
            dn.zero_()
            Fe = int(self.mlp["expert"]["ff"])
            for e in range(self.E):
                gu[e, 0, :Fe, :W].copy_(take(f"mlp.e{e}.gate"))
                gu[e, 1, :Fe, :W].copy_(take(f"mlp.e{e}.up"))
                dn[e, :W, :Fe].copy_(take(f"mlp.e{e}.down"))
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
            if name.endswith("norm") or name == "norm1":
                return torch.ones(shape, device=dev)
            if name in ("mlp.act", "mlp.correction"):
                return torch.zeros(shape, device=dev)
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

    @torch.no_grad()
    def forward_tokens(self, x: torch.Tensor, pending: Optional[Pending],
                       batch: TokenBatch) -> Pending:
        """x (N, W) f32: the residual before `pending`, updated in place."""
        s, dt = self.spec, self.in_w.dtype
        h = ragged.residual_norm(x, pending, self.norm_w,
                                 self.config.norm_groups, s.eps, self.K, dt)
        parts, rparts, r0 = ragged.input_projection(h, self.in_w, s)
        kl = self._kv_layer()
        kp, vp = batch.k_pages(kl), batch.v_pages(kl)
        q, gate, a2, rt = ragged.proj_post(
            parts, rparts, r0, s, self.q_norm_w,
            self.k_norm_w if s.has_kv else None,
            self.correction if s.routed else None, batch, kp, vp, dt)
        routed = (ragged.moe_experts(h, self.expert_gate_up_w,
                                     self.expert_down_w, rt)
                  if self.E else None)
        ragged.attn_ragged(q, kp, vp, batch, a2, s.dim, s.vdim, self.scale,
                           self.window, self.slopes, gate)
        out = ragged.linear_parts(a2, self.out_w)
        return Pending(out, routed, rt, h if rt is not None else None)

    def forward_inference(self, hidden: torch.Tensor, kv, start_pos,
                          position_ids=None) -> torch.Tensor:
        """Lockstep step of one block (offloaded stacks call blocks singly)."""
        if position_ids is not None:
            raise NotImplementedError(
                "learned positions follow the sequence: no position_ids")
        B, T, W = hidden.shape
        x = hidden.reshape(B * T, W).to(torch.float32, copy=True)
        p = self.forward_tokens(x, None, lockstep_batch(kv, start_pos, B, T))
        ragged.residual_norm(x, p)
        return x.view(B, T, W)

    # -- training ---------------------------------------------------------
    def forward_train(self, hidden: torch.Tensor, start_pos: int = 0,
                      ) -> torch.Tensor:
        """Differentiable full-sequence path, no KV cache. A layer that reads
        another's keys takes them from the source block's last call, which
        BlockStack runs just before (`train_source`)."""
        s, W, dt = self.spec, self.config.hidden_size, self.in_w.dtype
        B, T, _ = hidden.shape
        x = hidden.float()

        def rows(name):
            off, n = self._in_rows[name]
            return F.linear(h, self.in_w[off:off + n, :W])

        def rms(t, w, groups=1):
            return ref.grouped_rms_norm(t, w, groups, s.eps).to(dt)

        h = rms(x, self.norm_w, self.config.norm_groups)
        q = rms(rows("mix.q"), self.q_norm_w).view(B, T, s.heads, s.dim)
        if self.kv_source is None:
            k = rms(rows("mix.k"), self.k_norm_w).view(B, T, s.kv_heads, s.dim)
            v = rows("mix.v").view(B, T, s.kv_heads, s.vdim)
            self._train_kv = (k, v)
        else:
            src = getattr(self, "train_source", None)
            if src is None or getattr(src, "_train_kv", None) is None:
                raise RuntimeError(
                    f"layer {self.global_index} needs layer "
                    f"{self.kv_source} in the same training span")
            k, v = src._train_kv
        rep = s.heads // s.kv_heads
        kf = k.float().repeat_interleave(rep, dim=2).permute(0, 2, 3, 1)
        vf = v.float().repeat_interleave(rep, dim=2).transpose(1, 2)
        sc = torch.matmul(q.float().transpose(1, 2), kf.contiguous()) * self.scale
        i = torch.arange(T, device=x.device)
        dist = i.view(T, 1) - i.view(1, T)
        sc = sc - self.slopes.view(-1, 1, 1) * dist.float()
        seen = dist >= 0
        if self.window:
            seen &= dist < self.window
        a = torch.matmul(torch.softmax(sc.masked_fill(~seen, float("-inf")), -1),
                         vf)
        a = a.transpose(1, 2).reshape(B, T, s.heads * s.vdim)
        a = (a * torch.sigmoid(rows("mix.g").float())).to(dt)
        y = F.linear(a, self.out_w[:W, :s.heads * s.vdim]).float()
        down = (self.out_w[:W, s.act_col:s.act_col + s.ff] if s.act else None)
        if s.act == 1:
            act = ref.xielu(rows("mlp.up").float(), s.xielu_pos, s.xielu_neg)
            y = y + F.linear(act.to(dt), down).float()
        if s.routed:
            flat = h.reshape(B * T, W)
            off, n = self._in_rows["mlp.router"]
            logits = flat.float() @ self.in_w[off:off + n, :W].float().t()
            ids, wts, idw = ref.route_topk(logits, self.correction, s.experts,
                                           s.top, s.router_scale)
            out = idw[:, None] * flat.float()
            Fe = int(self.mlp["expert"]["ff"])
            for e in range(self.E):
                t, c = (ids == e).nonzero(as_tuple=True)
                if t.numel() == 0:
                    continue
                g = F.linear(flat[t], self.expert_gate_up_w[e, 0, :Fe, :W])
                u = F.linear(flat[t], self.expert_gate_up_w[e, 1, :Fe, :W])
                o = F.linear((F.silu(g.float()) * u.float()).to(dt),
                             self.expert_down_w[e, :W, :Fe])
                out = out.index_add(0, t, o.float() * wts[t, c, None])
            y = y + out.view(B, T, W)
        if s.act == 2:
            off, _ = self._in_rows["mlp.shared.sg"]
            sg = torch.sigmoid(h.float() @ self.in_w[off:off + 1, :W].float().t())
            act = (F.silu(rows("mlp.shared.gate").float())
                   * rows("mlp.shared.up").float() * sg)
            y = y + F.linear(act.to(dt), down).float()
        return x + y

    def forward(self, *args, **kw):
        return self.forward_inference(*args, **kw)
