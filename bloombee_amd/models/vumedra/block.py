"""Vumedra decoder block on the ragged-batch ops.

A norm around each sublayer: x <- x + norm1b(mixer(norm1(x))), then
x <- x + norm2b(ff(norm2(x))); a norm has one weight for all coordinates. What a
sublayer adds is left Pending with its norm, and the next norm's launch folds it.

One GEMM reads the normed rows of a mixer:
    attention   in_w [q | k | v]                 biases, norm per head
    mlstm       in_w [q | k | v | gate | log gates (computed in f32)]
    rglru       in_w [y | x]
and one those of a feed-forward:
    dense       ff_w [gate | up]
    routed      ff_w [shared expert's up | router (computed in f32)]
"""
from __future__ import annotations

import math
from typing import Callable, Dict, Optional, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.kv.batch import TokenBatch, lockstep_batch
from bloombee_amd.models.vumedra.config import VumedraConfig
from bloombee_amd.ops import ragged, recurrent
from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.ragged import (FfSpec, HeadSpec, Pending, pad_k,
                                     round_up)
from bloombee_amd.ops.recurrent import RglruWeights

DECAY_SCALE = -8.0   # log a = DECAY_SCALE * r * softplus(lam)


class VumedraBlock(torch.nn.Module):
    token_batched = True   # BlockStack hands whole steps to forward_tokens
    hip_modules = ("_hip_ragged", "_hip_recurrent")

    def __init__(self, config: VumedraConfig, layer_index: int = 0, rope=None):
        super().__init__()
        self.config = config
        self.layer_index = layer_index     # BlockStack rebases it to its pool
        self.global_index = layer_index
        layer = config.layers[layer_index]
        self.kind, self.mlp = layer["type"], layer.get("mlp")
        W = config.hidden_size
        self.K = pad_k(W)                  # stored inner size of h
        dt, f32 = config.dtype, torch.float32

        def p(*shape, dtype=f32):
            return torch.nn.Parameter(torch.zeros(*shape, dtype=dtype),
                                      requires_grad=False)

        # tensor name -> (weight, first row, rows)
        self._rows: Dict[str, Tuple[str, int, int]] = {}
        at = 0

        def section(weight: str, name: str, rows: int, align: int = 8) -> int:
            nonlocal at
            off = round_up(at, align)
            self._rows[name] = (weight, off, rows)
            at = off + rows
            return off

        # plain f32 parameters: tensor name -> attribute, shape
        self._vectors: Dict[str, Tuple[str, Tuple[int, ...]]] = {}

        def vector(name: str, attr: str, *shape: int) -> None:
            self._vectors[name] = (attr, shape)
            setattr(self, attr, p(*shape))

        self._mixer(config, layer["mixer"], section, vector, p)
        self.in_w = p(round_up(at, 64), self.K, dtype=dt)
        self.out_w = p(round_up(W, 64), self.out_cols, dtype=dt)
        self.norms = ["norm1", "norm1b"]
        if self.mlp is not None:
            self.norms += ["norm2", "norm2b"]
            at = 0
            self._feed_forward(section, p)
            self.ff_w = p(round_up(at, 64), self.K, dtype=dt)
        for n in self.norms:
            setattr(self, n + "_w", p(W))

    def _mixer(self, config, mx, section, vector, p) -> None:
        dt = config.dtype
        if self.kind == "attention":
            H, G = int(mx["heads"]), int(mx["kv_heads"])
            D, V = int(mx["dim"]), int(mx["vdim"])
            qt = mx.get("q_temp") or {"coef": 0.0, "every": 1.0}
            s = HeadSpec(heads=H, kv_heads=G, dim=D, vdim=V,
                         eps=config.rms_norm_eps, temp_coef=float(qt["coef"]),
                         temp_every=float(qt["every"]))
            self.scale = float(mx["scale"])
            s.q_off = section("in_w", "mix.q", H * D)
            s.k_off = section("in_w", "mix.k", G * D)
            s.v_off = section("in_w", "mix.v", G * V)
            vector("mix.q.b", "q_b", H * D)
            vector("mix.k.b", "k_b", G * D)
            vector("mix.v.b", "v_b", G * V)
            vector("mix.q.norm", "q_norm_w", D)
            vector("mix.k.norm", "k_norm_w", D)
            # one more score of zero, without a value
            self.sink = p(H)
            self.inner = H * V
            self.out_cols = pad_k(self.inner)
        else:
            s = config.recurrent_spec(self.global_index)
            if self.kind == "mlstm":
                H = s.heads
                s.q_off = section("in_w", "mix.q", H * s.dim)
                s.k_off = section("in_w", "mix.k", H * s.dim)
                s.v_off = section("in_w", "mix.v", H * s.vdim)
                s.g_off = section("in_w", "mix.g", H * s.vdim)
                # the gates start a 64-row block: the rows before it are a GEMM
                # of their own where they are computed apart
                s.router_off = section("in_w", "mix.i", H, 64)
                section("in_w", "mix.f", H, 1)
                s.router_n = 2 * H
                self.gate_b = p(2 * H)
                vector("mix.norm", "o_norm_w", H * s.vdim)
                self.inner = H * s.vdim
            else:
                C, B, D = s.width, s.blocks, s.block
                s.y_off = section("in_w", "mix.y", C)
                s.x_off = section("in_w", "mix.x", C)
                vector("mix.y.b", "y_b", C)
                vector("mix.x.b", "x_b", C)
                vector("mix.conv.b", "conv_b", C)
                self.taps = p(s.taps, C)
                self.gates_w = p(B, 2, s.block_p, s.block_p, dtype=dt)
                self.gates_b = p(2, C)
                self.decay = p(C)
                self.inner = C
            self.out_cols = s.out_cols = pad_k(self.inner)
        self.spec = s

    def _feed_forward(self, section, p) -> None:
        W, dt = self.config.hidden_size, self.config.dtype
        f = self.ff_spec = FfSpec()
        self.E = 0
        if self.mlp["kind"] == "dense":
            f.act, f.ff = 1, int(self.mlp["ff"])
            f.gate_off = section("ff_w", "mlp.gate", f.ff)
            f.up_off = section("ff_w", "mlp.up", f.ff)
        else:
            shared, rt = self.mlp.get("shared"), self.mlp["router"]
            if shared:
                f.act, f.ff = 2, int(shared["ff"])
                f.up_off = section("ff_w", "mlp.shared.up", f.ff)
            self.E = f.router_n = int(rt["experts"])
            f.top, f.sigmoid = int(rt["top"]), True
            f.router_off = section("ff_w", "mlp.router", self.E, 64)
            self.Fe = Fe = int(self.mlp["expert"]["ff"])
            self.expert_up_w = p(self.E, 1, round_up(Fe, 64), self.K, dtype=dt)
            self.expert_down_w = p(self.E, round_up(W, 64), round_up(Fe, 64),
                                   dtype=dt)
        if f.act:
            f.cols = pad_k(f.ff)
            self.down_w = p(round_up(W, 64), f.cols, dtype=dt)

    # -- weights ----------------------------------------------------------
    def _down_name(self) -> Optional[str]:
        if self.mlp is None or not self.ff_spec.act:
            return None
        return "mlp.down" if self.ff_spec.act == 1 else "mlp.shared.down"

    def tensor_shapes(self) -> Dict[str, Tuple[int, ...]]:
        """Checkpoint tensors of this layer, without the layer prefix."""
        s, W = self.spec, self.config.hidden_size
        out = {n: (rows, W) for n, (_, _, rows) in self._rows.items()}
        out.update({n: shape for n, (_, shape) in self._vectors.items()})
        out.update({n: () for n in self.norms})
        out["mix.o"] = (W, self.inner)
        if self.kind == "mlstm":
            out["mix.i.b"] = out["mix.f.b"] = (s.heads,)
        elif self.kind == "rglru":
            out["mix.conv"] = (s.width, s.taps)
            out["mix.lam"] = (s.width,)
            for n in ("mix.ra", "mix.ri"):
                out[n] = (s.blocks, s.block, s.block)
                out[n + ".b"] = (s.blocks, s.block)
        if self._down_name():
            out[self._down_name()] = (W, self.ff_spec.ff)
        for e in range(self.E if self.mlp is not None else 0):
            out[f"mlp.e{e}.up"], out[f"mlp.e{e}.down"] = (self.Fe, W), (W, self.Fe)
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

        for name, (weight, off, rows) in self._rows.items():
            getattr(self, weight)[off:off + rows, :W].copy_(take(name))
        for name, (attr, _) in self._vectors.items():
            getattr(self, attr).copy_(take(name))
        for name in self.norms:
            getattr(self, name + "_w").copy_(take(name))
        self.out_w[:W, :self.inner].copy_(take("mix.o"))
        if self.kind == "mlstm":
            self.gate_b[:s.heads].copy_(take("mix.i.b"))
            self.gate_b[s.heads:].copy_(take("mix.f.b"))
        elif self.kind == "rglru":
            self.taps.copy_(take("mix.conv").t())
            for g, n in enumerate(("mix.ra", "mix.ri")):
                self.gates_w[:, g, :s.block, :s.block].copy_(take(n))
                self.gates_b[g].copy_(take(n + ".b").reshape(-1))
            # softplus applied once here
            self.decay.copy_(DECAY_SCALE * F.softplus(take("mix.lam").double()))
        if self._down_name():
            self.down_w[:W, :self.ff_spec.ff].copy_(take(self._down_name()))
        for e in range(self.E if self.mlp is not None else 0):
            self.expert_up_w[e, 0, :self.Fe, :W].copy_(take(f"mlp.e{e}.up"))
            self.expert_down_w[e, :W, :self.Fe].copy_(take(f"mlp.e{e}.down"))
        return len(shapes)

    @torch.no_grad()
    def init_random(self, seed: Optional[int] = None):
        s = seed if seed is not None else 1234 + self.global_index
        dev = self.in_w.device
        gen = torch.Generator(device=dev).manual_seed(s)
        std = 0.02 / math.sqrt(2 * self.config.num_hidden_layers)
        shapes = self.tensor_shapes()
        # forgetting slowly
        means = {"mix.f.b": 3.0, "mix.lam": -4.0}

        def draw(name: str) -> torch.Tensor:
            shape = shapes[name]
            if name.startswith("norm") or name.endswith("norm"):
                return torch.ones(shape, device=dev)
            if name in means or name.endswith(".b"):
                return torch.full(shape, means.get(name, 0.0), device=dev)
            return torch.randn(shape, generator=gen, dtype=torch.float32,
                               device=dev).mul_(std)

        self.load_tensors(draw)
        return self

    # -- inference --------------------------------------------------------
    def _mix(self, h: torch.Tensor, batch: TokenBatch) -> torch.Tensor:
        s, dt = self.spec, self.in_w.dtype
        if self.kind == "mlstm":
            parts, gparts, i0 = ragged.input_projection(h, self.in_w, s)
            return recurrent.mlstm_mix(
                parts, gparts, i0, s, self.gate_b, self.o_norm_w,
                batch.cache.state(self.layer_index), batch, dt)
        parts = ragged.linear_parts(h, self.in_w)
        if self.kind == "rglru":
            w = RglruWeights(self.y_b, self.x_b, self.taps, self.conv_b,
                             self.gates_w, self.gates_b, self.decay)
            return recurrent.rglru_mix(
                parts, s, w, batch.cache.state(self.layer_index), batch, dt)
        kp, vp = batch.k_pages(self.layer_index), batch.v_pages(self.layer_index)
        q = ragged.head_post(parts, s, (self.q_b, self.k_b, self.v_b),
                             self.q_norm_w, self.k_norm_w, batch, kp, vp, dt)
        make = torch.empty if self.out_cols == self.inner else torch.zeros
        out = make(h.shape[0], self.out_cols, dtype=dt, device=h.device)
        ragged.attn_ragged(q, kp, vp, batch, out, s.dim, s.vdim, self.scale,
                           sinks=self.sink)
        return out

    @torch.no_grad()
    def forward_tokens(self, x: torch.Tensor, pending: Optional[Pending],
                       batch: TokenBatch) -> Pending:
        """x (N, W) f32: the residual before `pending`, updated in place."""
        eps, dt = self.config.rms_norm_eps, self.in_w.dtype
        h = ragged.residual_norm(x, pending, self.norm1_w, 1, eps, self.K, dt)
        left = Pending(ragged.linear_parts(self._mix(h, batch), self.out_w),
                       norm=self.norm1b_w, eps=eps)
        if self.mlp is None:
            return left
        f = self.ff_spec
        h = ragged.residual_norm(x, left, self.norm2_w, 1, eps, self.K, dt)
        parts, rparts, r0 = ragged.input_projection(h, self.ff_w, f)
        a, rt = ragged.ff_post(parts, rparts, r0, f, None, h.shape[0], h.device,
                               dt)
        routed = (ragged.moe_experts(h, self.expert_up_w, self.expert_down_w, rt,
                                     weight_input=True) if self.E else None)
        out = ragged.linear_parts(a, self.down_w) if f.act else None
        return Pending(out, routed, rt, norm=self.norm2b_w, eps=eps)

    def forward_inference(self, hidden: torch.Tensor, kv, start_pos,
                          position_ids=None) -> torch.Tensor:
        """Lockstep step of one block (offloaded stacks call blocks singly)."""
        if position_ids is not None:
            raise NotImplementedError(
                "recurrent layers follow the sequence: no position_ids")
        B, T, W = hidden.shape
        x = hidden.reshape(B * T, W).to(torch.float32, copy=True)
        self.forward_tokens(x, None, lockstep_batch(kv, start_pos, B, T)).settle(x)
        return x.view(B, T, W)

    # -- training ---------------------------------------------------------
    def _train_mixer(self, h: torch.Tensor, start_pos: int) -> torch.Tensor:
        s, W, dt = self.spec, self.config.hidden_size, self.in_w.dtype
        B, T, _ = h.shape

        def rows(name):
            _, off, n = self._rows[name]
            return F.linear(h, self.in_w[off:off + n, :W]).float()

        if self.kind == "mlstm":
            H, D, V = s.heads, s.dim, s.vdim
            q = rows("mix.q").view(B, T, H, D) * D ** -0.5
            k = rows("mix.k").view(B, T, H, D)
            v = rows("mix.v").view(B, T, H, V)
            i, f = ref.mlstm_gates(torch.cat([rows("mix.i"), rows("mix.f")], -1),
                                   self.gate_b, s.cap)
            zero = (h.new_zeros(H, D, V).float(), h.new_zeros(H, D).float(),
                    h.new_zeros(H).float())
            o = torch.stack([ref.mlstm_scan(q[b], k[b], v[b], i[b], f[b], *zero)[0]
                             for b in range(B)])
            o = ref.grouped_rms_norm(o, torch.ones(V, device=h.device), 1, s.eps)
            o = (o.reshape(B, T, H * V) * self.o_norm_w
                 * torch.sigmoid(rows("mix.g")))
        elif self.kind == "rglru":
            D = s.block
            u = ref.causal_conv(rows("mix.x") + self.x_b,
                                h.new_zeros(B, s.taps - 1, s.width).float(),
                                self.taps, self.conv_b).to(dt)
            la, x = ref.rglru_inputs(u, self.gates_w[:, :, :D, :D], self.gates_b,
                                     self.decay)
            o = torch.stack([ref.rglru_scan(la[b], x[b],
                                            torch.zeros_like(x[b, 0]))[0]
                             for b in range(B)])
            o = o * ref.gelu_tanh(rows("mix.y") + self.y_b)
        else:
            H, G, D, V = s.heads, s.kv_heads, s.dim, s.vdim
            pos = torch.arange(start_pos, start_pos + T, device=h.device)
            q = ref.grouped_rms_norm((rows("mix.q") + self.q_b).view(B, T, H, D),
                                     self.q_norm_w, 1, s.eps)
            q = q * ref.query_temperature(pos, s.temp_coef,
                                          s.temp_every).view(T, 1, 1)
            k = ref.grouped_rms_norm((rows("mix.k") + self.k_b).view(B, T, G, D),
                                     self.k_norm_w, 1, s.eps)
            v = (rows("mix.v") + self.v_b).view(B, T, G, V)
            k = k.to(dt).float().repeat_interleave(H // G, dim=2)
            v = v.to(dt).float().repeat_interleave(H // G, dim=2)
            sc = torch.matmul(q.to(dt).float().transpose(1, 2).contiguous(),
                              k.permute(0, 2, 3, 1).contiguous()) * self.scale
            later = torch.ones(T, T, dtype=torch.bool, device=h.device).triu(1)
            sc = sc.masked_fill(later, float("-inf"))
            sc = torch.cat([sc, self.sink.view(1, H, 1, 1).expand(B, H, T, 1)], -1)
            o = torch.matmul(torch.softmax(sc, -1)[..., :T],
                             v.transpose(1, 2).contiguous())
            o = o.transpose(1, 2).reshape(B, T, H * V)
        return F.linear(o.to(dt), self.out_w[:W, :self.inner]).float()

    def _train_ff(self, h: torch.Tensor) -> torch.Tensor:
        f, W, dt = self.ff_spec, self.config.hidden_size, self.in_w.dtype

        def rows(name, x=h):
            _, off, n = self._rows[name]
            return F.linear(x, self.ff_w[off:off + n, :W]).float()

        y = 0
        if f.act:
            a = (F.silu(rows("mlp.gate")) * rows("mlp.up") if f.act == 1
                 else torch.relu(rows("mlp.shared.up")) ** 2)
            y = F.linear(a.to(dt), self.down_w[:W, :f.ff]).float()
        if not self.E:
            return y
        flat = h.reshape(-1, W)
        _, off, n = self._rows["mlp.router"]
        logits = flat.float() @ self.ff_w[off:off + n, :W].float().t()
        ids, wts, _ = ref.route_topk(logits, None, self.E, f.top, f.scale,
                                     f.sigmoid)
        out = torch.zeros_like(flat, dtype=torch.float32)
        for e in range(self.E):
            t, c = (ids == e).nonzero(as_tuple=True)
            if t.numel() == 0:
                continue
            u = F.linear(flat[t], self.expert_up_w[e, 0, :self.Fe, :W]).float()
            a = torch.relu(u * wts[t, c, None]) ** 2
            out = out.index_add(0, t, F.linear(
                a.to(dt), self.expert_down_w[e, :W, :self.Fe]).float())
        return y + out.view(*h.shape[:-1], W)

    def forward_train(self, hidden: torch.Tensor, start_pos: int = 0,
                      ) -> torch.Tensor:
        """Differentiable full-sequence path, no KV cache and no state."""
        dt, eps = self.in_w.dtype, self.config.rms_norm_eps

        def rms(t, w):
            return ref.grouped_rms_norm(t, w, 1, eps)

        x = hidden.float()
        y = self._train_mixer(rms(x, self.norm1_w).to(dt), start_pos)
        x = x + rms(y, self.norm1b_w)
        if self.mlp is None:
            return x
        return x + rms(self._train_ff(rms(x, self.norm2_w).to(dt)),
                       self.norm2b_w)

    def forward(self, *args, **kw):
        return self.forward_inference(*args, **kw)
