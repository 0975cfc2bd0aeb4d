"""Fused steps of blocks over ragged batches.

The pieces, in the order a parallel-residual layer runs them (N rows, one per
token):

  residual_norm  x += what the previous layer left pending; h = norm(x)
  linear_parts   h @ W^T, as split-K f32 partials on decode-sized batches
  proj_post      q/k norm, K/V pages, activation, routing — one launch that
                 also folds the partials
  moe_experts    routed experts
  attn_ragged    attention + output gate
  linear_parts   [attention | activation] @ [W_o | W_down]^T, left Pending

Layers with a norm after every sum use sum_norm instead, and clamped_glu for
their feed-forward; other mixers are in ops/mixers.py.

Device tensors run the _hip_ragged extension and fail loudly without it; CPU
tensors run the forms in ops/reference.py. Activations are bf16 or f32; the
residual, norms, routing and attention weights are f32 in both.
"""
from __future__ import annotations

import importlib
from dataclasses import dataclass
from typing import Optional, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.ops import reference as ref

_hip_ragged = None   # loaded by the first device call

# head sizes the MFMA attention kernels are compiled for; pages and q are
# padded to the next one with zeros
HEAD_SIZES = (32, 64, 128, 256)
SKINNY_ROWS = 32   # up to here a GEMM is a weight stream (split-K kernel)


def _ext():
    global _hip_ragged
    if _hip_ragged is None:
        try:
            _hip_ragged = importlib.import_module("bloombee_amd.ops._hip_ragged")
        except ImportError as e:
            raise RuntimeError(
                "the _hip_ragged extension is not built but a tensor is on "
                "GPU. Run `python setup.py hip` (PYTORCH_ROCM_ARCH=gfx950). "
                f"Import error was: {e}") from e
    return _hip_ragged


def round_up(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def pad_head(d: int) -> int:
    """Stored size of a head of d elements."""
    for s in HEAD_SIZES:
        if d <= s:
            return s
    return round_up(d, 8)


def pad_k(k: int) -> int:
    """Stored length of a GEMM's inner dimension: 256 (the pipelined weight
    stream's stage) where that costs little, else 64."""
    p = round_up(k, 256)
    return p if p <= k * 1.07 else round_up(k, 64)


@dataclass
class Routing:
    ids: torch.Tensor   # (N, top) int32, -1 = identity expert
    wts: torch.Tensor   # (N, top) f32
    idw: torch.Tensor   # (N,) f32: summed weight of identity experts


@dataclass
class Pending:
    """What a layer still owes the residual: the output GEMM's partials and,
    for routed layers, the experts' rows and the layer's own input."""
    parts: torch.Tensor                      # (ks, N, >= W)
    routed: Optional[torch.Tensor] = None    # (N, top, >= W)
    routing: Optional[Routing] = None
    h: Optional[torch.Tensor] = None         # (N, >= W)

    def settle(self, x: torch.Tensor) -> None:
        residual_norm(x, self)


@dataclass
class Carried:
    """A layer that ends with a norm owes nothing; what it hands on is the
    residual's rows in the activation type, the next layer's input."""
    h: torch.Tensor                          # (N, stored inner size)

    def settle(self, x: torch.Tensor) -> None:
        pass


def residual_norm(x: torch.Tensor, pending: Optional[Pending],
                  weight: Optional[torch.Tensor] = None, groups: int = 1,
                  eps: float = 1e-5, cols: int = 0,
                  dtype: torch.dtype = torch.bfloat16,
                  ) -> Optional[torch.Tensor]:
    """x (N, W) f32 += pending, in place; returns norm(x) as (N, cols) in
    dtype with zero columns beyond W, or None without a weight."""
    N, W = x.shape
    p = pending
    rt = p.routing if p is not None else None
    if x.is_cuda:
        h = (torch.empty(N, cols or W, dtype=dtype, device=x.device)
             if weight is not None else None)
        _ext().residual_norm(
            x, p.parts if p else None,
            p.routed if p and p.routed is not None else None,
            rt.ids if rt else None, rt.idw if rt else None,
            p.h if rt else None, weight, groups, eps, h, 1.0, None, False)
        return h
    if p is not None:
        d = p.parts.float().sum(0)[:, :W]
        if rt is not None:
            if p.routed is not None:
                d = d + p.routed.float().sum(1)[:, :W]
            d = d + rt.idw[:, None] * p.h[:, :W].float()
        x += d
    if weight is None:
        return None
    y = ref.grouped_rms_norm(x, weight, groups, eps).to(dtype)
    return F.pad(y, (0, (cols or W) - W))


def sum_norm(x: torch.Tensor, parts: torch.Tensor,
             bias: Optional[torch.Tensor], weight: torch.Tensor, alpha: float,
             eps: float, cols: int, dtype: torch.dtype) -> torch.Tensor:
    """Norm after the sum: x (N, W) f32 <- rms(alpha x + sum of parts + bias)
    * weight, in place; returns its rows as (N, cols) in dtype with zero
    columns beyond W. parts (ks, N, >= W)."""
    N, W = x.shape
    if x.is_cuda:
        h = torch.empty(N, cols, dtype=dtype, device=x.device)
        _ext().residual_norm(x, parts, None, None, None, None, weight, 1, eps,
                             h, alpha, bias, True)
        return h
    y = alpha * x + parts.float().sum(0)[:, :W]
    if bias is not None:
        y = y + bias
    x.copy_(ref.grouped_rms_norm(y, weight, 1, eps))
    return input_rows(x, cols, dtype)


def input_rows(x: torch.Tensor, cols: int, dtype: torch.dtype) -> torch.Tensor:
    """x (N, W) f32 as (N, cols) in dtype, zero columns beyond W."""
    return F.pad(x.to(dtype), (0, cols - x.shape[1])).contiguous()


def clamped_glu(parts: torch.Tensor, g_off: int, u_off: int, ff: int,
                gate_b: Optional[torch.Tensor], up_b: Optional[torch.Tensor],
                limit: float, slope: float, cols: int,
                dtype: torch.dtype) -> torch.Tensor:
    """Gated feed-forward activation of a [gate | up] GEMM output in parts:
    g = min(gate, limit), u = clamp(up, -limit, limit),
    g * sigmoid(slope * g) * (u + 1), as (N, cols) with zeros beyond ff."""
    if parts.is_cuda:
        out = torch.empty(parts.shape[1], cols, dtype=dtype,
                          device=parts.device)
        _ext().clamped_glu(parts, g_off, u_off, ff, gate_b, up_b, limit, slope,
                           out)
        return out
    y = parts.float().sum(0)
    a = ref.clamped_glu(y[:, g_off:g_off + ff], y[:, u_off:u_off + ff], gate_b,
                        up_b, limit, slope)
    return F.pad(a.to(dtype), (0, cols - ff))


def softcap_(z: torch.Tensor, cap: float) -> torch.Tensor:
    """z <- cap * tanh(z / cap), f32, in place."""
    if z.is_cuda:
        _ext().softcap(z, cap)
        return z
    return z.div_(cap).tanh_().mul_(cap)


def embed_rows(ids: torch.Tensor, positions: torch.Tensor,
               table: torch.Tensor, pos_table: Optional[torch.Tensor],
               ) -> torch.Tensor:
    """table[ids] (+ pos_table[positions]) in f32, (..., W)."""
    if table.is_cuda:
        x = _ext().embed_rows(ids.reshape(-1).int(),
                              positions.reshape(-1).int(), table, pos_table)
        return x.view(*ids.shape, -1)
    if pos_table is None:
        return F.embedding(ids.long(), table).float()
    pos = positions.long().clamp(min=0)
    return (F.embedding(ids.long(), table).float()
            + F.embedding(pos, pos_table).float())


def linear_parts(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x (M, K) @ w (N, K)^T as (splits, M, N): f32 partials of the split-K
    weight-stream kernel for up to 32 bf16 rows, else one part in x's type
    from the vendor GEMM."""
    if (x.is_cuda and x.dtype == torch.bfloat16 and x.shape[0] <= SKINNY_ROWS):
        return _ext().gemm_parts(x, w, 0)
    return F.linear(x, w).unsqueeze(0)


def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x (M, K) @ w (N, K)^T with an f32 result, a few rows at a time (vocab
    projection of the rows that are sampled). One split: a vocabulary is wide,
    and a library sum over splits may not be capturable."""
    if x.is_cuda and x.dtype == torch.bfloat16:
        outs = [_ext().gemm_parts(xs.contiguous(), w, 1)[0]
                for xs in x.split(SKINNY_ROWS)]
        return outs[0] if len(outs) == 1 else torch.cat(outs)
    return F.linear(x.float(), w.float())


@dataclass
class ProjSpec:
    """Where the sections of the fused input projection lie, and what is done
    with them. Offsets are columns of the GEMM output; -1 = absent. The router
    section (experts' logits, then the shared expert's gate) is last, so that
    a bf16 GEMM can leave it out and an f32 one compute it."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    eps: float
    q_off: int = 0
    k_off: int = -1
    v_off: int = -1
    g_off: int = 0
    u_off: int = -1
    u2_off: int = -1
    router_off: int = -1     # first router column of the fused weight
    router_n: int = 0        # router columns in use
    act: int = 0             # 0 none, 1 xielu, 2 silu(gate) * up, gated
    ff: int = 0
    act_col: int = 0         # first activation column of a2
    a2_cols: int = 0         # inner size of the output projection
    xielu_pos: float = 0.0
    xielu_neg: float = 0.0
    experts: int = 0
    identity: int = 0
    top: int = 0
    router_scale: float = 1.0

    @property
    def has_kv(self) -> bool:
        return self.k_off >= 0

    @property
    def routed(self) -> bool:
        return self.experts + self.identity > 0


def input_projection(h: torch.Tensor, w: torch.Tensor, spec: ProjSpec,
                     ) -> Tuple[torch.Tensor, Optional[torch.Tensor], int]:
    """(parts, router parts, first router column in them)."""
    r = spec.router_off
    if r < 0:
        return linear_parts(h, w), None, 0
    if h.is_cuda and h.dtype == torch.bfloat16 and h.shape[0] > SKINNY_ROWS:
        return (F.linear(h, w[:r]).unsqueeze(0),
                _ext().router_gemm(h, w[r:r + spec.router_n]), 0)
    if not h.is_cuda:
        return (F.linear(h, w[:r]).unsqueeze(0),
                F.linear(h.float(), w[r:r + spec.router_n].float()).unsqueeze(0),
                0)
    parts = linear_parts(h, w)      # f32 either way
    return parts, parts, r


def proj_post(parts: torch.Tensor, rparts: Optional[torch.Tensor], r0: int,
              spec: ProjSpec, q_norm: torch.Tensor,
              k_norm: Optional[torch.Tensor],
              correction: Optional[torch.Tensor], batch,
              k_pages: torch.Tensor, v_pages: torch.Tensor,
              dtype: torch.dtype):
    """Returns q (N, H, stored dim), gate (N, H*vdim), a2 (N, a2_cols) with
    the attention columns still to be written, and Routing or None."""
    _, N, ld = parts.shape
    dev = parts.device
    H, G, D, V = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    dkp = k_pages.shape[3]
    sg = spec.experts + spec.identity
    if parts.is_cuda:
        q = torch.empty(N, H, dkp, dtype=dtype, device=dev)
        a2 = torch.empty(N, spec.a2_cols, dtype=dtype, device=dev)
        # one part of the activation type: the gate is read where it lies
        in_place = parts.shape[0] == 1 and parts.dtype == dtype
        gate = (parts[0][:, spec.g_off:spec.g_off + H * V] if in_place
                else torch.empty(N, H * V, dtype=dtype, device=dev))
        rt = None
        if spec.routed:
            rt = Routing(
                torch.empty(N, spec.top, dtype=torch.int32, device=dev),
                torch.empty(N, spec.top, dtype=torch.float32, device=dev),
                torch.empty(N, dtype=torch.float32, device=dev))
        _ext().proj_post(
            parts, rparts,
            [spec.q_off, spec.k_off, spec.v_off, spec.g_off, spec.u_off,
             spec.u2_off, r0, r0 + sg, H, G, D, V, int(spec.has_kv), spec.act,
             spec.ff, spec.act_col, spec.experts, spec.identity, spec.top],
            [spec.eps, spec.xielu_pos, spec.xielu_neg, spec.router_scale],
            q_norm, k_norm, correction, q, None if in_place else gate, a2,
            k_pages, v_pages, batch.page_table, batch.tok_seq, batch.tok_pos,
            rt.ids if rt else None, rt.wts if rt else None,
            rt.idw if rt else None)
        return q, gate, a2, rt

    y = parts.float().sum(0)
    cut = lambda off, n: y[:, off:off + n]
    q = ref.grouped_rms_norm(cut(spec.q_off, H * D), q_norm, 1, spec.eps)
    q = F.pad(q.view(N, H, D), (0, dkp - D)).to(dtype)
    if spec.has_kv:
        k = ref.grouped_rms_norm(cut(spec.k_off, G * D), k_norm, 1, spec.eps)
        k = k.view(N, G, D).to(dtype)
        v = cut(spec.v_off, G * V).reshape(N, G, V).to(dtype)
        P = k_pages.shape[2]
        live = (batch.tok_pos >= 0).nonzero()[:, 0]
        pos = batch.tok_pos[live].long()
        page = batch.page_table[batch.tok_seq[live].long(), pos // P].long()
        k_pages[page, :, pos % P, :D] = k[live]
        v_pages[page, :, :V, pos % P] = v[live]
    gate = cut(spec.g_off, H * V).to(dtype)
    a2 = torch.zeros(N, spec.a2_cols, dtype=dtype, device=dev)
    logits = rparts.sum(0)[:, r0:] if rparts is not None else None
    if spec.act == 1:
        act = ref.xielu(cut(spec.u_off, spec.ff), spec.xielu_pos,
                        spec.xielu_neg)
    elif spec.act == 2:
        g = cut(spec.u_off, spec.ff)
        act = (g * torch.sigmoid(g) * cut(spec.u2_off, spec.ff)
               * torch.sigmoid(logits[:, sg:sg + 1]))
    if spec.act:
        a2[:, spec.act_col:spec.act_col + spec.ff] = act.to(dtype)
    rt = None
    if spec.routed:
        rt = Routing(*ref.route_topk(logits[:, :sg], correction, spec.experts,
                                     spec.top, spec.router_scale))
    return q, gate, a2, rt


def moe_experts(h: torch.Tensor, gate_up: torch.Tensor, down: torch.Tensor,
                rt: Routing) -> torch.Tensor:
    """(N, top, W) weighted outputs of the chosen experts; the rows of
    identity choices are not defined. gate_up (E, 2, F, K), down (E, W, F),
    K, F and W padded to 64."""
    if h.is_cuda:
        return _ext().moe_experts(h, gate_up, down, rt.ids, rt.wts)
    return ref.moe_experts(h, gate_up, down, rt.ids, rt.wts)


def attn_ragged(q: torch.Tensor, k_pages: torch.Tensor,
                v_pages: Optional[torch.Tensor],
                batch, out: torch.Tensor, dim: int, vdim: int, scale: float,
                window: int = 0, slopes: Optional[torch.Tensor] = None,
                gate: Optional[torch.Tensor] = None,
                sinks: Optional[torch.Tensor] = None,
                table: Optional[torch.Tensor] = None,
                portions_only: bool = False) -> None:
    """Attention of a ragged batch into out[:, :H*vdim] (see
    reference.attn_ragged). Without v_pages the values are the first vdim
    elements of the keys. table: page table of pages that are not the
    cache's; portions_only leaves the rows of single tokens alone (where the
    sizes are those of the tiled kernels)."""
    table = batch.page_table if table is None else table
    if q.is_cuda:
        dec = batch.dec_list[:0] if portions_only else batch.dec_list
        _ext().attn_ragged(
            q, k_pages, v_pages, table, batch.tok_seq, batch.tok_pos, batch.cu,
            batch.q_start, batch.pre_list, dec, batch.max_new, batch.max_ctx,
            dim, vdim, scale, window, slopes, sinks, gate, out)
        return
    n = q.shape[1] * vdim
    out[:, :n] = ref.attn_ragged(q, k_pages, v_pages, batch, dim, vdim, scale,
                                 window, slopes, gate, sinks)
