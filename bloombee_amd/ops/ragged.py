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
their feed-forward. Layers with a norm around every sublayer leave sums Pending
with the norm they pass first; where attention and feed-forward have inputs of
their own, head_post (norms per head) or rope_post (rotations) and ff_post take
proj_post's place. join_rows lets a product read the residual beside other rows
and put its result in the residual's place. Other mixers are in ops/mixers.py and
ops/recurrent.py.

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
ROUTER_COLS = 256   # beyond, the vendor GEMM makes 32-bit columns, too


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
    idw: Optional[torch.Tensor]   # (N,) f32: summed weight of identity experts


@dataclass
class Pending:
    """What a layer still owes the residual: the output GEMM's partials and,
    for routed layers, the experts' rows and the layer's own input; with norm,
    all of it is RMS-normed with these weights first. The residual is scaled by
    keep before it is added: 0 puts the sum in its place."""
    parts: Optional[torch.Tensor]            # (ks, N, >= W)
    routed: Optional[torch.Tensor] = None    # (N, top, >= W)
    routing: Optional[Routing] = None
    h: Optional[torch.Tensor] = None         # (N, >= W)
    norm: Optional[torch.Tensor] = None      # (W,) f32
    eps: float = 0.0                         # of that norm
    bias: Optional[torch.Tensor] = None      # (W,) f32, added to parts
    keep: float = 1.0

    def settle(self, x: torch.Tensor) -> None:
        residual_norm(x, self, eps=self.eps)


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
    """x (N, W) f32 += pending, in place (rows may lie apart); returns norm(x) as
    (N, cols) in dtype with zero columns beyond W, or None without a weight. eps
    is that of the pending sum's own norm, too, if it has one."""
    N, W = x.shape
    p = pending
    rt = p.routing if p is not None else None
    idw = rt.idw if rt is not None else None
    if x.is_cuda:
        h = (torch.empty(N, cols or W, dtype=dtype, device=x.device)
             if weight is not None else None)
        _ext().residual_norm(
            x, p.parts if p else None,
            p.routed if p and p.routed is not None else None,
            rt.ids if rt else None, idw, p.h if idw is not None else None,
            weight, groups, eps, h, p.keep if p else 1.0, p.bias if p else None,
            False, p.norm if p else None, None)
        return h
    if p is not None:
        d = (p.parts.float().sum(0)[:, :W] if p.parts is not None
             else torch.zeros_like(x))
        if p.bias is not None:
            d = d + p.bias
        if p.routed is not None:
            d = d + p.routed.float().sum(1)[:, :W]
        if idw is not None:
            d = d + idw[:, None] * p.h[:, :W].float()
        if p.norm is not None:
            d = ref.grouped_rms_norm(d, p.norm, 1, eps)
        x.mul_(p.keep).add_(d)
    if weight is None:
        return None
    y = ref.grouped_rms_norm(x, weight, groups, eps).to(dtype)
    return F.pad(y, (0, (cols or W) - W))


def join_rows(x: torch.Tensor, pending: Optional[Pending],
              other: torch.Tensor, cols: int, dtype: torch.dtype) -> torch.Tensor:
    """x (N, W) f32 += pending, in place; returns [x | other] as (N, cols) in
    dtype with zero columns beyond 2 W. other (N, W) f32; the rows of both may lie
    apart."""
    p = pending
    if x.is_cuda:
        rt = p.routing if p is not None else None
        idw = rt.idw if rt is not None else None
        h = torch.empty(x.shape[0], cols, dtype=dtype, device=x.device)
        _ext().residual_norm(
            x, p.parts if p else None, p.routed if p else None,
            rt.ids if rt else None, idw, p.h if idw is not None else None, None,
            1, p.eps if p else 0.0, h, p.keep if p else 1.0,
            p.bias if p else None, False, p.norm if p else None, other)
        return h
    if p is not None:
        p.settle(x)
    return input_rows(torch.cat([x, other], 1), cols, dtype)


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
                             h, alpha, bias, True, None, None)
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


def sinusoid_turns(width: int) -> torch.Tensor:
    """Frequencies 10000^(-2 i / width) over 2 pi of a sinusoidal position
    vector, sine at entry 2 i and cosine at 2 i + 1; float64."""
    i = torch.arange((width + 1) // 2, dtype=torch.float64)
    base = torch.tensor(10000.0, dtype=torch.float64)
    return torch.pow(base, -2.0 * i / width) / (2 * torch.pi)


@dataclass
class PairTable:
    """Embedding of token pairs: row (previous * mul_prev + token * mul_cur)
    mod buckets, the last row where there is no previous token."""
    table: torch.Tensor   # (buckets + 1, W)
    mul_prev: int
    mul_cur: int

    @property
    def buckets(self) -> int:
        return self.table.shape[0] - 1

    def rows(self, ids: torch.Tensor, prev: torch.Tensor) -> torch.Tensor:
        r = (prev.long() * self.mul_prev + ids.long() * self.mul_cur) \
            % self.buckets
        return torch.where(prev < 0, self.buckets, r)


def previous_ids(ids: torch.Tensor, last: torch.Tensor) -> torch.Tensor:
    """The token before each of ids (B, T); last (B,): the one before a row's
    first, -1 = none."""
    last = last.to(device=ids.device, dtype=ids.dtype).view(-1, 1)
    return torch.cat([last, ids[:, :-1]], 1)


def embed_rows(ids: torch.Tensor, positions: torch.Tensor,
               table: torch.Tensor, pos_table: Optional[torch.Tensor],
               prev: Optional[torch.Tensor] = None,
               pairs: Optional[PairTable] = None,
               turns: Optional[torch.Tensor] = None, scale: float = 1.0,
               copies: int = 1) -> torch.Tensor:
    """scale * table[ids] (+ pos_table[positions]) (+ the row of each token and
    its predecessor) (+ sinusoidal positions) in f32, `copies` times side by side:
    (..., copies * W)."""
    if table.is_cuda:
        x = _ext().embed_rows(
            ids.reshape(-1).int(), positions.reshape(-1).int(), table, pos_table,
            prev.reshape(-1).int() if pairs is not None else None,
            pairs.table if pairs is not None else None,
            [pairs.buckets, pairs.mul_prev, pairs.mul_cur]
            if pairs is not None else [], turns, scale, copies)
        return x.view(*ids.shape, -1)
    x = F.embedding(ids.long(), table).float() * scale
    pos = positions.long().clamp(min=0)
    if pos_table is not None:
        x = x + F.embedding(pos, pos_table).float()
    if pairs is not None:
        x = x + F.embedding(pairs.rows(ids, prev), pairs.table).float()
    if turns is not None:
        x = x + ref.sinusoid(pos, turns, table.shape[1])
    return x if copies == 1 else torch.cat([x] * copies, -1)


def linear_parts(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x (M, K) @ w (N, K)^T as (splits, M, N): f32 partials of the split-K
    weight-stream kernel for up to 32 bf16 rows, else one part in x's type
    from the vendor GEMM."""
    if (x.is_cuda and x.dtype == torch.bfloat16 and x.shape[0] <= SKINNY_ROWS):
        return _ext().gemm_parts(x, w, 0)
    return F.linear(x, w).unsqueeze(0)


def linear_sums(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """linear_parts with 32-bit sums for any number of rows: for what takes the
    residual's place."""
    if x.is_cuda and x.dtype == torch.bfloat16 and x.shape[0] > SKINNY_ROWS:
        return torch.mm(x, w.t(), out_dtype=torch.float32).unsqueeze(0)
    return linear_parts(x, w)


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


def router_logits(h: torch.Tensor, w: torch.Tensor, n: int) -> torch.Tensor:
    """h (N, K) @ the first n rows of w (rows, K)^T in f32: (splits, N, >= n)."""
    if not h.is_cuda:
        return F.linear(h.float(), w[:n].float()).unsqueeze(0)
    if h.dtype == torch.bfloat16 and h.shape[0] > SKINNY_ROWS:
        return (linear_sums(h, w[:n]) if n > ROUTER_COLS
                else _ext().router_gemm(h, w[:n]))
    return linear_parts(h, w)      # f32 either way


def input_projection(h: torch.Tensor, w: torch.Tensor, spec,
                     ) -> Tuple[torch.Tensor, Optional[torch.Tensor], int]:
    """(parts, router parts, first router column in them). The router's columns
    spec.router_off .. + router_n, the last ones, are computed in f32."""
    r = spec.router_off
    if r < 0:
        return linear_parts(h, w), None, 0
    if not h.is_cuda or (h.dtype == torch.bfloat16 and h.shape[0] > SKINNY_ROWS):
        return (F.linear(h, w[:r]).unsqueeze(0),
                router_logits(h, w[r:], spec.router_n), 0)
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


@dataclass
class HeadSpec:
    """A q, k, v projection with biases and a norm per head, and the columns of
    its sections. temp_coef, temp_every: queries are multiplied by
    1 + coef * ln(floor((position + 1) / every) + 1)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    eps: float
    q_off: int = 0
    k_off: int = 0
    v_off: int = 0
    temp_coef: float = 0.0
    temp_every: float = 1.0
    router_off: int = -1


def head_post(parts: torch.Tensor, spec: HeadSpec, biases, q_norm: torch.Tensor,
              k_norm: torch.Tensor, batch, k_pages: torch.Tensor,
              v_pages: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """Normed queries (N, H, stored dim); keys and values go to the pages.
    biases: of q, k and v, each (columns,) f32 or None; q_norm, k_norm (dim,)."""
    s = spec
    _, N, _ = parts.shape
    H, G, D, V = s.heads, s.kv_heads, s.dim, s.vdim
    dkp = k_pages.shape[3]
    if parts.is_cuda:
        q = torch.empty(N, H, dkp, dtype=dtype, device=parts.device)
        _ext().head_post(
            parts, [s.q_off, s.k_off, s.v_off, H, G, D, V],
            [s.eps, s.temp_coef, s.temp_every], *biases, q_norm, k_norm, q,
            k_pages, v_pages, batch.page_table, batch.tok_seq, batch.tok_pos)
        return q
    y = parts.float().sum(0)

    def heads(off, n, d, bias):
        t = y[:, off:off + n * d]
        return (t if bias is None else t + bias).reshape(N, n, d)

    q = ref.grouped_rms_norm(heads(s.q_off, H, D, biases[0]), q_norm, 1, s.eps)
    q = q * ref.query_temperature(batch.tok_pos, s.temp_coef,
                                  s.temp_every).view(N, 1, 1)
    k = ref.grouped_rms_norm(heads(s.k_off, G, D, biases[1]), k_norm, 1, s.eps)
    v = heads(s.v_off, G, V, biases[2])
    P = k_pages.shape[2]
    live = (batch.tok_pos >= 0).nonzero()[:, 0]
    pos = batch.tok_pos[live].long()
    page = batch.page_table[batch.tok_seq[live].long(), pos // P].long()
    k_pages[page, :, pos % P, :D] = k[live].to(dtype)
    v_pages[page, :, :V, pos % P] = v[live].to(dtype)
    return F.pad(q, (0, dkp - D)).to(dtype)


@dataclass
class RopeSpec:
    """A q, k, v projection whose queries and keys turn: every head has `maps`
    queries (and keys) of dim elements, of each of which the first rot_dims are
    rotated, element i with element i + rot_dims / 2."""
    heads: int
    kv_heads: int
    maps: int
    dim: int
    vdim: int
    rot_dims: int
    q_off: int = 0
    k_off: int = 0
    v_off: int = 0
    amp: float = 1.0      # factor of cosine and sine

    @property
    def dk(self) -> int:
        """Stored size of one query or key."""
        return pad_head(self.dim)


def rope_post(parts: torch.Tensor, spec: RopeSpec, turns: torch.Tensor, batch,
              k_pages: torch.Tensor, v_pages: torch.Tensor,
              dtype: torch.dtype) -> torch.Tensor:
    """Rotated queries (N, H, maps, dk); keys, the maps of a head one after the
    other, and values go to the pages. turns (rot_dims / 2,) f64."""
    s = spec
    _, N, _ = parts.shape
    H, G, M, D, V = s.heads, s.kv_heads, s.maps, s.dim, s.vdim
    if parts.is_cuda:
        q = torch.empty(N, H, M, s.dk, dtype=dtype, device=parts.device)
        _ext().rope_post(
            parts, [s.q_off, s.k_off, s.v_off, H, G, M, D, V, s.rot_dims], s.amp,
            turns, q, k_pages, v_pages, batch.page_table, batch.tok_seq,
            batch.tok_pos)
        return q
    y = parts.float().sum(0)

    def heads(off, n):
        t = y[:, off:off + n * M * D].reshape(N, n, M, D)
        return F.pad(ref.rotate_half(t, batch.tok_pos, turns, s.amp),
                     (0, s.dk - D)).to(dtype)

    k = heads(s.k_off, G).view(N, G, M * s.dk)
    v = y[:, s.v_off:s.v_off + G * V].reshape(N, G, V).to(dtype)
    P = k_pages.shape[2]
    live = (batch.tok_pos >= 0).nonzero()[:, 0]
    pos = batch.tok_pos[live].long()
    page = batch.page_table[batch.tok_seq[live].long(), pos // P].long()
    k_pages[page, :, pos % P] = k[live]
    v_pages[page, :, :V, pos % P] = v[live]
    return heads(s.q_off, H)


@dataclass
class FfSpec:
    """A feed-forward's input projection: dense columns (one activation), then
    the router's, which start a 64-row block."""
    act: int = 0             # 0 none, 1 silu(gate) * up, 2 relu(up)^2
    ff: int = 0
    gate_off: int = -1
    up_off: int = -1
    cols: int = 0            # inner size of the output projection
    router_off: int = -1
    router_n: int = 0
    top: int = 0
    sigmoid: bool = False    # scores: sigmoid, else softmax
    renorm: bool = False     # the chosen weights sum to scale
    scale: float = 1.0


def ff_post(parts: Optional[torch.Tensor], rparts: Optional[torch.Tensor],
            r0: int, spec: FfSpec, correction: Optional[torch.Tensor], n: int,
            device, dtype: torch.dtype):
    """Activations (N, cols), zero beyond ff, and Routing or None."""
    s, E = spec, spec.router_n
    if parts is not None and parts.is_cuda or rparts is not None and rparts.is_cuda:
        out = torch.empty(n, s.cols, dtype=dtype, device=device)
        rt = None
        if E:
            rt = Routing(
                torch.empty(n, s.top, dtype=torch.int32, device=device),
                torch.empty(n, s.top, dtype=torch.float32, device=device), None)
        first = s.gate_off if s.act == 1 else s.up_off
        _ext().ff_post(
            parts if s.act else None, rparts if E else None,
            [s.act, first, s.up_off, s.ff, r0, E, 0, s.top, int(s.sigmoid),
             int(s.renorm)],
            s.scale, correction, out, rt.ids if rt else None,
            rt.wts if rt else None, None)
        return out, rt
    out = torch.zeros(n, s.cols, dtype=dtype)
    if s.act:
        y = parts.float().sum(0)
        u = y[:, s.up_off:s.up_off + s.ff]
        a = (F.silu(y[:, s.gate_off:s.gate_off + s.ff]) * u if s.act == 1
             else torch.relu(u) ** 2)
        out[:, :s.ff] = a.to(dtype)
    rt = None
    if E:
        ids, wts, _ = ref.route_topk(rparts.sum(0)[:, r0:r0 + E], correction, E,
                                     s.top, s.scale, s.sigmoid, s.renorm)
        rt = Routing(ids, wts, None)
    return out, rt


def route(h: torch.Tensor, w: torch.Tensor, spec: FfSpec) -> Routing:
    """Experts of feed-forwards without dense columns: w (rows, K), the router's
    rows first."""
    return ff_post(None, router_logits(h, w, spec.router_n), 0, spec, None,
                   h.shape[0], h.device, h.dtype)[1]


@dataclass
class GluSpec:
    """Activation of gated experts: g sigmoid(slope g) (u + shift) with
    g = min(gate, limit) and u = clamp(up, -limit, limit). silu(gate) * up as it
    stands."""
    limit: float = float("inf")
    slope: float = 1.0
    shift: float = 0.0


SILU = GluSpec()


def moe_experts(h: torch.Tensor, up: torch.Tensor, down: torch.Tensor,
                rt: Routing, weight_input: bool = False,
                act: GluSpec = SILU) -> torch.Tensor:
    """(N, top, W) weighted outputs of the chosen experts; the rows of
    identity choices are not defined. up (E, 2, F, K): the gated activation act,
    or (E, 1, F, K): relu(up)^2; down (E, W, F); K, F and W padded to 64. The
    weight multiplies an expert's output, or its input."""
    consts = (act.limit, act.slope, act.shift)
    if h.is_cuda:
        return _ext().moe_experts(h, up, down, rt.ids, rt.wts, weight_input,
                                  *consts)
    return ref.moe_experts(h, up, down, rt.ids, rt.wts, weight_input, *consts)


def attn_ragged(q: torch.Tensor, k_pages: torch.Tensor,
                v_pages: Optional[torch.Tensor],
                batch, out: torch.Tensor, dim: int, vdim: int, scale: float,
                window: int = 0, slopes: Optional[torch.Tensor] = None,
                gate: Optional[torch.Tensor] = None,
                sinks: Optional[torch.Tensor] = None,
                table: Optional[torch.Tensor] = None,
                portions_only: bool = False, chunk: int = 0) -> None:
    """Attention of a ragged batch into out[:, :H*vdim] (see
    reference.attn_ragged): a window of the last keys, or a chunk of the positions
    counted from the sequence's start (0 = none). Without v_pages the values are the first vdim
    elements of the keys. table: page table of pages that are not the
    cache's; portions_only leaves the rows of single tokens alone (where the
    sizes are those of the tiled kernels)."""
    table = batch.page_table if table is None else table
    if q.is_cuda:
        dec = batch.dec_list[:0] if portions_only else batch.dec_list
        _ext().attn_ragged(
            q, k_pages, v_pages, table, batch.tok_seq, batch.tok_pos, batch.cu,
            batch.q_start, batch.pre_list, dec, batch.max_new, batch.max_ctx,
            dim, vdim, scale, window, chunk, slopes, sinks, gate, out)
        return
    n = q.shape[1] * vdim
    out[:, :n] = ref.attn_ragged(q, k_pages, v_pages, batch, dim, vdim, scale,
                                 window, slopes, gate, sinks, chunk)
