"""Token mixers over ragged batches beside plain attention (ops/ragged.py):
latent attention, differential attention, gated linear attention, and gated linear
attention whose forget gate also decides what is written.

They take the output of a layer's fused input GEMM (parts, as linear_parts
returns it) and give the mixer output, the input of the layer's output GEMM.
Single tokens and portions of prompts of one step take different kernels and fill
different rows of one result.

Device tensors run the _hip_mixers, _hip_differential, _hip_hgrn and _hip_ragged
extensions and fail loudly without them; CPU tensors run the forms in
ops/reference.py.
"""
from __future__ import annotations

import importlib
import math
from dataclasses import dataclass
from typing import Optional, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.ops import ragged
from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.ragged import RopeSpec, pad_head, round_up

_loaded = {}   # extension modules, by the first device call of each


def _ext(name: str = "_hip_mixers"):
    if name not in _loaded:
        try:
            _loaded[name] = importlib.import_module(f"bloombee_amd.ops.{name}")
        except ImportError as e:
            raise RuntimeError(
                f"the {name} extension is not built but a tensor is on "
                "GPU. Run `python setup.py hip` (PYTORCH_ROCM_ARCH=gfx950). "
                f"Import error was: {e}") from e
    return _loaded[name]


def _mixed(out_cols: int, used: int, n: int, dtype, device) -> torch.Tensor:
    """Result of a mixer: kernels write `used` columns, the rest is zero."""
    make = torch.empty if out_cols == used else torch.zeros
    return make(n, out_cols, dtype=dtype, device=device)


# ---------------------------------------------------------------------------
# rotations
# ---------------------------------------------------------------------------

def _frequencies(base: float, dims: int) -> torch.Tensor:
    i = torch.arange(dims // 2, dtype=torch.float64)
    return torch.pow(torch.tensor(base, dtype=torch.float64), -2.0 * i / dims)


def rotary_turns(base: float, dims: int) -> torch.Tensor:
    """Frequencies base^(-2 i / dims) over 2 pi, float64: turns per position."""
    return _frequencies(base, dims) / (2 * torch.pi)


def banded_turns(base: float, dims: int, factor: float, low: float, high: float,
                 original: float) -> torch.Tensor:
    """rotary_turns stretched by wavelength (reference.banded_frequencies)."""
    return ref.banded_frequencies(_frequencies(base, dims), factor, low, high,
                                  original) / (2 * torch.pi)


def yarn_turns(base: float, dims: int, factor: float, original: float,
               fast: float, slow: float) -> Tuple[torch.Tensor, float]:
    """rotary_turns stretched pair by pair (YaRN): pairs that turn more than
    `fast` times over the original context keep their frequency, those that turn
    less than `slow` times have it divided by factor, a linear ramp between. Also
    the factor of cosine and sine that goes with it."""
    def pair(turns: float) -> float:
        return (dims * math.log(original / (2 * math.pi * turns))
                / (2 * math.log(base)))

    lo = max(math.floor(pair(fast)), 0)
    hi = min(math.ceil(pair(slow)), dims - 1)
    f = _frequencies(base, dims)
    i = torch.arange(dims // 2, dtype=torch.float64)
    ramp = ((i - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    f = f / factor * ramp + f * (1 - ramp)
    return f / (2 * torch.pi), 0.1 * math.log(factor) + 1


def half_order(dims: int, size: int) -> torch.Tensor:
    """The kernels turn element i with element i + dims / 2. Rows of a projection
    whose elements 2 i and 2 i + 1 turn together, taken in this order, do the same
    as they are: a score does not notice an order that queries and keys share."""
    i = torch.arange(size)
    return torch.cat([i[0:dims:2], i[1:dims:2], i[dims:]])


# ---------------------------------------------------------------------------
# latent attention
# ---------------------------------------------------------------------------

# latent and rotated sizes the decode kernel is compiled for
LATENT_SIZES = (64, 128, 256, 512)
ROTATED_SIZES = (32, 64, 128)


def _stored(n: int, sizes) -> int:
    for s in sizes:
        if n <= s:
            return s
    return round_up(n, 32)


def pad_key(d: int) -> int:
    """Stored size of a per-head key of d elements in the prompt kernel."""
    return 192 if 128 < d <= 192 else pad_head(d)


@dataclass
class LatentSpec:
    """Sizes of a latent attention layer and where the sections of its input
    projection lie (columns; -1 = absent: the layer reads another's latents)."""
    heads: int
    dim: int            # unrotated query/key elements of a head
    rot: int            # rotated part, shared by the heads on the key side
    rot_dims: int       # elements of it that turn
    vdim: int
    q_rank: int
    rank: int
    scale: float
    window: int         # 0 = none
    eps: float
    q_off: int = 0
    c_off: int = -1
    g_off: int = 0
    out_cols: int = 0   # inner size of the output projection
    q_cols: int = 0     # inner size of the query projection
    amp: float = 1.0    # factor of cosine and sine

    @property
    def has_kv(self) -> bool:
        return self.c_off >= 0

    @property
    def rp(self) -> int:
        """Stored size of a latent."""
        return _stored(self.rank, LATENT_SIZES)

    @property
    def ck(self) -> int:
        """Stored size of a key, [latent | rotated part]."""
        return self.rp + _stored(self.rot, ROTATED_SIZES)

    @property
    def tiled(self) -> bool:
        """The MFMA kernels take these sizes."""
        return (self.rank <= LATENT_SIZES[-1] and self.rot <= ROTATED_SIZES[-1]
                and self.dim + self.rot <= 256 and self.vdim <= 256)


@dataclass
class LatentWeights:
    uk: torch.Tensor      # (H, rp, dim padded to 32): W_uk transposed
    uv: torch.Tensor      # (H, vdim padded to 64, rp)
    ukv: torch.Tensor     # (H * dim + H * vdim padded, ck): [W_uk | W_uv]
    sink: Optional[torch.Tensor]


def latent_post(parts: torch.Tensor, spec: LatentSpec, q_norm: torch.Tensor,
                c_norm: Optional[torch.Tensor], turns: torch.Tensor, batch,
                pages: torch.Tensor, dtype: torch.dtype,
                ) -> Tuple[torch.Tensor, torch.Tensor]:
    """Norms the query latent; norms c, rotates the shared key part and writes
    both to the page slots. Returns (query latent (N, q_cols), gate)."""
    _, N, _ = parts.shape
    s, dev = spec, parts.device
    gn = s.heads * s.vdim
    if parts.is_cuda:
        cq = torch.empty(N, s.q_cols, dtype=dtype, device=dev)
        in_place = parts.shape[0] == 1 and parts.dtype == dtype
        gate = (parts[0][:, s.g_off:s.g_off + gn] if in_place
                else torch.empty(N, gn, dtype=dtype, device=dev))
        _ext().latent_post(
            parts, [s.q_off, s.c_off, s.g_off, s.q_rank, s.rank, s.rot,
                    s.rot_dims, s.rp, gn, int(s.has_kv)], s.eps, s.amp, q_norm,
            c_norm, turns, cq, None if in_place else gate, pages,
            batch.page_table, batch.tok_seq, batch.tok_pos)
        return cq, gate
    y = parts.float().sum(0)
    cq = ref.grouped_rms_norm(y[:, s.q_off:s.q_off + s.q_rank], q_norm, 1, s.eps)
    if s.has_kv:
        c = ref.grouped_rms_norm(y[:, s.c_off:s.c_off + s.rank], c_norm, 1, s.eps)
        at = s.c_off + s.rank
        r = ref.rotate_half(y[:, at:at + s.rot], batch.tok_pos, turns, s.amp)
        P = pages.shape[2]
        live = (batch.tok_pos >= 0).nonzero()[:, 0]
        pos = batch.tok_pos[live].long()
        page = batch.page_table[batch.tok_seq[live].long(), pos // P].long()
        pages[page, 0, pos % P, :s.rank] = c[live].to(dtype)
        pages[page, 0, pos % P, s.rp:s.rp + s.rot] = r[live].to(dtype)
    return (F.pad(cq.to(dtype), (0, s.q_cols - s.q_rank)),
            y[:, s.g_off:s.g_off + gn].to(dtype))


def _absorbed(parts: torch.Tensor, spec: LatentSpec, w: LatentWeights,
              turns: torch.Tensor, batch, gate, pages, dtype) -> torch.Tensor:
    """Every row in the latent space, plain attention kernel: 32-bit runs and
    sizes beyond the tiles."""
    s = spec
    N, H = parts.shape[1], s.heads
    if parts.is_cuda:
        q = torch.empty(N, H, s.dim + s.rot, dtype=dtype, device=parts.device)
        _ext().latent_rope(parts, turns, batch.tok_pos, s.dim, s.rot,
                           s.rot_dims, s.amp, q)
    else:
        y = parts.float().sum(0)[:, :H * (s.dim + s.rot)].view(N, H, -1)
        q = torch.cat([y[..., :s.dim], ref.rotate_half(
            y[..., s.dim:], batch.tok_pos, turns, s.amp)], -1).to(dtype)
    qn = q[..., :s.dim].transpose(0, 1).contiguous()
    lat = torch.bmm(qn, w.uk[:, :, :s.dim].transpose(1, 2).contiguous())
    ql = torch.zeros(N, H, s.ck, dtype=dtype, device=q.device)
    ql[..., :s.rp] = lat.transpose(0, 1)
    ql[..., s.rp:s.rp + s.rot] = q[..., s.dim:]
    o = torch.empty(N, H * s.rp, dtype=dtype, device=q.device)
    ragged.attn_ragged(ql, pages, None, batch, o, s.ck, s.rp, s.scale, s.window,
                       sinks=w.sink)
    ol = o.view(N, H, s.rp).transpose(0, 1).contiguous()
    v = torch.bmm(ol, w.uv.transpose(1, 2).contiguous())[..., :s.vdim]
    v = v.transpose(0, 1).reshape(N, H * s.vdim)
    out = _mixed(s.out_cols, H * s.vdim, N, dtype, q.device)
    out[:, :H * s.vdim] = v * torch.sigmoid(gate.float()).to(v.dtype)
    return out


def latent_attention(parts: torch.Tensor, spec: LatentSpec, w: LatentWeights,
                     turns: torch.Tensor, batch, gate: torch.Tensor,
                     pages: torch.Tensor, dtype: torch.dtype) -> torch.Tensor:
    """Gated attention output (N, out_cols) from the query GEMM's parts.

    Single tokens meet the cached latents themselves (their queries are taken
    into the latent space). Portions of prompts meet per-head keys and values,
    which one GEMM makes from the latents their window sees."""
    s = spec
    if not (parts.is_cuda and dtype == torch.bfloat16 and s.tiled):
        return _absorbed(parts, s, w, turns, batch, gate, pages, dtype)
    N, H = parts.shape[1], s.heads
    out = _mixed(s.out_cols, H * s.vdim, N, dtype, parts.device)
    if batch.dec_list.numel():
        _ext().latent_decode(
            parts, turns, pages, batch.page_table, batch.tok_pos, batch.cu,
            batch.q_start, batch.dec_list, batch.max_ctx, s.dim, s.rot, s.rot_dims,
            s.amp, s.vdim, s.scale, s.window, w.uk, w.uv, w.sink, gate, out)
    if batch.pre_list.numel():
        ctx = batch.context(s.window)
        n, P = ctx.pages.numel(), pages.shape[2]
        lat = pages.view(pages.shape[0], P, s.ck).index_select(0, ctx.pages)
        kv = F.linear(lat.view(n * P, s.ck), w.ukv)
        dk, dv = pad_key(s.dim + s.rot), pad_head(s.vdim)
        k = torch.empty(n, H, P, dk, dtype=dtype, device=out.device)
        v = torch.empty(n, H, dv, P, dtype=dtype, device=out.device)
        _ext().latent_scatter(kv, lat, ctx.valid, s.dim, s.rot, s.vdim, s.rp,
                              k, v)
        q = torch.empty(N, H, dk, dtype=dtype, device=out.device)
        _ext().latent_rope(parts, turns, batch.tok_pos, s.dim, s.rot,
                           s.rot_dims, s.amp, q)
        ragged.attn_ragged(q, k, v, batch, out, s.dim + s.rot, s.vdim, s.scale,
                           s.window, gate=gate, sinks=w.sink, table=ctx.table,
                           portions_only=True)
    return out


# ---------------------------------------------------------------------------
# differential attention
# ---------------------------------------------------------------------------

@dataclass
class DiffSpec:
    """Two attentions per head over the same values and how they combine:
    rms(a1 - lam a2) factor, the norm over the head's values and without a
    weight. A key's two maps lie one after the other in its page slot."""
    rope: RopeSpec
    scale: float
    lam: float
    factor: float
    eps: float
    window: int = 0       # 0 = none
    chunk: int = 0
    out_cols: int = 0     # inner size of the output projection


def differential_attention(parts: torch.Tensor, spec: DiffSpec,
                           turns: torch.Tensor, batch, k_pages: torch.Tensor,
                           v_pages: torch.Tensor,
                           dtype: torch.dtype) -> torch.Tensor:
    """(N, out_cols) from the input GEMM's parts; keys and values go to the
    pages."""
    s, r = spec, spec.rope
    N = parts.shape[1]
    q = ragged.rope_post(parts, r, turns, batch, k_pages, v_pages, dtype)
    used = r.heads * r.vdim
    out = _mixed(s.out_cols, used, N, dtype, parts.device)
    if parts.is_cuda:
        _ext("_hip_differential").attn_differential(
            q, k_pages, v_pages, batch.page_table, batch.tok_seq, batch.tok_pos,
            batch.cu, batch.q_start, batch.pre_list, batch.dec_list, batch.max_new,
            batch.max_ctx, r.dim, r.vdim, s.scale, s.window, s.chunk, s.lam,
            s.factor, s.eps, out)
        return out
    out[:, :used] = ref.attn_differential(q, k_pages, v_pages, batch, r.dim,
                                          r.vdim, s.scale, s.lam, s.factor, s.eps,
                                          s.window, s.chunk)
    return out


# ---------------------------------------------------------------------------
# gated linear attention
# ---------------------------------------------------------------------------

@dataclass
class GlaSpec:
    """Sizes of a gated linear attention layer and the columns of its input
    projection. The decay section (the first, low-rank factor's output) is
    last and computed in f32 (input_projection's router section)."""
    heads: int
    dim: int
    vdim: int
    tau: float
    eps: float
    q_off: int = 0
    k_off: int = 0
    v_off: int = 0
    g_off: int = 0
    router_off: int = -1
    router_n: int = 0     # rank of the decay projection
    out_cols: int = 0


def gla_mix(parts: torch.Tensor, aparts: torch.Tensor, a0: int, spec: GlaSpec,
            a2: torch.Tensor, a2_b: torch.Tensor, norm: torch.Tensor,
            state: torch.Tensor, batch, dtype: torch.dtype) -> torch.Tensor:
    """Gated linear attention of a step, states updated in place: (N,
    out_cols). aparts (splits, N, >= a0 + rank) f32: decay projection from
    column a0 on; a2 (rank, H * dim), state (slots, H, dim, vdim)."""
    s = spec
    N, H = parts.shape[1], s.heads
    out = _mixed(s.out_cols, H * s.vdim, N, dtype, parts.device)
    dims = [s.q_off, s.k_off, s.v_off, s.g_off, a0, H, s.dim, s.vdim]
    consts = [s.dim ** -0.5, 1.0 / s.tau, s.eps]
    if parts.is_cuda:
        steps = [batch.dec_list]
        if batch.pre_list.numel():
            C = (_ext().gla_chunk(s.dim, s.vdim, a2.shape[0])
                 if dtype == torch.bfloat16 else 0)
            if C:
                ch = batch.chunks(C)
                y = (parts[0] if parts.shape[0] == 1 and parts.dtype == dtype
                     else parts.sum(0).to(dtype))
                a1 = aparts[0] if aparts.shape[0] == 1 else aparts.sum(0)
                _ext().gla_chunks(y, a1, dims, consts, a2, a2_b, norm, state,
                                  batch.slots, batch.q_start, batch.pre_list,
                                  ch.row0, ch.len, ch.cu, out)
            else:
                steps.append(batch.pre_list)
        for seqs in steps:
            if seqs.numel():
                _ext().gla_step(parts, aparts, dims, consts, a2, a2_b, norm,
                                state, batch.slots, batch.tok_pos, batch.cu,
                                seqs, out)
        return out
    y = parts.float().sum(0)
    cut = lambda off, d: y[:, off:off + H * d].reshape(N, H, d)
    q, k, v = cut(s.q_off, s.dim) * consts[0], cut(s.k_off, s.dim), \
        cut(s.v_off, s.vdim)
    r = a2.shape[0]
    alpha = ref.channel_decays(aparts.sum(0)[:, a0:a0 + r], a2, a2_b,
                               s.tau).view(N, H, s.dim)
    o = _scan_sequences(q, k, v, alpha, state, batch)
    o = ref.grouped_rms_norm(o, norm, 1, s.eps).reshape(N, H * s.vdim)
    g = y[:, s.g_off:s.g_off + H * s.vdim]
    out[:, :H * s.vdim] = (o * F.silu(g)).to(dtype)
    return out


def _scan_sequences(q, k, v, alpha, state, batch) -> torch.Tensor:
    """reference.gla_scan of every sequence of a step, states in place."""
    o = torch.zeros(*q.shape[:2], v.shape[-1])
    for i, (a, b) in enumerate(zip(batch.cu[:-1].tolist(), batch.cu[1:].tolist())):
        if int(batch.tok_pos[a]) < 0:
            continue
        slot = int(batch.slots[i])
        S = state[slot] if int(batch.q_start[i]) > 0 else \
            torch.zeros_like(state[slot])
        o[a:b], state[slot] = ref.gla_scan(q[a:b], k[a:b], v[a:b], alpha[a:b], S)
    return o


# ---------------------------------------------------------------------------
# gated linear attention that writes what it forgets (HGRN2)
# ---------------------------------------------------------------------------

@dataclass
class HgrnSpec:
    """Sizes of the layer and the columns of its input projection. The forget
    gate's logits are last and computed in f32 (input_projection's router
    section)."""
    heads: int
    dim: int
    vdim: int
    eps: float
    q_off: int = 0
    v_off: int = 0
    router_off: int = -1
    router_n: int = 0     # heads * dim
    out_cols: int = 0


def hgrn_mix(parts: torch.Tensor, fparts: torch.Tensor, f0: int, spec: HgrnSpec,
             f_b: torch.Tensor, lower: torch.Tensor, norm: torch.Tensor,
             state: torch.Tensor, batch, dtype: torch.dtype) -> torch.Tensor:
    """(N, out_cols) of a step, states updated in place. Per head
    S <- diag(f) S + (1 - f) v^T, o = S^T silu(q), normed over vdim, with
    f = lower + (1 - lower) sigmoid(z + f_b). fparts (splits, N, >= f0 + heads *
    dim) f32: z from column f0 on; f_b, lower (heads * dim,) f32."""
    s = spec
    N, H, n = parts.shape[1], s.heads, s.heads * s.dim
    out = _mixed(s.out_cols, H * s.vdim, N, dtype, parts.device)
    dims = [s.q_off, s.v_off, f0, H, s.dim, s.vdim]
    if parts.is_cuda:
        ext = _ext("_hip_hgrn")
        steps = [batch.dec_list]
        if batch.pre_list.numel():
            C = ext.hgrn_chunk(s.dim, s.vdim) if dtype == torch.bfloat16 else 0
            if C:
                ch = batch.chunks(C)
                y = (parts[0] if parts.shape[0] == 1 and parts.dtype == dtype
                     else parts.sum(0).to(dtype))
                z = fparts[0] if fparts.shape[0] == 1 else fparts.sum(0)
                ext.hgrn_chunks(y, z, dims, s.eps, f_b, lower, norm, state,
                                batch.slots, batch.q_start, batch.pre_list,
                                ch.row0, ch.len, ch.cu, out)
            else:
                steps.append(batch.pre_list)
        for seqs in steps:
            if seqs.numel():
                ext.hgrn_step(parts, fparts, dims, s.eps, f_b, lower, norm,
                              state, batch.slots, batch.tok_pos, batch.cu, seqs,
                              out)
        return out
    y = parts.float().sum(0)
    f, k = ref.forget_gates(fparts.sum(0)[:, f0:f0 + n], f_b, lower)
    head = lambda t: t.reshape(N, H, -1)
    o = _scan_sequences(head(F.silu(y[:, s.q_off:s.q_off + n])), head(k),
                        head(y[:, s.v_off:s.v_off + H * s.vdim]), head(f), state,
                        batch)
    o = ref.grouped_rms_norm(o, norm, 1, s.eps)
    out[:, :H * s.vdim] = o.reshape(N, H * s.vdim).to(dtype)
    return out
