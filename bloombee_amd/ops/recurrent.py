"""Recurrent token mixers over ragged batches whose gates are scalars or
channels: the matrix memory with exponential gates (mLSTM) and the gated linear
recurrent unit with its short convolution (RG-LRU).

Both take the output of a layer's fused input GEMM (parts, as linear_parts
returns it) and give the gated mixer output, the input of the layer's output
GEMM; states are updated in place. Single tokens and portions of prompts of one
step take different kernels and fill different rows of one result.

Device tensors run the _hip_recurrent extension and fail loudly without it; CPU
tensors run the forms in ops/reference.py.
"""
from __future__ import annotations

import importlib
from dataclasses import dataclass
from typing import Dict

import torch
import torch.nn.functional as F

from bloombee_amd.ops import reference as ref
from bloombee_amd.ops.mixers import _mixed

_hip_recurrent = None   # loaded by the first device call


def _ext():
    global _hip_recurrent
    if _hip_recurrent is None:
        try:
            _hip_recurrent = importlib.import_module(
                "bloombee_amd.ops._hip_recurrent")
        except ImportError as e:
            raise RuntimeError(
                "the _hip_recurrent extension is not built but a tensor is on "
                "GPU. Run `python setup.py hip` (PYTORCH_ROCM_ARCH=gfx950). "
                f"Import error was: {e}") from e
    return _hip_recurrent


def _portions(batch):
    """(sequence, first row, end row, continues) of every sequence that is not
    an empty slot; host loop of the CPU forms."""
    cu = batch.cu.tolist()
    for i, (a, b) in enumerate(zip(cu[:-1], cu[1:])):
        if int(batch.tok_pos[a]) >= 0:
            yield i, a, b, int(batch.q_start[i]) > 0


# ---------------------------------------------------------------------------
# matrix memory
# ---------------------------------------------------------------------------

@dataclass
class MlstmSpec:
    """Sizes of a matrix memory layer and the columns of its input projection.
    The gate section (input gates, then forget gates) is last and computed in
    f32 (input_projection's router section)."""
    heads: int
    dim: int
    vdim: int
    cap: float          # of the gates' logits
    eps: float
    q_off: int = 0
    k_off: int = 0
    v_off: int = 0
    g_off: int = 0
    router_off: int = -1
    router_n: int = 0   # 2 * heads
    out_cols: int = 0

    def state_shapes(self) -> Dict[str, tuple]:
        H, D, V = self.heads, self.dim, self.vdim
        return {"S": (H, D, V), "n": (H, D), "m": (H,)}


def mlstm_mix(parts: torch.Tensor, gparts: torch.Tensor, i0: int,
              spec: MlstmSpec, gate_b: torch.Tensor, norm: torch.Tensor,
              state: Dict[str, torch.Tensor], batch,
              dtype: torch.dtype) -> torch.Tensor:
    """Matrix memory of a step: (N, out_cols). gparts (splits, N, >= i0 + 2 H)
    f32: gate logits from column i0 on; gate_b (2 H,), norm (H * vdim,)."""
    s = spec
    N, H = parts.shape[1], s.heads
    out = _mixed(s.out_cols, H * s.vdim, N, dtype, parts.device)
    dims = [s.q_off, s.k_off, s.v_off, s.g_off, i0, H, s.dim, s.vdim]
    consts = [s.dim ** -0.5, s.cap, s.eps]
    st = (state["S"], state["n"], state["m"])
    if parts.is_cuda:
        steps = [batch.dec_list]
        if batch.pre_list.numel():
            C = (_ext().mlstm_chunk(s.dim, s.vdim)
                 if dtype == torch.bfloat16 else 0)
            if C:
                ch = batch.chunks(C)
                y = (parts[0] if parts.shape[0] == 1 and parts.dtype == dtype
                     else parts.sum(0).to(dtype))
                g = gparts[0] if gparts.shape[0] == 1 else gparts.sum(0)
                _ext().mlstm_chunks(
                    y, g, dims, consts, gate_b, norm, *st,
                    st[2].index_select(0, batch.slots), batch.slots,
                    batch.q_start, batch.pre_list, ch.row0, ch.len, ch.cu, out)
            else:
                steps.append(batch.pre_list)
        for seqs in steps:
            if seqs.numel():
                _ext().mlstm_step(parts, gparts, dims, consts, gate_b, norm,
                                  *st, batch.slots, batch.tok_pos, batch.cu,
                                  seqs, out)
        return out
    y = parts.float().sum(0)
    cut = lambda off, d: y[:, off:off + H * d].reshape(N, H, d)
    q, k, v = cut(s.q_off, s.dim) * consts[0], cut(s.k_off, s.dim), \
        cut(s.v_off, s.vdim)
    i, f = ref.mlstm_gates(gparts.sum(0)[:, i0:i0 + 2 * H], gate_b, s.cap)
    o = torch.zeros(N, H, s.vdim)
    for n, a, b, goes_on in _portions(batch):
        slot = int(batch.slots[n])
        old = [t[slot] if goes_on else torch.zeros_like(t[slot]) for t in st]
        o[a:b], new = ref.mlstm_scan(q[a:b], k[a:b], v[a:b], i[a:b], f[a:b], *old)
        for t, x in zip(st, new):
            t[slot] = x
    o = ref.grouped_rms_norm(o, torch.ones(s.vdim), 1, s.eps)
    o = o.reshape(N, H * s.vdim) * norm
    g = y[:, s.g_off:s.g_off + H * s.vdim]
    out[:, :H * s.vdim] = (o * torch.sigmoid(g)).to(dtype)
    return out


# ---------------------------------------------------------------------------
# gated linear recurrent unit
# ---------------------------------------------------------------------------

@dataclass
class RglruSpec:
    """Sizes of a gated linear recurrent unit and the columns of its input
    projection."""
    width: int
    blocks: int         # of the gates' block-diagonal products
    taps: int           # of the convolution
    y_off: int = 0
    x_off: int = 0
    out_cols: int = 0
    router_off: int = -1

    @property
    def block(self) -> int:
        return self.width // self.blocks

    @property
    def block_p(self) -> int:
        """Stored size of a block."""
        return (self.block + 63) // 64 * 64

    def state_shapes(self) -> Dict[str, tuple]:
        return {"S": (self.width,), "conv": (self.taps - 1, self.width)}


@dataclass
class RglruWeights:
    y_b: torch.Tensor       # (W,) f32, as all but gates
    x_b: torch.Tensor
    taps: torch.Tensor      # (K, W), the current token's last
    conv_b: torch.Tensor
    gates: torch.Tensor     # (B, 2, block_p, block_p) [out, in] of r and i
    gates_b: torch.Tensor   # (2, W)
    decay: torch.Tensor     # (W,): log a = decay * r


def rglru_mix(parts: torch.Tensor, spec: RglruSpec, w: RglruWeights,
              state: Dict[str, torch.Tensor], batch,
              dtype: torch.dtype) -> torch.Tensor:
    """Gated linear recurrent unit of a step: (N, out_cols)."""
    s = spec
    N, W, B, D = parts.shape[1], s.width, s.blocks, s.block
    out = _mixed(s.out_cols, W, N, dtype, parts.device)
    if parts.is_cuda:
        make = torch.empty if s.block_p == D else torch.zeros
        u = make(N, B * s.block_p, dtype=dtype, device=parts.device)
        common = (parts, [s.y_off, s.x_off, W, s.taps, B, s.block_p],
                  [w.y_b, w.x_b, w.taps, w.conv_b, w.gates_b, w.decay],
                  state["S"], state["conv"], u, batch.slots, batch.tok_seq,
                  batch.tok_pos, batch.q_start, batch.cu)
        _ext().rglru_conv(*common)
        if dtype != torch.bfloat16:
            ub = u.view(N, B, s.block_p)[..., :D].transpose(0, 1).contiguous()
            gw = w.gates[:, :, :D, :D].reshape(B, 2 * D, D)
            z = torch.bmm(ub, gw.transpose(1, 2).contiguous())
            for seqs in (batch.dec_list, batch.pre_list):
                _ext().rglru_seq(*common, z, seqs, out)
            return out
        if batch.dec_list.numel():
            _ext().rglru_step(*common, w.gates, batch.dec_list, out)
        if batch.pre_list.numel():
            ch = batch.chunks(_ext().rglru_chunk())
            _ext().rglru_chunks(*common, w.gates, batch.pre_list, ch.row0,
                                ch.len, ch.cu, out)
        return out
    y = parts.float().sum(0)
    x = y[:, s.x_off:s.x_off + W] + w.x_b
    branch = ref.gelu_tanh(y[:, s.y_off:s.y_off + W] + w.y_b)
    for n, a, b, goes_on in _portions(batch):
        slot = int(batch.slots[n])
        past, S = state["conv"][slot], state["S"][slot]
        if goes_on:
            # entries ahead of the sequence's start are not its own
            past = past.clone()
            past[:max(0, s.taps - 1 - int(batch.q_start[n]))] = 0
        else:
            past, S = torch.zeros_like(past), torch.zeros_like(S)
        u = ref.causal_conv(x[a:b], past, w.taps, w.conv_b).to(dtype)
        states, last = ref.rglru_scan(
            *ref.rglru_inputs(u, w.gates[:, :, :D, :D], w.gates_b, w.decay), S)
        state["S"][slot] = last
        state["conv"][slot] = torch.cat([past, x[a:b]])[b - a:]
        out[a:b, :W] = (states * branch[a:b]).to(dtype)
    return out
