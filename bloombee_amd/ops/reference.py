"""Pure-PyTorch fp32 reference implementations of every hot op.

These serve two purposes:
  1. CPU execution path (this container has no GPU; the loopback swarm tests
     and the bloom-560m plumbing config run on CPU).
  2. Numerics golden references for the HIP kernels (tests compare the gfx950
     kernels against these in fp32, mirroring the reference's parity suite,
     e.g. test_mha_gen_llama_decode_parity.py).

Functional parity targets in the reference (ai-decentralized/BloomBee):
  rms_norm           <- flexgen_utils/pytorch_backend.py:111-120
  rope               <- flexgen_utils/pytorch_backend.py:59-110
  attention          <- pytorch_backend.py:665-916 (mha_llama / mha_gen_llama)
  swiglu (mlp core)  <- pytorch_backend.py:1033-1048 (mlp_llama)
  paged KV           <- server/paged_kv.py
  4-bit group quant  <- flexgen_utils/compression.py:94-210

The layouts here are the MI355X-native ones (NOT the reference's):
  hidden      (B, T, H)            bf16
  q           (B, Hq, Tq, D)
  k/v (new)   (B, Hkv, T, D)
  KV pages    (n_pages, Hkv, page_size, D)   -- 4 KB contiguous per
              (page, head) slab at D=128/bf16: one coalesced burst per wave.
  page_table  (B, max_pages_per_seq) int32
"""
from __future__ import annotations

import math
from typing import Optional, Tuple

import torch
import torch.nn.functional as F


# ---------------------------------------------------------------------------
# Normalization
# ---------------------------------------------------------------------------

def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    """RMSNorm with fp32 variance accumulation (ref pytorch_backend.py:111-120)."""
    xf = x.float()
    var = xf.pow(2).mean(dim=-1, keepdim=True)
    y = xf * torch.rsqrt(var + eps)
    return (y * weight.float()).to(x.dtype)


def rms_norm_residual(
    x: torch.Tensor, residual: torch.Tensor, weight: torch.Tensor, eps: float = 1e-5
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Fused residual-add + RMSNorm: h = x + residual; y = rmsnorm(h).

    The fusion target: on MI355X the elementwise add would otherwise be a
    separate HBM round trip (fuse elementwise work into the
    producing kernel).
    """
    h = (x.float() + residual.float()).to(x.dtype)
    return h, rms_norm(h, weight, eps)


def layer_norm(
    x: torch.Tensor, weight: torch.Tensor, bias: Optional[torch.Tensor], eps: float = 1e-5
) -> torch.Tensor:
    """LayerNorm for bloom/falcon-family blocks (ref pytorch_backend.py mha/mlp)."""
    xf = x.float()
    mu = xf.mean(dim=-1, keepdim=True)
    var = (xf - mu).pow(2).mean(dim=-1, keepdim=True)
    y = (xf - mu) * torch.rsqrt(var + eps)
    y = y * weight.float()
    if bias is not None:
        y = y + bias.float()
    return y.to(x.dtype)


# ---------------------------------------------------------------------------
# RoPE
# ---------------------------------------------------------------------------

def banded_frequencies(inv_freq: torch.Tensor, factor: float, low: float,
                       high: float, original: float) -> torch.Tensor:
    """Rotary frequencies stretched to longer contexts by wavelength (llama-3
    style): kept where the wavelength is below original / high, divided by factor
    where it is above original / low, blended between."""
    wavelen = 2 * math.pi / inv_freq
    smooth = (original / wavelen - low) / (high - low)
    out = (1 - smooth) * inv_freq / factor + smooth * inv_freq
    out = torch.where(wavelen > original / low, inv_freq / factor, out)
    return torch.where(wavelen < original / high, inv_freq, out)


def rope_cos_sin(
    head_dim: int, max_pos: int, theta: float = 10000.0, device=None, dtype=torch.float32,
    scaling: Optional[dict] = None,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Host-precomputed RoPE tables (guide Appendix B: precompute trig on host).

    Returns cos, sin of shape (max_pos, head_dim // 2), fp32.
    Supports llama-3 style rope scaling when ``scaling`` carries
    {factor, low_freq_factor, high_freq_factor, original_max_position_embeddings}.
    """
    inv_freq = 1.0 / (theta ** (torch.arange(0, head_dim, 2, dtype=torch.float64) / head_dim))
    if scaling is not None and scaling.get("rope_type", scaling.get("type")) == "llama3":
        inv_freq = banded_frequencies(
            inv_freq, scaling["factor"], scaling["low_freq_factor"],
            scaling["high_freq_factor"],
            scaling["original_max_position_embeddings"])
    t = torch.arange(max_pos, dtype=torch.float64)
    freqs = torch.outer(t, inv_freq)
    cos = freqs.cos().to(dtype)
    sin = freqs.sin().to(dtype)
    if device is not None:
        cos, sin = cos.to(device), sin.to(device)
    return cos, sin


def rope_apply(
    q: torch.Tensor, k: torch.Tensor, cos: torch.Tensor, sin: torch.Tensor,
    position_ids: torch.Tensor,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Rotary embedding with arbitrary position_ids (tree positions for
    spec-decode ride through here; ref pytorch_backend.py:59-110).

    q: (B, Hq, T, D); k: (B, Hkv, T, D); position_ids: (B, T) int64/int32.
    cos/sin: (max_pos, D/2) fp32. Rotation convention: interleaved-free
    "half-split" (HF llama): x1 = x[..., :D/2], x2 = x[..., D/2:].
    """
    B, _, T, D = q.shape
    pos = position_ids.long()
    c = cos[pos].unsqueeze(1).float()  # (B, 1, T, D/2)
    s = sin[pos].unsqueeze(1).float()

    def rot(x):
        xf = x.float()
        x1, x2 = xf[..., : D // 2], xf[..., D // 2:]
        o1 = x1 * c - x2 * s
        o2 = x2 * c + x1 * s
        return torch.cat([o1, o2], dim=-1).to(x.dtype)

    return rot(q), rot(k)


# ---------------------------------------------------------------------------
# Activation / MLP core
# ---------------------------------------------------------------------------

def swiglu(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """SiLU(gate) * up (ref mlp_llama, pytorch_backend.py:1033-1048)."""
    g = gate.float()
    return (g * torch.sigmoid(g) * up.float()).to(gate.dtype)


def gelu_tanh(x: torch.Tensor) -> torch.Tensor:
    xf = x.float()
    return (0.5 * xf * (1.0 + torch.tanh(0.7978845608028654 * (xf + 0.044715 * xf ** 3)))).to(x.dtype)


# ---------------------------------------------------------------------------
# Paged KV cache primitives
# ---------------------------------------------------------------------------

def kv_write(
    k_new: torch.Tensor, v_new: torch.Tensor,
    k_pages: torch.Tensor, v_pages: torch.Tensor,
    page_table: torch.Tensor, start_pos: torch.Tensor,
) -> None:
    """Scatter new K/V into the paged cache, in place.

    k_new/v_new: (B, Hkv, T, D); k_pages: (n_pages, Hkv, P, D) token-major;
    v_pages: (n_pages, Hkv, D, P) d-major (transposed for direct MFMA
    B-fragment loads in the decode kernel — see PagedKVCache.v_pages);
    page_table: (B, max_pages) int32; start_pos: (B,) int32 — absolute position
    of k_new[:, :, 0]. (ref paged_kv.py:137-204 `write`, MI-native layout.)
    """
    B, Hkv, T, D = k_new.shape
    P = k_pages.shape[2]
    for b in range(B):
        s = int(start_pos[b])
        for t in range(T):
            pos = s + t
            page = int(page_table[b, pos // P])
            slot = pos % P
            k_pages[page, :, slot, :] = k_new[b, :, t, :]
            v_pages[page, :, :, slot] = v_new[b, :, t, :]


def kv_gather(
    k_pages: torch.Tensor, v_pages: torch.Tensor,
    page_table: torch.Tensor, ctx_len: int, batch_index: int,
) -> Tuple[torch.Tensor, torch.Tensor]:
    """Gather a sequence prefix back to dense (Hkv, ctx_len, D) tensors
    (ref paged_kv.py:265-316 `gather_prefix`)."""
    P = k_pages.shape[2]
    n = (ctx_len + P - 1) // P
    pages = page_table[batch_index, :n].long()
    k = k_pages[pages].permute(1, 0, 2, 3).reshape(k_pages.shape[1], n * P, -1)[:, :ctx_len]
    # v_pages is d-major (n_pages, Hkv, D, P) -> (Hkv, n, P, D) -> (Hkv, ctx, D)
    v = v_pages[pages].permute(1, 0, 3, 2).reshape(v_pages.shape[1], n * P, -1)[:, :ctx_len]
    return k, v


# ---------------------------------------------------------------------------
# Attention over the paged cache (decode AND prefill use the same entry)
# ---------------------------------------------------------------------------

def attn_paged(
    q: torch.Tensor,
    k_pages: torch.Tensor, v_pages: torch.Tensor,
    page_table: torch.Tensor,
    q_start: torch.Tensor,
    scale: Optional[float] = None,
    tree_mask: Optional[torch.Tensor] = None,
    sliding_window: Optional[int] = None,
    alibi_slopes: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    """Causal attention of q against the paged KV cache.

    Query i of sequence b sits at absolute position ``q_start[b] + i`` and
    attends to cache positions <= that position (its own k/v must already be
    written to the pages — `kv_write` first, then `attn_paged`; this single
    entry replaces the reference's separate mha_llama / mha_gen_llama pair,
    pytorch_backend.py:665-916).

    q: (B, Hq, Tq, D) -> out (B, Hq, Tq, D), GQA via Hq % Hkv == 0.
    tree_mask: (B, Tq, Tq) bool over the NEW tokens (True = may attend),
    used by tree-structured speculative verify (ref backend.py:944-1047);
    positions before q_start stay fully visible.
    sliding_window: if set, query at position p attends only to
    positions > p - sliding_window (gemma-family per-layer sliding attention).
    """
    B, Hq, Tq, D = q.shape
    Hkv = k_pages.shape[1]
    G = Hq // Hkv
    if scale is None:
        scale = 1.0 / math.sqrt(D)
    out = torch.empty_like(q)
    for b in range(B):
        s = int(q_start[b])
        ctx = s + Tq
        k, v = kv_gather(k_pages, v_pages, page_table, ctx, b)  # (Hkv, ctx, D)
        kf, vf = k.float(), v.float()
        qf = q[b].float()  # (Hq, Tq, D)
        # scores: (Hq, Tq, ctx)
        kg = kf.repeat_interleave(G, dim=0)
        vg = vf.repeat_interleave(G, dim=0)
        scores = torch.einsum("htd,hcd->htc", qf, kg) * scale
        if alibi_slopes is not None:
            # ALiBi (bloom family): softmax-shift-invariant absolute form
            # bias[h, :, j] = slope_h * j (HF bloom build_alibi_tensor)
            scores = scores + alibi_slopes.float().to(q.device).view(-1, 1, 1) * \
                torch.arange(ctx, dtype=torch.float32,
                             device=q.device).view(1, 1, ctx)
        dev = q.device
        pos_q = torch.arange(s, s + Tq, device=dev).unsqueeze(1)  # (Tq, 1)
        pos_k = torch.arange(ctx, device=dev).unsqueeze(0)        # (1, ctx)
        mask = pos_k <= pos_q
        if sliding_window is not None:
            mask &= pos_k > (pos_q - sliding_window)
        if tree_mask is not None:
            # new-token block (positions >= s) follows the tree mask instead
            new_block = torch.zeros(Tq, ctx, dtype=torch.bool, device=dev)
            new_block[:, s:] = tree_mask[b].to(dev)
            old_block = mask.clone()
            old_block[:, s:] = False
            mask = old_block | new_block
        scores = scores.masked_fill(~mask.to(scores.device).unsqueeze(0), float("-inf"))
        p = torch.softmax(scores, dim=-1)
        out[b] = torch.einsum("htc,hcd->htd", p, vg).to(q.dtype)
    return out


# ---------------------------------------------------------------------------
# 4-bit group quantization (ref flexgen_utils/compression.py:94-210)
# ---------------------------------------------------------------------------

def quant4_pack(x: torch.Tensor, group_size: int = 64) -> Tuple[torch.Tensor, torch.Tensor, torch.Tensor]:
    """Group-wise 4-bit min/max quantization along the last dim.

    Returns (packed uint8 [.., G, group_size//2], scale fp16 [.., G], zero fp16 [.., G]).
    """
    orig_shape = x.shape
    assert orig_shape[-1] % group_size == 0
    g = x.float().reshape(*orig_shape[:-1], -1, group_size)
    mn = g.min(dim=-1, keepdim=True).values
    mx = g.max(dim=-1, keepdim=True).values
    scale = (mx - mn).clamp_min(1e-8) / 15.0
    q = ((g - mn) / scale).round().clamp(0, 15).to(torch.uint8)
    packed = (q[..., 0::2] | (q[..., 1::2] << 4)).contiguous()
    return packed, scale.squeeze(-1).half(), mn.squeeze(-1).half()


def quant4_unpack(
    packed: torch.Tensor, scale: torch.Tensor, zero: torch.Tensor,
    dtype: torch.dtype = torch.bfloat16,
) -> torch.Tensor:
    lo = (packed & 0xF).float()
    hi = (packed >> 4).float()
    q = torch.stack([lo, hi], dim=-1).reshape(*packed.shape[:-1], -1)
    x = q * scale.float().unsqueeze(-1) + zero.float().unsqueeze(-1)
    return x.reshape(*packed.shape[:-2], -1).to(dtype)


def alibi_slopes(n_heads: int) -> torch.Tensor:
    """HF bloom build_alibi_tensor slopes (positive, per head; the absolute
    bias slope*j is softmax-shift-equivalent to the -slope*(i-j) distance
    penalty)."""
    import math as _m

    closest = 2 ** _m.floor(_m.log2(n_heads))
    base = 2.0 ** (-(2.0 ** -(_m.log2(closest) - 3)))
    slopes = [base ** (i + 1) for i in range(closest)]
    if closest < n_heads:
        extra_base = 2.0 ** (-(2.0 ** -(_m.log2(2 * closest) - 3)))
        slopes += [extra_base ** (2 * i + 1) for i in range(n_heads - closest)]
    return torch.tensor(slopes, dtype=torch.float32)


def attn_paged_topk(
    q: torch.Tensor,
    k_pages: torch.Tensor, v_pages: torch.Tensor,
    page_table: torch.Tensor,
    ctx_lens: torch.Tensor,
    sparsity: float,
    scale: Optional[float] = None,
    alibi_slopes: Optional[torch.Tensor] = None,
) -> torch.Tensor:
    """Top-k sparse decode attention (parity: reference
    pytorch_backend.py:935-968 `_sparse_attention_value` driven by
    Policy.attn_sparsity): scores are computed against the full K cache,
    then only the top ceil(sparsity*ctx) positions' V rows participate in
    the weighted sum — the V fetch (the expensive half when the cache is
    host-resident) touches a fraction of the cache. sparsity >= 1 is exact
    dense attention. q: (B, Hq, 1, D)."""
    B, Hq, Tq, D = q.shape
    assert Tq == 1, "top-k sparse path is decode-only (one query token)"
    Hkv = k_pages.shape[1]
    G = Hq // Hkv
    if scale is None:
        scale = 1.0 / math.sqrt(D)
    out = torch.empty_like(q)
    for b in range(B):
        ctx = int(ctx_lens[b])
        k, v = kv_gather(k_pages, v_pages, page_table, ctx, b)  # (Hkv, ctx, D)
        kg = k.float().repeat_interleave(G, dim=0)              # (Hq, ctx, D)
        vg = v.float().repeat_interleave(G, dim=0)
        qf = q[b, :, 0].float()                                 # (Hq, D)
        scores = torch.einsum("hd,hcd->hc", qf, kg) * scale     # (Hq, ctx)
        if alibi_slopes is not None:
            scores = scores + alibi_slopes.float().to(q.device).view(-1, 1) * \
                torch.arange(ctx, dtype=torch.float32, device=q.device)
        kkeep = max(1, min(ctx, math.ceil(sparsity * ctx)))
        top = scores.topk(kkeep, dim=-1)                        # (Hq, kkeep)
        w = torch.softmax(top.values, dim=-1)                   # renormalized
        vsel = torch.gather(
            vg, 1, top.indices.unsqueeze(-1).expand(-1, -1, D))  # (Hq, kk, D)
        out[b, :, 0] = torch.einsum("hk,hkd->hd", w, vsel).to(q.dtype)
    return out


def attn_paged_mixed(
    q: torch.Tensor,
    k_pages: torch.Tensor, v_pages: torch.Tensor,
    page_table: torch.Tensor,
    ctx_lens: torch.Tensor,
    host_k: torch.Tensor, host_v: torch.Tensor,
    scale: Optional[float] = None,
) -> torch.Tensor:
    """Mixed-device decode attention (parity: reference
    pytorch_backend.py:969-1014 `_mixed_device_attention` — KV split into a
    device-resident recent segment and a host-resident old segment; the host
    part is computed fp32 on CPU and the two partial softmaxes are merged).

    host_k/host_v: (B, Hkv, S_host, D) on CPU — positions [0, S_host).
    The paged pool holds positions [S_host, S_host + ctx_lens[b]).
    q: (B, Hq, 1, D) on any device. Merge is exact (log-sum-exp), so the
    result equals dense attention over the concatenated cache.
    """
    B, Hq, Tq, D = q.shape
    assert Tq == 1, "mixed-device path is decode-only"
    Hkv = k_pages.shape[1]
    G = Hq // Hkv
    S_host = host_k.shape[2]
    if scale is None:
        scale = 1.0 / math.sqrt(D)
    out = torch.empty_like(q)
    for b in range(B):
        qf = q[b, :, 0].float()  # (Hq, D)
        # host segment on CPU (fp32)
        qc = qf.cpu()
        kh = host_k[b].float().repeat_interleave(G, dim=0)  # (Hq, S_host, D)
        vh = host_v[b].float().repeat_interleave(G, dim=0)
        s_h = torch.einsum("hd,hcd->hc", qc, kh) * scale
        m_h = s_h.max(-1, keepdim=True).values
        p_h = torch.exp(s_h - m_h)
        l_h = p_h.sum(-1)                                   # (Hq,)
        o_h = torch.einsum("hc,hcd->hd", p_h, vh)
        # device-resident recent segment via the paged pool
        ctx = int(ctx_lens[b])
        k, v = kv_gather(k_pages, v_pages, page_table, ctx, b)
        kg = k.float().repeat_interleave(G, dim=0)
        vg = v.float().repeat_interleave(G, dim=0)
        s_d = torch.einsum("hd,hcd->hc", qf, kg) * scale
        m_d = s_d.max(-1, keepdim=True).values
        p_d = torch.exp(s_d - m_d)
        l_d = p_d.sum(-1)
        o_d = torch.einsum("hc,hcd->hd", p_d, vg)
        # exact merge of the two partial softmaxes
        m_hd, m_dd = m_h[:, 0].to(q.device), m_d[:, 0]
        o_hd, l_hd = o_h.to(q.device), l_h.to(q.device)
        m = torch.maximum(m_hd, m_dd)
        c_h = torch.exp(m_hd - m).unsqueeze(-1)
        c_d = torch.exp(m_dd - m).unsqueeze(-1)
        denom = l_hd.unsqueeze(-1) * c_h + l_d.unsqueeze(-1) * c_d
        out[b, :, 0] = ((o_hd * c_h + o_d * c_d) / denom).to(q.dtype)
    return out


def moe_gemm_grouped(A: torch.Tensor, W: torch.Tensor, off: torch.Tensor,
                     rowmap: Optional[torch.Tensor] = None,
                     scale: Optional[torch.Tensor] = None,
                     S: Optional[int] = None) -> torch.Tensor:
    """Reference for the grouped expert GEMM (ops/hip/moe_gemm.hip):
    per-slot C[s] = A[row(s)] @ W[expert(s)]^T * scale[s]; slots grouped by
    expert via the off prefix sums. fp32 accumulation like the MFMA path."""
    E, N, K = W.shape
    offs = off.tolist()
    if S is None:
        S = offs[-1]
    C = torch.zeros(S, N, dtype=A.dtype, device=A.device)
    for e in range(E):
        a, b = offs[e], offs[e + 1]
        if b <= a:
            continue
        slots = torch.arange(a, b, device=A.device)
        rows = rowmap[slots].long() if rowmap is not None else slots
        y = A[rows].float() @ W[e].float().t()
        if scale is not None:
            y = y * scale[slots].float().unsqueeze(1)
        C[slots] = y.to(A.dtype)
    return C


# ---------------------------------------------------------------------------
# Ragged batches (ops/ragged.py): the CPU forms of its kernels
# ---------------------------------------------------------------------------

def grouped_rms_norm(x: torch.Tensor, weight: torch.Tensor, groups: int,
                     eps: float) -> torch.Tensor:
    """RMS norm of `groups` equal consecutive parts of the last dim, each by
    its own mean square; fp32 in and out."""
    xf = x.float()
    g = xf.reshape(*xf.shape[:-1], groups, -1)
    g = g * torch.rsqrt(g.pow(2).mean(-1, keepdim=True) + eps)
    return g.reshape(xf.shape) * weight.float()


def distance_slopes(n_heads: int) -> torch.Tensor:
    """Per-head linear distance penalties 2^(-8 (h+1) / n_heads). Equal to
    alibi_slopes where n_heads is a power of two, and only there."""
    h = torch.arange(1, n_heads + 1, dtype=torch.float64)
    return torch.pow(2.0, -8.0 * h / n_heads).float()


def xielu(z: torch.Tensor, pos: float, neg: float) -> torch.Tensor:
    """pos z^2 + z/2 above zero, neg (e^z - 1 - z) + z/2 below; pos and neg
    are the positive curvatures (softplus already applied)."""
    below = neg * (torch.expm1(z.clamp(max=0.0)) - z)
    return torch.where(z > 0, pos * z * z, below) + 0.5 * z


def route_topk(logits: torch.Tensor, correction: torch.Tensor, experts: int,
               top: int, scale: float, sigmoid: bool = False,
               renorm: bool = False):
    """Softmax (or sigmoid) scores; the choice adds `correction`, the weights do not and
    are not renormalized, unless renorm: then a token's weights sum to scale
    (with softmax scores: a softmax over the chosen logits). Outputs from
    `experts` on are identity experts.
    Returns ids (N, top) int32 with -1 for identity choices, weights (N, top)
    and the identity experts' summed weight (N,)."""
    s = (torch.sigmoid(logits.float()) if sigmoid
         else torch.softmax(logits.float(), dim=-1))
    choice = s if correction is None else s + correction.float()
    # stable sort: the lowest index wins a tie
    ids = torch.sort(choice, dim=-1, descending=True,
                     stable=True).indices[:, :top]
    w = torch.gather(s, 1, ids)
    if renorm:
        w = w / w.sum(-1, keepdim=True)
    w = w * scale
    ident = ids >= experts
    idw = (w * ident).sum(-1)
    return torch.where(ident, -1, ids).int(), w, idw


def attn_ragged(q, k_pages, v_pages, batch, dim: int, vdim: int, scale: float,
                window: int = 0, slopes=None, gate=None,
                sinks=None, chunk: int = 0) -> torch.Tensor:
    """Paged attention of a ragged batch: q (N, H, >= dim) -> (N, H * vdim).
    Row n sees positions j of its own sequence with 0 <= pos - j (< window),
    with chunk only those of its own stretch of that many positions;
    score = q.k * scale - slope_h * (pos - j); sinks_h is one more score that
    has no value; out *= sigmoid(gate). Without v_pages the values are the
    first vdim elements of the keys."""
    N, H = q.shape[0], q.shape[1]
    G = k_pages.shape[1]
    out = torch.zeros(N, H, vdim, dtype=torch.float32, device=q.device)
    for s in range(batch.page_table.shape[0]):
        rows = ((batch.tok_seq == s) & (batch.tok_pos >= 0)).nonzero()[:, 0]
        if rows.numel() == 0:
            continue
        pos = batch.tok_pos[rows].long()
        ctx = int(pos.max()) + 1
        k, v = kv_gather(k_pages, v_pages if v_pages is not None
                         else k_pages.transpose(2, 3), batch.page_table, ctx, s)
        k = k[..., :dim].float().repeat_interleave(H // G, dim=0)
        v = v[..., :vdim].float().repeat_interleave(H // G, dim=0)
        sc = torch.matmul(q[rows, :, :dim].float().transpose(0, 1),
                          k.transpose(1, 2)) * scale          # (H, R, ctx)
        dist = pos.view(-1, 1) - torch.arange(ctx, device=q.device).view(1, -1)
        if slopes is not None:
            sc = sc - slopes.view(-1, 1, 1) * dist.float()
        seen = dist >= 0
        if window > 0:
            seen &= dist < window
        if chunk > 0:
            seen &= dist <= pos.view(-1, 1) % chunk
        sc = sc.masked_fill(~seen, float("-inf"))
        if sinks is not None:
            sc = torch.cat([sc, sinks.float().view(-1, 1, 1).expand(
                -1, sc.shape[1], 1)], -1)
        p = torch.softmax(sc, dim=-1)[..., :ctx]
        out[rows] = torch.matmul(p, v).transpose(0, 1)
    out = out.reshape(N, H * vdim)
    if gate is not None:
        out = out * torch.sigmoid(gate.float())
    return out.to(q.dtype)


def attn_differential(q, k_pages, v_pages, batch, dim: int, vdim: int,
                      scale: float, lam: float, factor: float, eps: float,
                      window: int = 0, chunk: int = 0) -> torch.Tensor:
    """Two attentions per head over the same values: q (N, H, 2, stored dim),
    keys (np, G, P, 2 * stored dim); (a1 - lam * a2), RMS-normed per head, times
    factor: (N, H * vdim)."""
    N, H, _, dp = q.shape
    a = [attn_ragged(q[:, :, m].float(), k_pages[..., m * dp:(m + 1) * dp],
                     v_pages, batch, dim, vdim, scale, window, chunk=chunk)
         for m in range(2)]
    o = (a[0] - lam * a[1]).view(N, H, vdim)
    one = torch.ones(vdim, device=q.device)
    return (grouped_rms_norm(o, one, 1, eps) * factor).reshape(N, H * vdim).to(
        q.dtype)


def moe_experts(h, up, down, ids, wts, weight_input: bool = False,
                limit: float = math.inf, slope: float = 1.0,
                shift: float = 0.0) -> torch.Tensor:
    """y (N, top, W): wts * down(act) of every chosen expert, or down of the
    activation of wts * h; act = g sigmoid(slope g) (u + shift) with
    g = min(gate h, limit), u = clamp(up h, -limit, limit) with two planes
    (E, 2, F, K) of first weights, relu(up h)^2 with one. Rows of skipped
    choices (id < 0) are zero."""
    N, top = ids.shape
    y = torch.zeros(N, top, down.shape[1], dtype=torch.float32, device=h.device)
    for e in range(up.shape[0]):
        t, k = (ids == e).nonzero(as_tuple=True)
        if t.numel() == 0:
            continue
        x, w = h[t].float(), wts[t, k, None]
        if weight_input:
            x, w = x * w, 1.0
        z = x @ up[e, -1].float().t()
        if up.shape[1] == 2:
            g = (x @ up[e, 0].float().t()).clamp(max=limit)
            z = g * torch.sigmoid(slope * g) * (z.clamp(-limit, limit) + shift)
        else:
            z = torch.relu(z) ** 2
        y[t, k] = (z.to(h.dtype).float() @ down[e].float().t()) * w
    return y.to(h.dtype)


def sinusoid(positions: torch.Tensor, turns: torch.Tensor,
             width: int) -> torch.Tensor:
    """(..., width) f32: sine of position * frequency i at entry 2 i, cosine at
    2 i + 1; turns: frequencies / 2 pi in float64."""
    r = positions.double()[..., None] * turns
    ang = (r - r.round()) * (2 * math.pi)
    y = torch.stack([torch.sin(ang), torch.cos(ang)], -1).flatten(-2)
    return y[..., :width].float()


def query_temperature(positions: torch.Tensor, coef: float,
                      every: float) -> torch.Tensor:
    """1 + coef * ln(floor((position + 1) / every) + 1), fp32."""
    steps = torch.floor((positions.double().clamp(min=0) + 1) / every)
    return (1 + coef * torch.log1p(steps)).float()


def clamped_glu(gate, up, gate_b, up_b, limit: float, slope: float):
    """g = min(gate + b, limit), u = clamp(up + b, -limit, limit);
    g * sigmoid(slope * g) * (u + 1), fp32."""
    g = gate if gate_b is None else gate + gate_b
    u = up if up_b is None else up + up_b
    g = g.clamp(max=limit)
    return g * torch.sigmoid(slope * g) * (u.clamp(-limit, limit) + 1)


def rotate_half(x: torch.Tensor, positions: torch.Tensor,
                turns: torch.Tensor, amp: float = 1.0) -> torch.Tensor:
    """Rotary positions on the first 2 * len(turns) elements of the last axis,
    element i with element i + len(turns). x (N, ..., D), positions (N,);
    turns: frequencies / 2 pi in float64, angles are reduced in float64; amp
    multiplies cosine and sine."""
    half = turns.numel()
    r = positions.double().clamp(min=0)[:, None] * turns
    ang = ((r - r.round()) * (2 * math.pi)).reshape(
        r.shape[0], *[1] * (x.dim() - 2), half)
    c = (amp * torch.cos(ang)).to(x.dtype)
    s = (amp * torch.sin(ang)).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def channel_decays(a1, a2, a2_b, tau: float) -> torch.Tensor:
    """sigmoid(a1 @ a2 + b)^(1 / tau), fp32. a2 (r, channels)."""
    z = a1.float() @ a2.float() + a2_b.float()
    return torch.exp(F.logsigmoid(z) / tau)


def forget_gates(z, bias, lower):
    """f = lower + (1 - lower) sigmoid(z + bias) and 1 - f, fp32."""
    z = z.float() + bias
    return (lower + (1 - lower) * torch.sigmoid(z),
            (1 - lower) * torch.sigmoid(-z))


def gla_scan(q, k, v, alpha, state):
    """Gated linear attention of one sequence, token by token: q, k, alpha
    (T, H, D), v (T, H, V), state (H, D, V) -> o (T, H, V), new state."""
    out = []
    for t in range(q.shape[0]):
        state = (alpha[t].unsqueeze(-1) * state
                 + k[t].unsqueeze(-1) * v[t].unsqueeze(-2))
        out.append((state * q[t].unsqueeze(-1)).sum(-2))
    return torch.stack(out), state


def mlstm_gates(z: torch.Tensor, bias: torch.Tensor, cap: float):
    """Log gates (N, H) of a matrix memory from z (N, 2 H), input gates first:
    i = cap tanh(z / cap), f = log sigmoid(cap tanh(z / cap)), fp32."""
    z = cap * torch.tanh((z.float() + bias) / cap)
    i, f = z.chunk(2, -1)
    return i, F.logsigmoid(f)


def mlstm_scan(q, k, v, i, f, S, n, m):
    """Matrix memory of one sequence, token by token: q, k (T, H, D), v
    (T, H, V), log gates i, f (T, H), state S (H, D, V), n (H, D), running
    maximum m (H,) -> o (T, H, V), new state."""
    out = []
    for t in range(q.shape[0]):
        new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        ki = k[t] * add.unsqueeze(-1)
        S = keep[:, None, None] * S + ki.unsqueeze(-1) * v[t].unsqueeze(-2)
        n = keep[:, None] * n + ki
        m = new
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out.append((S * q[t].unsqueeze(-1)).sum(-2) / den.unsqueeze(-1))
    return torch.stack(out), (S, n, m)


def causal_conv(x: torch.Tensor, past: torch.Tensor, taps: torch.Tensor,
                bias: torch.Tensor) -> torch.Tensor:
    """Per-channel convolution of x (..., T, C) after past (..., K - 1, C), taps
    (K, C) with the current token's last."""
    K, T = taps.shape[0], x.shape[-2]
    full = torch.cat([past, x], -2)
    return bias + sum(taps[j] * full[..., j:j + T, :] for j in range(K))


def rglru_inputs(u, gates_w, gates_b, decay):
    """What enters a gated linear recurrent unit, from u (..., C): log a and
    sqrt(1 - a^2) * i * u, with r and i the sigmoids of a block-diagonal product,
    gates_w (B, 2, C / B, C / B) [out, in], gates_b (2, C), log a = decay * r."""
    B, _, D, _ = gates_w.shape
    ub = u.float().reshape(-1, B, D).transpose(0, 1)
    z = [torch.matmul(ub, gates_w[:, g].float().transpose(1, 2).contiguous())
         .transpose(0, 1).reshape(u.shape) + gates_b[g] for g in range(2)]
    log_a = decay * torch.sigmoid(z[0])
    x = torch.sqrt(-torch.expm1(2 * log_a)) * torch.sigmoid(z[1]) * u.float()
    return log_a, x


def rglru_scan(log_a, x, S):
    """S <- exp(log_a) S + x token by token: (T, C) -> states (T, C), last."""
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(log_a[t]) * S + x[t]
        out.append(S)
    return torch.stack(out), S
