"""Ragged step batches: tokens of many sequences as one flat row list.

A lockstep session advances B sequences by the same T tokens. A TokenBatch has
no such shape: every sequence brings its own number of new tokens, so portions
of prompts run beside single decoded tokens, and the kernels see N = sum(T_s)
rows with a sequence index and an absolute position each. A lockstep step is
the special case of equal lengths (``lockstep_batch``), so a block needs one
forward only.

Everything the kernels read lives in device int32 tensors, so a captured decode
graph replays against the same TokenBatch after its buffers are rewritten
(``DecodeSlots``). A row with position -1 is an empty slot: it writes no K/V
and its outputs mean nothing.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np
import torch

from bloombee_amd.kv.paged import PagedKVCache, PagedKVError


@dataclass
class Context:
    """What the portions of a step see through a window, as whole pages: the
    pages one after the other, and a table of where each one went."""

    pages: torch.Tensor   # (n,) int32 page ids of the cache
    valid: torch.Tensor   # (n,) int32 tokens in use of each
    table: torch.Tensor   # (S, max pages) int32: place in `pages`, 0 = none


@dataclass
class Chunks:
    """The portions of a step cut into chunks of at most C tokens."""

    row0: torch.Tensor    # (n,) int32 first row
    len: torch.Tensor     # (n,) int32 tokens
    cu: torch.Tensor      # (portions + 1,) int32 first chunk of each


@dataclass
class TokenBatch:
    """One step's rows. N rows, S sequences; rows of a sequence are adjacent."""

    cache: PagedKVCache
    tok_seq: torch.Tensor      # (N,) int32: row of page_table
    tok_pos: torch.Tensor      # (N,) int32: absolute position, -1 = empty slot
    cu: torch.Tensor           # (S+1,) int32: first row of each sequence
    q_start: torch.Tensor      # (S,) int32: position of its first new token
    page_table: torch.Tensor   # (S, max_pages) int32
    pre_list: torch.Tensor     # sequences that bring two tokens or more
    dec_list: torch.Tensor     # sequences that bring one
    max_new: int               # longest portion
    max_ctx: int               # longest context after this step (upper bound)
    slots: Optional[torch.Tensor] = None   # (S,) int32: recurrent state rows
    # (N, W) f32: the embedding output, for layers that read it again
    embedded: Optional[torch.Tensor] = None
    # host copies of starts, counts and page lists, where a step has portions
    host: Optional[Tuple[Sequence[int], Sequence[int],
                         Sequence[Sequence[int]]]] = None
    _cut: Dict[tuple, object] = field(default_factory=dict)

    def _portions(self):
        if self.host is None:
            raise PagedKVError("a captured decode step has no portions")
        starts, counts, pages = self.host
        return [(i, int(st), int(n), pages[i]) for i, (st, n)
                in enumerate(zip(starts, counts)) if n > 1]

    def context(self, window: int) -> Context:
        """Cached tokens the portions of two tokens or more see (0 = all)."""
        key = ("context", window)
        if key not in self._cut:
            P = self.cache.page_size
            table = np.zeros(tuple(self.page_table.shape), dtype=np.int32)
            ids: List[int] = []
            valid: List[int] = []
            for i, st, n, pages in self._portions():
                a = max(0, st - window + 1) // P if window > 0 else 0
                b = (st + n + P - 1) // P
                table[i, a:b] = np.arange(len(ids), len(ids) + b - a)
                ids.extend(pages[a:b])
                valid.extend([P] * (b - a - 1) + [st + n - (b - 1) * P])
            t = _upload([np.asarray(ids, dtype=np.int32),
                         np.asarray(valid, dtype=np.int32), table],
                        self.cache.device)
            self._cut[key] = Context(*t)
        return self._cut[key]

    def chunks(self, C: int) -> Chunks:
        key = ("chunks", C)
        if key not in self._cut:
            first = np.concatenate([[0], np.cumsum(self.host[1])])
            row0: List[int] = []
            length: List[int] = []
            cu = [0]
            for i, _, n, _ in self._portions():
                for at in range(0, n, C):
                    row0.append(int(first[i]) + at)
                    length.append(min(C, n - at))
                cu.append(len(row0))
            self._cut[key] = Chunks(*_upload(
                [np.asarray(v, dtype=np.int32) for v in (row0, length, cu)],
                self.cache.device))
        return self._cut[key]

    def split_hidden(self, hidden: torch.Tensor, width: int) -> torch.Tensor:
        """The residual among the columns of hidden states (N, columns), as a
        view; what travels behind it is kept for the layers that read it."""
        if hidden.shape[1] > width:
            self.embedded = hidden[:, width:]
        return hidden[:, :width]

    @property
    def n_tokens(self) -> int:
        return self.tok_seq.numel()

    def k_pages(self, layer: int) -> torch.Tensor:
        return self.cache.k_pages(layer)

    def v_pages(self, layer: int) -> torch.Tensor:
        return self.cache.v_pages(layer)


def _upload(arrays: Sequence[np.ndarray], device: torch.device):
    """All index arrays of a step in one transfer; returns device views."""
    sizes = [a.size for a in arrays]
    # 16 B alignment for every view
    offs = np.cumsum([0] + [(n + 3) // 4 * 4 for n in sizes])
    host = torch.zeros(int(offs[-1]), dtype=torch.int32,
                       pin_memory=device.type == "cuda")
    buf = host.numpy()
    for a, o, n in zip(arrays, offs, sizes):
        buf[o:o + n] = a.reshape(-1)
    dev = host.to(device, non_blocking=True) if device.type == "cuda" else host
    return [dev[int(o):int(o) + n].view(a.shape)
            for a, o, n in zip(arrays, offs, sizes)]


def build_batch(cache: PagedKVCache, starts: Sequence[int],
                counts: Sequence[int], pages: Sequence[Sequence[int]],
                slots: Optional[Sequence[int]] = None) -> TokenBatch:
    """starts/counts: first position and number of new tokens of each
    sequence; pages: its page list, already long enough for them; slots: its
    recurrent state row."""
    S = len(starts)
    if S == 0 or min(counts) < 1:
        raise PagedKVError("a step needs at least one token per sequence")
    P = cache.page_size
    for s0, n, pg in zip(starts, counts, pages):
        if (s0 + n + P - 1) // P > len(pg):
            raise PagedKVError("sequence has fewer pages than tokens")
    cnt = np.asarray(counts, dtype=np.int32)
    st = np.asarray(starts, dtype=np.int32)
    cu = np.zeros(S + 1, dtype=np.int32)
    np.cumsum(cnt, out=cu[1:])
    seq = np.repeat(np.arange(S, dtype=np.int32), cnt)
    pos = np.arange(cu[-1], dtype=np.int32) - cu[seq] + st[seq]
    table = np.zeros((S, max(len(pg) for pg in pages)), dtype=np.int32)
    for i, pg in enumerate(pages):
        table[i, :len(pg)] = pg
    pre = np.nonzero(cnt > 1)[0].astype(np.int32)
    dec = np.nonzero(cnt == 1)[0].astype(np.int32)
    sl = np.asarray([-1] * S if slots is None else slots, dtype=np.int32)
    t = _upload([seq, pos, cu, st, table, pre, dec, sl], cache.device)
    return TokenBatch(cache, *t[:5], pre_list=t[5], dec_list=t[6],
                      max_new=int(cnt.max()), max_ctx=int((st + cnt).max()),
                      slots=t[7], host=(starts, counts, pages))


def session_batch(parts: Sequence[Tuple["object", int]]) -> TokenBatch:
    """Batch over whole sessions: parts are (SessionHandle, new tokens) whose
    extend() has already run; every sequence of a session brings as many."""
    starts: List[int] = []
    counts: List[int] = []
    pages: List[Sequence[int]] = []
    slots: List[int] = []
    for handle, n in parts:
        for s in handle.seqs:
            starts.append(s.l_spec - n)
            counts.append(n)
            pages.append(s.pages)
            slots.append(s.slot)
    cache = parts[0][0].cache
    return build_batch(cache, starts, counts, pages, slots)


def lockstep_batch(kv, start_pos: torch.Tensor, B: int, T: int) -> TokenBatch:
    """Batch of a lockstep session step (SessionHandle or SessionView): rows
    [b, t] at start_pos[b] + t. Device-side only, so that a decode step that is
    captured into a graph follows start_pos and the page table on replay."""
    handle = getattr(kv, "handle", kv)
    if getattr(kv, "pos_offset", 0):
        raise PagedKVError("host-prefix (mixed-device) sessions have no "
                           "ragged step")
    dev = handle.cache.device
    table = kv.page_table()
    st = start_pos.to(device=dev, dtype=torch.int32)
    idx = torch.arange(B, dtype=torch.int32, device=dev)
    if T == 1:
        seq, pos = idx, st
    else:
        seq = idx.repeat_interleave(T)
        pos = (st.view(B, 1) + torch.arange(T, dtype=torch.int32, device=dev)
               ).reshape(-1)
    none = idx[:0]
    host = None
    if T > 1:
        seqs = kv.seqs      # already extended by the step's tokens
        host = ([s.l_spec - T for s in seqs], [T] * B, [s.pages for s in seqs])
    return TokenBatch(
        handle.cache, seq, pos,
        cu=torch.arange(0, B * T + 1, T, dtype=torch.int32, device=dev),
        q_start=st, page_table=table,
        pre_list=none if T == 1 else idx, dec_list=idx if T == 1 else none,
        max_new=T, max_ctx=table.shape[1] * handle.cache.page_size,
        slots=kv.state_slots(), host=host)


class DecodeSlots:
    """Fixed device buffers of a decode step of up to B sequences, for graph
    capture: fill() writes this step's rows, unused slots stay empty."""

    def __init__(self, cache: PagedKVCache, B: int, max_len: int):
        dev = cache.device
        self.B = B
        self.max_pages = (max_len + cache.page_size - 1) // cache.page_size
        n = 4 * B + B * self.max_pages
        self._dev = torch.zeros(n, dtype=torch.int32, device=dev)
        self.ids = self._dev[:B]
        pos = self._dev[B:2 * B]
        slots = self._dev[2 * B:3 * B]
        self.prev = self._dev[3 * B:4 * B]   # token before each, -1 = none
        idx = torch.arange(B, dtype=torch.int32, device=dev)
        self.batch = TokenBatch(
            cache, tok_seq=idx, tok_pos=pos,
            cu=torch.arange(B + 1, dtype=torch.int32, device=dev),
            q_start=pos, page_table=self._dev[4 * B:].view(B, self.max_pages),
            pre_list=idx[:0], dec_list=idx, max_new=1,
            max_ctx=self.max_pages * cache.page_size, slots=slots)

    def fill(self, tokens: Sequence[int], positions: Sequence[int],
             pages: Sequence[Sequence[int]],
             slots: Optional[Sequence[int]] = None,
             prev: Optional[Sequence[int]] = None) -> None:
        B, n = self.B, len(tokens)
        host = torch.zeros(self._dev.numel(), dtype=torch.int32,
                           pin_memory=self._dev.is_cuda)
        buf = host.numpy()
        buf[:n] = tokens
        buf[B:2 * B] = -1
        buf[B:B + n] = positions
        if slots is not None:
            buf[2 * B:2 * B + n] = slots
        if prev is not None:
            buf[3 * B:3 * B + n] = prev
        table = buf[4 * B:].reshape(B, self.max_pages)
        for i, pg in enumerate(pages):
            table[i, :len(pg)] = pg
        self._dev.copy_(host, non_blocking=True)
