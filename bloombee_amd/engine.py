"""Local (single-process) inference engine: embeddings + block stack + LM head.

This is the innermost compute loop shared by:
  * bench.py at N=1 (the whole model on one MI355X),
  * the per-worker stage runner in parallel/pipeline.py (a contiguous block
    range per rank),
  * the server backend (server/backend.py) which serves the same blocks over
    the decentralized transport.

The reference splits this across DistributedLlamaModel (client embeddings +
lm_head, models/llama/model.py:45-118) and per-server block execution; here
the same Blocks object serves both local and distributed paths.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch
import torch.nn.functional as F

from bloombee_amd.kv.batch import (DecodeSlots, TokenBatch, lockstep_batch,
                                   session_batch)
from bloombee_amd.kv.paged import (AllocationFailed, PagedKVCache,
                                   SessionHandle)
from bloombee_amd.models.auto import get_block_class
from bloombee_amd.models.base import (ModelConfig, get_family,
                                      resolve_config)
from bloombee_amd.models.llama.block import RopeTables
from bloombee_amd.utils.logging import get_logger
from bloombee_amd import ops
from bloombee_amd.ops import ragged

logger = get_logger(__name__)


class BlockStack(torch.nn.Module):
    """A contiguous range [start, end) of transformer blocks on one device."""

    def __init__(self, config: ModelConfig, start: int, end: int,
                 device="cpu", seed: int = 0):
        super().__init__()
        self.config = config
        self.start, self.end = start, end
        block_cls = get_block_class(config.model_type)
        self.rope = (None if getattr(block_cls, "token_batched", False)
                     else RopeTables(config))
        # blocks that run whole ragged steps (kv/batch.py)
        self.token_batched = self.rope is None
        self.blocks = torch.nn.ModuleList()
        owners: Dict[int, torch.nn.Module] = {}   # of weights, by first layer
        for i in range(start, end):
            blk = block_cls(config, layer_index=i, rope=self.rope).to(device)
            j = config.weights_of(i)
            if j in owners:
                blk.share_weights(owners[j])
            else:
                blk.init_random(seed=seed * 10_000 + j)
                owners[j] = blk
            blk.layer_index = i - start  # KV page index local to this stack's pool
            self.blocks.append(blk)
        # chain blocks so each one's down-proj epilogue can leave row
        # sum-of-squares for the next one's fused input rmsnorm
        # (llama/block.py fuse_norm path); first block has no producer
        # and keeps the separate-norm launch
        for j in range(1, len(self.blocks)):
            # bypass Module.__setattr__: a plain reference, not a submodule
            object.__setattr__(self.blocks[j], "prev_block",
                               self.blocks[j - 1])
        for blk in self.blocks:
            src = getattr(blk, "kv_source", None)
            if src is not None and src >= start:
                object.__setattr__(blk, "train_source",
                                   self.blocks[src - start])
        self.device = torch.device(device)

    def make_kv(self, max_tokens: int,
                max_seqs: Optional[int] = None) -> PagedKVCache:
        """max_seqs: state slots of recurrent layers (default: configured)."""
        # per-layer KV geometry hooks (gemma-4 heterogeneous head_dim/kv heads;
        # kv_layout also names value sizes and shared layers)
        if hasattr(self.config, "kv_layout"):
            geometry = self.config.kv_layout(self.start, self.end)
        elif hasattr(self.config, "kv_geometry"):
            hkv, dims = self.config.kv_geometry(self.start, self.end)
            geometry = dict(num_kv_heads=hkv, head_dim=dims)
        else:
            geometry = dict(num_kv_heads=self.config.num_key_value_heads,
                            head_dim=self.config.head_dim)
        from bloombee_amd.config import get_config
        kvc = get_config().kv
        P = kvc.page_size
        # the decode kernels walk KV in 32-position tiles and require page
        # boundaries to align (attn_decode_mfma.hip: "P | 32")
        if 32 % P != 0:
            raise ValueError(f"BBAMD_KV_PAGE_SIZE must divide 32, got {P}")
        return PagedKVCache(
            num_layers=len(self.blocks),
            **geometry,
            max_tokens=max_tokens,
            page_size=P,
            device=self.device,
            dtype=self.config.dtype,
            max_seqs=max_seqs or kvc.max_seqs,
        )

    @torch.no_grad()
    def forward_inference(self, hidden: torch.Tensor, kv: SessionHandle,
                          start_pos: torch.Tensor,
                          position_ids: Optional[torch.Tensor] = None,
                          tree_mask: Optional[torch.Tensor] = None,
                          deep_prompts: Optional[torch.Tensor] = None,
                          ) -> torch.Tensor:
        # deep p-tuning (ref client/ptune.py deep mode): deep_prompts is
        # (n_local_blocks, pre, H); block i's slice is added to the prompt
        # positions (< pre) of its input. Decode steps past the prompt
        # region skip the addition entirely.
        sp0 = int(start_pos[0]) if deep_prompts is not None else 0
        pre = deep_prompts.shape[1] if deep_prompts is not None else 0
        n_over = min(pre - sp0, hidden.shape[1]) if sp0 < pre else 0
        if self.token_batched:
            if tree_mask is not None or position_ids is not None:
                raise NotImplementedError(
                    f"{self.config.model_type}: no tree-structured steps")
            B, T, C = hidden.shape
            x = hidden.reshape(B * T, C).to(torch.float32, copy=True)
            hook = None
            if n_over > 0:
                def hook(i):
                    dp = deep_prompts[i, sp0:sp0 + n_over].to(x.dtype)
                    x.view(B, T, C)[:, :n_over, :dp.shape[-1]] += dp
            self.forward_batch(x, lockstep_batch(kv, start_pos, B, T), hook)
            return x.view(B, T, C)
        for i, blk in enumerate(self.blocks):
            if n_over > 0:
                dp = deep_prompts[i, sp0:sp0 + n_over].to(hidden.dtype)
                hidden[:, :n_over] += dp
            if tree_mask is not None:
                hidden = blk.forward_inference(hidden, kv, start_pos,
                                               position_ids, tree_mask=tree_mask)
            else:
                hidden = blk.forward_inference(hidden, kv, start_pos, position_ids)
        return hidden

    @torch.no_grad()
    def forward_batch(self, hidden: torch.Tensor, batch: TokenBatch,
                      before_block=None) -> torch.Tensor:
        """One ragged step: hidden (N, columns) f32 through all blocks, in place.
        A block may leave something to the next one (its sum, for that one's norm
        to fold in); before_block(i) needs the sum, so it forces the fold."""
        x = batch.split_hidden(hidden, self.config.hidden_size)
        left = None
        for i, blk in enumerate(self.blocks):
            if before_block is not None:
                if left is not None:
                    left.settle(x)
                left = None
                before_block(i)
            left = blk.forward_tokens(x, left, batch)
        left.settle(x)
        return hidden

    def forward_train(self, hidden: torch.Tensor, start_pos: int = 0,
                      deep_prompts: Optional[torch.Tensor] = None) -> torch.Tensor:
        pre = deep_prompts.shape[1] if deep_prompts is not None else 0
        for i, blk in enumerate(self.blocks):
            if pre > 0 and hidden.shape[1] >= pre:
                # functional (not in-place) so prompt grads flow in backward
                dp = deep_prompts[i].to(hidden.dtype).unsqueeze(0)
                dp = F.pad(dp, (0, hidden.shape[-1] - dp.shape[-1]))
                hidden = torch.cat([hidden[:, :pre] + dp, hidden[:, pre:]], 1)
            hidden = blk.forward_train(hidden, start_pos)
        return hidden


class LocalEngine:
    """Whole model in one process: greedy decode for bench/tests.

    Client-side pieces (embeddings, final norm, LM head) follow the reference
    client split (client/lm_head.py, models/llama/model.py:80-118).
    """

    def __init__(self, config_or_name, device="cpu", seed: int = 0,
                 kv_max_tokens: int = 1 << 16, quantize_q4: bool = False,
                 checkpoint_dir: Optional[str] = None,
                 max_seqs: Optional[int] = None):
        cfg = (config_or_name if isinstance(config_or_name, ModelConfig)
               else resolve_config(config_or_name))
        # a servable weight folder loads its weights, a preset draws them
        if checkpoint_dir is None and isinstance(config_or_name, str):
            from bloombee_amd.server.from_pretrained import is_servable
            if is_servable(config_or_name):
                checkpoint_dir = config_or_name
        self.config = cfg
        self.device = torch.device(device)
        head_cls = get_family(cfg.model_type).head_cls
        self.head = None
        if head_cls is not None:
            self.head = head_cls(cfg, device=device, seed=seed,
                                 checkpoint_dir=checkpoint_dir)
        else:
            self._init_plain_head(cfg, device, seed, checkpoint_dir)
        self.stack = BlockStack(cfg, 0, cfg.num_hidden_layers, device=device, seed=seed)
        if checkpoint_dir is not None:
            from bloombee_amd.server.from_pretrained import load_block_weights
            for i, blk in enumerate(self.stack.blocks):
                load_block_weights(blk, checkpoint_dir, i)
        if quantize_q4:
            # 4-bit weight-compressed decode (w4_gemm.hip): ~4x less weight
            # memory + HBM traffic. Used for cheap same-weights draft models
            # (speculative decoding) and compressed serving.
            for blk in self.stack.blocks:
                if hasattr(blk, "quantize_weights_q4"):
                    blk.quantize_weights_q4()
        self.kv_pool = self.stack.make_kv(kv_max_tokens, max_seqs)
        self._decode_graphs: Dict[tuple, "_DecodeGraph"] = {}

    def _init_plain_head(self, cfg, device, seed, checkpoint_dir) -> None:
        gen = torch.Generator().manual_seed(seed)
        dt = cfg.dtype
        # family head shape: bloom/falcon use LayerNorm heads; bloom also
        # layer-norms the embedding output (HF word_embeddings_layernorm)
        self.embed_ln = cfg.model_type == "bloom"
        self.ln_final = cfg.model_type in ("bloom", "falcon")
        self.embed_scale = (cfg.hidden_size ** 0.5
                            if cfg.model_type == "gemma4" else 1.0)
        self.embed = (torch.randn(cfg.vocab_size, cfg.hidden_size, generator=gen)
                      .mul_(0.02).to(dt).to(device))
        self.final_norm_w = torch.ones(cfg.hidden_size, dtype=dt, device=device)
        self.final_norm_b = torch.zeros(cfg.hidden_size, dtype=dt, device=device)
        if self.embed_ln:
            self.embed_ln_w = torch.ones(cfg.hidden_size, dtype=dt, device=device)
            self.embed_ln_b = torch.zeros(cfg.hidden_size, dtype=dt, device=device)
        if cfg.tie_word_embeddings:
            self.lm_head_w = self.embed
        else:
            self.lm_head_w = (torch.randn(cfg.vocab_size, cfg.hidden_size, generator=gen)
                              .mul_(0.02).to(dt).to(device))
        if checkpoint_dir is not None:
            from bloombee_amd.server.from_pretrained import load_client_weights
            cw = load_client_weights(checkpoint_dir)
            if cw["embed"] is None or cw["final_norm"] is None:
                raise FileNotFoundError(f"no client weights under {checkpoint_dir}")
            self.embed.copy_(cw["embed"])
            self.final_norm_w.copy_(cw["final_norm"])
            if not cfg.tie_word_embeddings:
                if cw["lm_head"] is None:
                    raise FileNotFoundError(f"no lm_head under {checkpoint_dir}")
                self.lm_head_w.copy_(cw["lm_head"])

    @torch.no_grad()
    def logits_for(self, hidden_last: torch.Tensor) -> torch.Tensor:
        """hidden_last: (B, H) -> (B, V)"""
        if self.head is not None:
            return self.head.logits(self.head.final_norm(hidden_last))
        if self.ln_final:
            y = ops.layer_norm(hidden_last, self.final_norm_w, self.final_norm_b,
                               self.config.layer_norm_epsilon)
        else:
            y = ops.rms_norm(hidden_last, self.final_norm_w, self.config.rms_norm_eps)
        return F.linear(y, self.lm_head_w)

    def _embed(self, input_ids: torch.Tensor,
               start: Optional[torch.Tensor] = None,
               kv: Optional[SessionHandle] = None) -> torch.Tensor:
        """(B, T) ids; start (B,): position of each row's first token (families
        that embed positions only, default 0); kv: the session they continue
        (families that embed pairs of tokens only)."""
        if self.head is not None:
            B, T = input_ids.shape
            input_ids = input_ids.to(self.device)
            prev = None
            if self.head.uses_previous:
                if kv is None:
                    raise NotImplementedError(
                        f"{self.config.model_type}: embeds tokens with the ones "
                        f"before them, which this step does not follow")
                prev = ragged.previous_ids(input_ids, kv.previous(self.device))
                kv.last_ids = input_ids[:, -1].clone()
            pos = torch.arange(T, dtype=torch.int32, device=self.device)
            pos = (pos.expand(B, T) if start is None
                   else start.view(B, 1).int() + pos)
            return self.head.embed(input_ids, pos, prev)
        h = F.embedding(input_ids.to(self.device), self.embed)
        if self.embed_scale != 1.0:
            h = h * self.embed_scale
        if self.embed_ln:
            h = ops.layer_norm(h, self.embed_ln_w, self.embed_ln_b,
                               self.config.layer_norm_epsilon)
        return h

    # -- ragged steps ------------------------------------------------------
    @torch.no_grad()
    def step(self, entries: Sequence[Tuple[SessionHandle, Sequence[int],
                                           Sequence[int]]],
             ) -> torch.Tensor:
        """One step over a mixed batch: entries are (one-sequence session, its
        next tokens, the places among them whose logits are wanted). Returns
        (wanted, V) f32 in the order of the entries. Only the new tokens run;
        each session's cache carries what came before.

        Families without ragged blocks run the entries one after the other."""
        V, limit = self.config.vocab_size, self.config.max_position_embeddings
        need = 0
        P = self.kv_pool.page_size
        for h, toks, want in entries:
            n = len(toks)
            if h.batch_size != 1 or n < 1:
                raise ValueError("an entry is one sequence with new tokens")
            if not all(0 <= t < V for t in toks):
                raise ValueError(f"token id outside [0, {V})")
            if not all(0 <= w < n for w in want):
                raise ValueError("wanted place outside the entry's tokens")
            if h.seqs[0].l_spec + n > min(limit, h.max_length):
                raise ValueError(f"sequence would exceed "
                                 f"{min(limit, h.max_length)} positions")
            need += (h.seqs[0].l_spec + n + P - 1) // P - len(h.seqs[0].pages)
        if len({id(h) for h, _, _ in entries}) != len(entries):
            raise ValueError("a sequence can enter a step once")
        if need > self.kv_pool.free_page_count():
            raise AllocationFailed(
                f"step needs {need} pages, "
                f"{self.kv_pool.free_page_count()} are free")
        for h, toks, _ in entries:
            h.extend(len(toks))
        if self.stack.token_batched:
            batch = session_batch([(h, len(t)) for h, t, _ in entries])
            ids = [t for _, toks, _ in entries for t in toks]
            prev = None
            if self.head.uses_previous:
                prev = [t for h, toks, _ in entries
                        for t in [int(h.previous("cpu")), *toks[:-1]]]
            both = torch.tensor([ids] if prev is None else [ids, prev],
                                dtype=torch.int32).to(self.device)
            hidden = self.stack.forward_batch(
                self.head.embed(both[0], batch.tok_pos,
                                None if prev is None else both[1]), batch)
            for h, toks, _ in entries:
                h.last_ids = [toks[-1]]
        else:
            outs = []
            for h, toks, _ in entries:
                start = torch.tensor([h.seqs[0].l_spec - len(toks)],
                                     dtype=torch.int32, device=self.device)
                ids = torch.tensor([list(toks)])
                outs.append(self.stack.forward_inference(
                    self._embed(ids, start), h, start)[0])
            hidden = torch.cat(outs)
        rows, at = [], 0
        for _, toks, want in entries:
            rows += [at + w for w in want]
            at += len(toks)
        if not rows:
            return torch.empty(0, V, device=self.device)
        idx = torch.tensor(rows, dtype=torch.long).to(self.device)
        return self.logits_for(hidden[idx]).float()

    @torch.no_grad()
    def decode(self, entries: Sequence[Tuple[SessionHandle, int]],
               ) -> torch.Tensor:
        """step() for a batch that brings one token per sequence and wants
        every logit; replays a captured graph where the device allows."""
        from bloombee_amd.config import get_config
        n = len(entries)
        if not (self.stack.token_batched and self.device.type == "cuda"
                and get_config().use_hip_graphs):
            return self.step([(h, [t], [0]) for h, t in entries])
        slots = 1
        while slots < n:
            slots *= 2
        need = max(h.seqs[0].l_spec + 1 for h, _ in entries)
        limit = min(self.config.max_position_embeddings,
                    self.kv_pool.max_tokens)
        if need > limit:
            raise ValueError(f"sequence would exceed {limit} positions")
        g = self._decode_graphs.get(slots)
        if g is None:
            g = self._decode_graphs[slots] = _DecodeGraph(self, slots, limit)
        return g.run(entries)

    @torch.no_grad()
    def prefill(self, input_ids: torch.Tensor, kv: SessionHandle) -> torch.Tensor:
        """input_ids: (B, T). Returns greedy next token ids (B,)."""
        B, T = input_ids.shape
        start = torch.tensor([s.l_spec for s in kv.seqs], dtype=torch.int32,
                             device=self.device)
        kv.extend(T)
        hidden = self._embed(input_ids, start, kv)
        hidden = self.stack.forward_inference(hidden, kv, start)
        return self.logits_for(hidden[:, -1]).argmax(-1)

    @torch.no_grad()
    def decode_step(self, input_ids: torch.Tensor, kv: SessionHandle) -> torch.Tensor:
        """input_ids: (B,) last tokens. Returns next token ids (B,)."""
        start = torch.tensor([s.l_spec for s in kv.seqs], dtype=torch.int32,
                             device=self.device)
        kv.extend(1)
        hidden = self._embed(input_ids.view(-1, 1), start, kv)
        hidden = self.stack.forward_inference(hidden, kv, start)
        return self.logits_for(hidden[:, -1]).argmax(-1)

    @torch.no_grad()
    def generate_greedy(self, input_ids: torch.Tensor, max_new_tokens: int) -> torch.Tensor:
        B, T = input_ids.shape
        if self.stack.token_batched:
            from bloombee_amd.scheduler import BatchScheduler
            sched = BatchScheduler(self)
            reqs = [sched.submit(row, max_new_tokens)
                    for row in input_ids.tolist()]
            sched.run()
            return torch.tensor([r.output for r in reqs], device=self.device)
        kv = self.kv_pool.allocate(B, T + max_new_tokens + 1)
        try:
            toks = [self.prefill(input_ids, kv)]
            for _ in range(max_new_tokens - 1):
                toks.append(self.decode_step(toks[-1], kv))
            return torch.stack(toks, dim=1)
        finally:
            kv.close()

    def make_graphed_decoder(self, kv: SessionHandle):
        """Single-token GREEDY decode step (B=1) as a hipGraph replay
        against a FIXED session handle. The whole step — embed, blocks,
        logits, softmax, (prob, argmax) — is inside the graph; the host
        writes (token, position) into one pinned staging buffer, replays,
        and reads ONE 8-byte pair back. Measured motivation
        (benchmarks/gstep_micro.py): the eager step costs ~350 µs/node
        and even post-replay eager softmax/argmax ops add ~100 µs EACH —
        fatal for small draft models in speculative decoding.

        Returns step(token:int, position:int) -> (next_tok:int,
        prob:float, probs_buffer). probs_buffer is the graph-owned softmax
        output — clone it before the next replay if kept. The caller owns
        kv growth (extend/rollback) BEFORE each step. Falls back to an
        eager closure off-GPU."""
        from bloombee_amd.config import get_config

        on_gpu = (self.device.type == "cuda"
                  and get_config().use_hip_graphs)
        staging = torch.zeros(2, dtype=torch.long,
                              pin_memory=on_gpu)
        dev_in = torch.zeros(2, dtype=torch.long, device=self.device)

        def _body():
            ids = dev_in[0:1].view(1, 1)
            pos = dev_in[1:2].to(torch.int32)
            h = self._embed(ids, pos)
            h = self.stack.forward_inference(h, kv, pos)
            logits = self.logits_for(h[:, -1]).float()
            p = torch.softmax(logits[0], -1)
            pv, ti = p.max(-1)
            return p, torch.stack((ti.to(torch.float32), pv))

        if not on_gpu:
            def step_eager(tok: int, position: int):
                dev_in[0] = tok
                dev_in[1] = position
                p, pair = _body()
                return int(pair[0]), float(pair[1]), p
            return step_eager

        # warm the allocator/kernels, then capture (thread_local keeps other
        # threads' work — e.g. the channels pump — legal during capture)
        for _ in range(2):
            kv.extend(1, speculative=True)
            kv.page_table()
            _body()
            kv.rollback()
        graph = torch.cuda.CUDAGraph()
        kv.extend(1, speculative=True)
        kv.page_table()
        with torch.cuda.graph(graph, capture_error_mode="thread_local"):
            p_buf, pair_buf = _body()
        kv.rollback()
        pair_host = torch.zeros(2, dtype=torch.float32, pin_memory=True)

        def step(tok: int, position: int):
            staging[0] = tok
            staging[1] = position
            dev_in.copy_(staging, non_blocking=True)
            kv.page_table()  # flush any new page ids
            graph.replay()
            pair_host.copy_(pair_buf, non_blocking=False)  # syncs
            return int(pair_host[0]), float(pair_host[1]), p_buf

        return step

    def make_graphed_chain(self, kv: SessionHandle, depth: int):
        """A whole greedy draft CHAIN (depth single-token steps, each step's
        argmax fed on-device into the next embed) as ONE hipGraph replay —
        one host round-trip per drafting round instead of per node (the
        per-node graphed step still costs ~150 µs of host floor,
        benchmarks/gstep_micro.py).

        Caller per round: rollback, extend(depth, speculative=True),
        page_table(), then chain(token, position0) -> (tokens[depth],
        probs[depth]) on the host. Off-GPU returns None (callers fall back
        to per-node stepping)."""
        from bloombee_amd.config import get_config

        if self.device.type != "cuda" or not get_config().use_hip_graphs:
            return None
        staging = torch.zeros(2, dtype=torch.long, pin_memory=True)
        dev_in = torch.zeros(2, dtype=torch.long, device=self.device)
        out_host = torch.zeros(2, depth, dtype=torch.float32, pin_memory=True)

        def _body():
            toks = torch.zeros(depth, dtype=torch.float32,
                               device=self.device)
            prbs = torch.zeros(depth, dtype=torch.float32,
                               device=self.device)
            cur = dev_in[0:1]
            pos0 = dev_in[1:2]
            for i in range(depth):
                sp = (pos0 + i).to(torch.int32)
                h = self._embed(cur.view(1, 1), sp)
                h = self.stack.forward_inference(h, kv, sp)
                logits = self.logits_for(h[:, -1]).float()
                p = torch.softmax(logits[0], -1)
                pv, ti = p.max(-1)
                toks[i] = ti.to(torch.float32)
                prbs[i] = pv
                cur = ti.view(1)
            return torch.stack((toks, prbs))

        for _ in range(2):  # allocator/kernel warmup
            kv.extend(depth, speculative=True)
            kv.page_table()
            _body()
            kv.rollback()
        graph = torch.cuda.CUDAGraph()
        kv.extend(depth, speculative=True)
        kv.page_table()
        with torch.cuda.graph(graph, capture_error_mode="thread_local"):
            out_buf = _body()
        kv.rollback()

        def chain(tok: int, position0: int):
            staging[0] = tok
            staging[1] = position0
            dev_in.copy_(staging, non_blocking=True)
            kv.page_table()
            graph.replay()
            out_host.copy_(out_buf, non_blocking=False)  # syncs
            return ([int(t) for t in out_host[0]],
                    [float(p) for p in out_host[1]])

        return chain


class _DecodeGraph:
    """A captured decode step for up to `slots` sequences: embedding, blocks,
    norm and logits replay against the buffers of one DecodeSlots."""

    WARMUP = 2

    def __init__(self, engine: LocalEngine, slots: int, limit: int):
        self.engine = engine
        self.slots = DecodeSlots(engine.kv_pool, slots, limit)
        self.graph = None
        self.calls = 0
        self.logits: Optional[torch.Tensor] = None

    def _body(self) -> torch.Tensor:
        eng, b = self.engine, self.slots.batch
        x = eng.stack.forward_batch(
            eng.head.embed(self.slots.ids, b.tok_pos, self.slots.prev), b)
        return eng.logits_for(x)

    def run(self, entries) -> torch.Tensor:
        """The result is the graph's buffer: used up before the next call."""
        for h, _ in entries:
            h.extend(1)
        seqs = [h.seqs[0] for h, _ in entries]
        prev = ([int(h.previous("cpu")) for h, _ in entries]
                if self.engine.head.uses_previous else None)
        self.slots.fill([t for _, t in entries], [s.l_spec - 1 for s in seqs],
                        [s.pages for s in seqs], [s.slot for s in seqs], prev)
        for h, t in entries:
            h.last_ids = [t]
        n = len(entries)
        if self.graph is None and self.calls < self.WARMUP:
            self.calls += 1
            return self._body()[:n]
        if self.graph is None:
            self.graph = torch.cuda.CUDAGraph()
            with torch.cuda.graph(self.graph,
                                  capture_error_mode="thread_local"):
                self.logits = self._body()
            logger.info("ragged decode step of %d slots captured as hipGraph",
                        self.slots.B)
        self.graph.replay()
        return self.logits[:n]
