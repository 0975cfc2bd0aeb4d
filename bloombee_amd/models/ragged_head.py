"""Client side of the ragged-batch families: token (and learned position)
embeddings, final norm and vocabulary projection as one module, shared by
LocalEngine, the pipeline and the swarm client, and the distributed model
classes over it.

What differs between families are properties of the config: `embedding_scale`
(of the token's row), `learned_positions` (a table "pos" is added to the
embedding), `hidden_columns` (a multiple of the width: the embedding output
travels behind the residual), `sinusoidal_positions`, `bigram` (a
table "bigram" of hashed token pairs is added: buckets, mul_prev, mul_cur),
`norm_groups`, `norm_offset` (norm weights are stored as their distance from it),
`scalar_norm` (one norm weight for all coordinates), `logit_softcap` (0 = none).
"""
from __future__ import annotations

from typing import Optional

import torch
import torch.nn.functional as F

from bloombee_amd.client.sequential import RemoteSequential
from bloombee_amd.models.base import ModelConfig
from bloombee_amd.models.llama.model import (DistributedLlamaForCausalLM,
                                             DistributedLlamaModel)
from bloombee_amd.ops import ragged
from bloombee_amd.ops.ragged import PairTable, pad_k, round_up


class RaggedHead(torch.nn.Module):
    """What surrounds the blocks. Hidden states are 32-bit."""

    def __init__(self, config: ModelConfig, device="cpu", seed: int = 0,
                 checkpoint_dir: Optional[str] = None):
        super().__init__()
        self.config = config
        self.groups = getattr(config, "norm_groups", 1)
        self.norm_offset = getattr(config, "norm_offset", 0.0)
        self.softcap = getattr(config, "logit_softcap", 0.0)
        self.embed_scale = getattr(config, "embedding_scale", 1.0)
        self.copies = config.hidden_columns // config.hidden_size
        W, V, dt = config.hidden_size, config.vocab_size, config.dtype

        def p(*shape, dtype=dt):
            return torch.nn.Parameter(
                torch.zeros(*shape, dtype=dtype, device=device),
                requires_grad=False)

        self.embed_w = p(V, W)
        self.pos_w = (p(config.max_position_embeddings, W)
                      if getattr(config, "learned_positions", False) else None)
        pair = getattr(config, "bigram", None)
        self.pair_w = p(pair["buckets"] + 1, W) if pair else None
        self.pairs = (PairTable(self.pair_w, pair["mul_prev"], pair["mul_cur"])
                      if pair else None)
        self.turns = None
        if getattr(config, "sinusoidal_positions", False):
            self.turns = torch.nn.Parameter(
                ragged.sinusoid_turns(W).to(device), requires_grad=False)
        self.scalar_norm = getattr(config, "scalar_norm", False)
        self.norm_w = p(W, dtype=torch.float32)
        self.head_w = p(round_up(V, 64), pad_k(W))   # zero padding
        if checkpoint_dir is not None:
            from bloombee_amd.server.from_pretrained import NativeCheckpoint
            self.load_tensors(NativeCheckpoint(checkpoint_dir).get)
        else:
            gen = torch.Generator().manual_seed(seed)
            draw = {"embed": (V, W), "head": (V, W)}
            if self.pos_w is not None:
                draw["pos"] = tuple(self.pos_w.shape)
            if self.pair_w is not None:
                draw["bigram"] = tuple(self.pair_w.shape)
            ts = {n: torch.randn(s, generator=gen).mul_(0.02)
                  for n, s in draw.items()}
            ts["final.norm"] = torch.full(() if self.scalar_norm else (W,),
                                          1.0 - self.norm_offset)
            self.load_tensors(ts.__getitem__)

    @torch.no_grad()
    def load_tensors(self, get) -> None:
        W, V = self.config.hidden_size, self.config.vocab_size
        for name, w in (("embed", self.embed_w), ("pos", self.pos_w),
                        ("bigram", self.pair_w), ("final.norm", self.norm_w),
                        ("head", self.head_w[:V, :W])):
            if w is None:
                continue
            t = get(name)
            one = name == "final.norm" and self.scalar_norm
            if t.shape != (() if one else w.shape):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, expected "
                                 f"{() if one else tuple(w.shape)}")
            w.copy_(t)
        self.norm_w.add_(self.norm_offset)

    @property
    def uses_previous(self) -> bool:
        """embed() needs the token before each."""
        return self.pairs is not None

    def embed(self, ids: torch.Tensor, positions: torch.Tensor,
              prev: Optional[torch.Tensor] = None) -> torch.Tensor:
        """ids, positions of one shape -> (..., columns) f32; prev: the token before
        each, -1 = none (only if uses_previous)."""
        if self.uses_previous and prev is None:
            raise ValueError("this family embeds tokens with the ones before "
                             "them: they are missing")
        return ragged.embed_rows(ids, positions, self.embed_w, self.pos_w, prev,
                                 self.pairs, self.turns, self.embed_scale,
                                 self.copies)

    def final_norm(self, hidden: torch.Tensor) -> torch.Tensor:
        W = self.config.hidden_size
        x = hidden.reshape(-1, hidden.shape[-1]).float()[:, :W]
        h = ragged.residual_norm(x, None, self.norm_w, self.groups,
                                 self.config.rms_norm_eps, self.head_w.shape[1],
                                 self.head_w.dtype)
        return h.view(*hidden.shape[:-1], -1)

    def logits(self, normed: torch.Tensor) -> torch.Tensor:
        """(..., V) f32 from final_norm's output."""
        y = ragged.linear_f32(normed.reshape(-1, normed.shape[-1]), self.head_w)
        if self.softcap:
            y = ragged.softcap_(y, self.softcap)
        return y[:, :self.config.vocab_size].reshape(
            *normed.shape[:-1], self.config.vocab_size)

    # differentiable forms (fine-tuning)
    def train_norm(self, hidden: torch.Tensor) -> torch.Tensor:
        from bloombee_amd.ops.reference import grouped_rms_norm
        hidden = hidden[..., :self.config.hidden_size]
        y = grouped_rms_norm(hidden, self.norm_w, self.groups,
                             self.config.rms_norm_eps).to(self.head_w.dtype)
        return F.pad(y, (0, self.head_w.shape[1] - y.shape[-1]))

    def train_logits(self, normed: torch.Tensor) -> torch.Tensor:
        y = F.linear(normed, self.head_w)[..., :self.config.vocab_size]
        if self.softcap:
            y = self.softcap * torch.tanh(y.float() / self.softcap)
        return y


class DistributedRaggedModel(DistributedLlamaModel):
    head_cls = RaggedHead

    def __init__(self, config: ModelConfig, client_config, model_name: str,
                 seed: int = 0, device: str = "cpu", manager=None,
                 pre_seq_len: int = 0, deep_ptune: bool = False,
                 checkpoint_dir: Optional[str] = None):
        torch.nn.Module.__init__(self)
        self.config = config
        self.device_ = torch.device(device)
        self.checkpoint_dir = checkpoint_dir
        self.head = self.head_cls(config, device=device, seed=seed,
                                  checkpoint_dir=checkpoint_dir)
        self.remote = RemoteSequential(client_config, model_name,
                                       config.num_hidden_layers,
                                       manager=manager)
        self.pre_seq_len = pre_seq_len
        self.prompt_embeds = self.deep_prompts = None
        if pre_seq_len > 0:
            self.prompt_embeds = torch.nn.Parameter(
                torch.randn(pre_seq_len, config.hidden_size, device=device)
                .mul_(0.02))
            if deep_ptune:
                self.deep_prompts = torch.nn.Parameter(
                    torch.zeros(config.num_hidden_layers, pre_seq_len,
                                config.hidden_size, device=device))

    @property
    def uses_previous(self) -> bool:
        return self.head.uses_previous

    def prompt_hidden(self, like: torch.Tensor) -> torch.Tensor:
        p = super().prompt_hidden(like)
        return torch.cat([p] * self.head.copies, -1)

    def embed(self, input_ids: torch.Tensor, start_pos: int = 0,
              last: Optional[torch.Tensor] = None) -> torch.Tensor:
        """last (B,): the token before each row's first, None = there is none."""
        B, T = input_ids.shape
        ids = input_ids.to(self.device_)
        pos = torch.arange(start_pos, start_pos + T, dtype=torch.int32,
                           device=self.device_).expand(B, T)
        prev = None
        if self.uses_previous:
            prev = ragged.previous_ids(
                ids, torch.full((B,), -1) if last is None else last)
        return self.head.embed(ids, pos, prev)

    def final_norm(self, hidden: torch.Tensor) -> torch.Tensor:
        if hidden.requires_grad:
            return self.head.train_norm(hidden)
        return self.head.final_norm(hidden.to(self.device_))


class _LMHead(torch.nn.Module):
    def __init__(self, head: RaggedHead):
        super().__init__()
        self.head = head

    def forward(self, normed: torch.Tensor) -> torch.Tensor:
        if normed.requires_grad:
            return self.head.train_logits(normed)
        return self.head.logits(normed)


class DistributedRaggedForCausalLM(DistributedLlamaForCausalLM):
    model_cls = DistributedRaggedModel

    def __init__(self, config, client_config, model_name, seed=0, device="cpu",
                 manager=None, pre_seq_len=0, deep_ptune=False,
                 checkpoint_dir=None):
        torch.nn.Module.__init__(self)
        self.config = config
        self.transformer = self.model_cls(
            config, client_config, model_name, seed=seed, device=device,
            manager=manager, pre_seq_len=pre_seq_len, deep_ptune=deep_ptune,
            checkpoint_dir=checkpoint_dir)
        self.lm_head = _LMHead(self.transformer.head)
