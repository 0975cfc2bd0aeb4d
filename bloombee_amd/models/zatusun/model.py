"""Client side of the Zatusun family: scaled embeddings with learned positions, a
final norm that scales by one plus its stored weight, capped logits
(models/ragged_head.py)."""
from __future__ import annotations

from bloombee_amd.models.ragged_head import (DistributedRaggedForCausalLM,
                                             DistributedRaggedModel,
                                             RaggedHead)


class ZatusunHead(RaggedHead):
    pass


class DistributedZatusunModel(DistributedRaggedModel):
    head_cls = ZatusunHead


class DistributedZatusunForCausalLM(DistributedRaggedForCausalLM):
    model_cls = DistributedZatusunModel
