"""Client side of the Risepel family: embeddings without positions, a final
norm that scales by one plus its stored weight, capped logits
(models/ragged_head.py)."""
from __future__ import annotations

from bloombee_amd.models.ragged_head import (DistributedRaggedForCausalLM,
                                             DistributedRaggedModel,
                                             RaggedHead)


class RisepelHead(RaggedHead):
    pass


class DistributedRisepelModel(DistributedRaggedModel):
    head_cls = RisepelHead


class DistributedRisepelForCausalLM(DistributedRaggedForCausalLM):
    model_cls = DistributedRisepelModel
