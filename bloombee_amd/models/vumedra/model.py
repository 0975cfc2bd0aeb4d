"""Client side of the Vumedra family: embeddings of tokens, token pairs and
sinusoidal positions, a final norm with one weight (models/ragged_head.py)."""
from __future__ import annotations

from bloombee_amd.models.ragged_head import (DistributedRaggedForCausalLM,
                                             DistributedRaggedModel,
                                             RaggedHead)


class VumedraHead(RaggedHead):
    pass


class DistributedVumedraModel(DistributedRaggedModel):
    head_cls = VumedraHead


class DistributedVumedraForCausalLM(DistributedRaggedForCausalLM):
    model_cls = DistributedVumedraModel
