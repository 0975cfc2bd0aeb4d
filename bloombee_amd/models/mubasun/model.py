"""Client side of the Mubasun family: learned positions and a grouped final
norm (models/ragged_head.py)."""
from __future__ import annotations

from bloombee_amd.models.ragged_head import (DistributedRaggedForCausalLM,
                                             DistributedRaggedModel,
                                             RaggedHead)


class MubasunHead(RaggedHead):
    pass


class DistributedMubasunModel(DistributedRaggedModel):
    head_cls = MubasunHead


class DistributedMubasunForCausalLM(DistributedRaggedForCausalLM):
    model_cls = DistributedMubasunModel
