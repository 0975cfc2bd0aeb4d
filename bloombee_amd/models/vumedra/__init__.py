from bloombee_amd.models.base import FamilyEntry, register_model_family
from bloombee_amd.models.vumedra.block import VumedraBlock  # noqa: F401
from bloombee_amd.models.vumedra.config import (  # noqa: F401
    VUMEDRA_PRESETS,
    VumedraConfig,
)
from bloombee_amd.models.vumedra.model import (  # noqa: F401
    DistributedVumedraForCausalLM,
    DistributedVumedraModel,
    VumedraHead,
)

register_model_family(
    "vumedra",
    FamilyEntry(config_cls=VumedraConfig, block_cls=VumedraBlock,
                model_cls=DistributedVumedraModel,
                causal_lm_cls=DistributedVumedraForCausalLM,
                head_cls=VumedraHead, architecture="Vumedra",
                presets=VUMEDRA_PRESETS),
)
