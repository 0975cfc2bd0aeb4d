from bloombee_amd.models.base import FamilyEntry, register_model_family
from bloombee_amd.models.risepel.block import RisepelBlock  # noqa: F401
from bloombee_amd.models.risepel.config import (  # noqa: F401
    RISEPEL_PRESETS,
    RisepelConfig,
)
from bloombee_amd.models.risepel.model import (  # noqa: F401
    DistributedRisepelForCausalLM,
    DistributedRisepelModel,
    RisepelHead,
)

register_model_family(
    "risepel",
    FamilyEntry(config_cls=RisepelConfig, block_cls=RisepelBlock,
                model_cls=DistributedRisepelModel,
                causal_lm_cls=DistributedRisepelForCausalLM,
                head_cls=RisepelHead, architecture="Risepel",
                presets=RISEPEL_PRESETS),
)
