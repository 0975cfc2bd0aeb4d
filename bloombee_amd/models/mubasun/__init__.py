from bloombee_amd.models.base import FamilyEntry, register_model_family
from bloombee_amd.models.mubasun.block import MubasunBlock  # noqa: F401
from bloombee_amd.models.mubasun.config import (  # noqa: F401
    MUBASUN_PRESETS,
    MubasunConfig,
)
from bloombee_amd.models.mubasun.model import (  # noqa: F401
    DistributedMubasunForCausalLM,
    DistributedMubasunModel,
    MubasunHead,
)

register_model_family(
    "mubasun",
    FamilyEntry(config_cls=MubasunConfig, block_cls=MubasunBlock,
                model_cls=DistributedMubasunModel,
                causal_lm_cls=DistributedMubasunForCausalLM,
                head_cls=MubasunHead, architecture="Mubasun",
                presets=MUBASUN_PRESETS),
)
