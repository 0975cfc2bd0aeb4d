from bloombee_amd.models.base import FamilyEntry, register_model_family
from bloombee_amd.models.zatusun.block import ZatusunBlock  # noqa: F401
from bloombee_amd.models.zatusun.config import (  # noqa: F401
    ZATUSUN_PRESETS,
    ZatusunConfig,
)
from bloombee_amd.models.zatusun.model import (  # noqa: F401
    DistributedZatusunForCausalLM,
    DistributedZatusunModel,
    ZatusunHead,
)

register_model_family(
    "zatusun",
    FamilyEntry(config_cls=ZatusunConfig, block_cls=ZatusunBlock,
                model_cls=DistributedZatusunModel,
                causal_lm_cls=DistributedZatusunForCausalLM,
                head_cls=ZatusunHead, architecture="Zatusun",
                presets=ZATUSUN_PRESETS),
)
