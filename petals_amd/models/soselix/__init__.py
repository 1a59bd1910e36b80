from petals_amd.models import register_block
from petals_amd.models.soselix.block import SoselixBlock
from petals_amd.models.soselix.config import SoselixConfig

register_block("soselix")(SoselixBlock)


def _register_models():
    from petals_amd.models.soselix.model import (
        DistributedSoselixForCausalLM,
        DistributedSoselixForSequenceClassification,
        DistributedSoselixModel,
    )
    from petals_amd.utils import auto_config

    auto_config.register_model_classes(
        "soselix",
        config=SoselixConfig,
        model=DistributedSoselixModel,
        model_for_causal_lm=DistributedSoselixForCausalLM,
        model_for_sequence_classification=DistributedSoselixForSequenceClassification,
    )
