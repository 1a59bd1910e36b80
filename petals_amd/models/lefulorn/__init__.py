from petals_amd.models import register_block
from petals_amd.models.lefulorn.block import LefulornBlock
from petals_amd.models.lefulorn.config import LefulornConfig

register_block("lefulorn")(LefulornBlock)


def _register_models():
    from petals_amd.models.lefulorn.model import (
        DistributedLefulornForCausalLM,
        DistributedLefulornForSequenceClassification,
        DistributedLefulornModel,
    )
    from petals_amd.utils import auto_config

    auto_config.register_model_classes(
        "lefulorn",
        config=LefulornConfig,
        model=DistributedLefulornModel,
        model_for_causal_lm=DistributedLefulornForCausalLM,
        model_for_sequence_classification=DistributedLefulornForSequenceClassification,
    )
