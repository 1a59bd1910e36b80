from petals_amd.models import register_block
from petals_amd.models.tulezen.block import TulezenBlock
from petals_amd.models.tulezen.config import TulezenConfig

register_block("tulezen")(TulezenBlock)


def _register_models():
    from petals_amd.models.tulezen.model import (
        DistributedTulezenForCausalLM,
        DistributedTulezenForSequenceClassification,
        DistributedTulezenModel,
    )
    from petals_amd.utils import auto_config

    auto_config.register_model_classes(
        "tulezen",
        config=TulezenConfig,
        model=DistributedTulezenModel,
        model_for_causal_lm=DistributedTulezenForCausalLM,
        model_for_sequence_classification=DistributedTulezenForSequenceClassification,
    )
