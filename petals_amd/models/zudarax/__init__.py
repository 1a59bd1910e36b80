from petals_amd.models import register_block
from petals_amd.models.zudarax.block import ZudaraxBlock
from petals_amd.models.zudarax.config import ZudaraxConfig

register_block("zudarax")(ZudaraxBlock)


def _register_models():
    from petals_amd.models.zudarax.model import (
        DistributedZudaraxForCausalLM,
        DistributedZudaraxForSequenceClassification,
        DistributedZudaraxModel,
    )
    from petals_amd.utils import auto_config

    auto_config.register_model_classes(
        "zudarax",
        config=ZudaraxConfig,
        model=DistributedZudaraxModel,
        model_for_causal_lm=DistributedZudaraxForCausalLM,
        model_for_sequence_classification=DistributedZudaraxForSequenceClassification,
    )
