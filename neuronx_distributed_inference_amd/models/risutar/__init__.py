from neuronx_distributed_inference_amd.models.risutar.modeling_risutar import (  # noqa: F401
    RisutarForCausalLM,
    RisutarInferenceConfig,
)
