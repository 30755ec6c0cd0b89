from neuronx_distributed_inference_amd.models.sitidra.modeling_sitidra import (  # noqa: F401
    SitidraForCausalLM,
    SitidraInferenceConfig,
)
