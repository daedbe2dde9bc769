from gridllm_amd.models.registry import (HybridSpec, ModelSpec,  # noqa: F401
                                         get_spec, list_specs)


def model_class(spec):
    """The class that runs a spec."""
    if isinstance(spec, HybridSpec):
        from gridllm_amd.models.hybrid import HybridModel
        return HybridModel
    from gridllm_amd.models.llama import LlamaModel
    return LlamaModel
