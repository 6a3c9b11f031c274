from .configs import HybridConfig, ModelConfig, get_model_config, MODEL_PRESETS
from .hybrid import HybridModel
from .llama import LlamaModel

# configuration class -> the model that runs it
MODEL_CLASSES = {ModelConfig: LlamaModel, HybridConfig: HybridModel}


def build_model(config, **kwargs):
    """The model of a configuration (kwargs: device, dtype, seed and the
    tensor-parallel placement)."""
    return MODEL_CLASSES[type(config)](config, **kwargs)


__all__ = [
    "ModelConfig", "HybridConfig", "get_model_config", "MODEL_PRESETS",
    "LlamaModel", "HybridModel", "MODEL_CLASSES", "build_model",
]
