"""Model definitions hosted by the inference engine: random-init presets (no
network for checkpoints; the benchmark measures architecture-shaped compute,
reference) and checkpoint folders."""

from .config import ModelConfig, get_config, PRESETS  # noqa: F401
from .hybrid import KoridraModel, KotutarModel  # noqa: F401
from .llama import LlamaModel  # noqa: F401

# architecture of a config -> model class
MODEL_CLASSES = {"Llama": LlamaModel, "Koridra": KoridraModel,
                 "Kotutar": KotutarModel}


def build_model(key, device, dtype=None, tp=None):
    """The model of a key, by the architecture of its config."""
    import torch
    return MODEL_CLASSES[get_config(key).architecture](
        key, device, dtype=dtype or torch.bfloat16, tp=tp)
