"""Model classes by architecture."""

from fei_amd.models.bokenex import BokenexModel
from fei_amd.models.llama import LlamaModel
from fei_amd.models.tobarax import TobaraxModel

MODEL_CLASSES = {"llama": LlamaModel, "tobarax": TobaraxModel,
                 "bokenex": BokenexModel}


def model_class(spec):
    """The decoder class that runs ``spec``."""
    try:
        return MODEL_CLASSES[spec.arch]
    except KeyError:
        raise ValueError(f"{spec.name}: no decoder for architecture "
                         f"{spec.arch!r}") from None


__all__ = ["BokenexModel", "LlamaModel", "MODEL_CLASSES", "TobaraxModel", "model_class"]
