from tokensprint_amd.models import (fubepel, palelix, pinedra, qwen3, sisepel,  # noqa: F401
                                    zolorax, zonopel)           # (register the architectures)
from tokensprint_amd.models.model import Model
from tokensprint_amd.models.spec import LayerSpec, ModelSpec, PartSpec, Run

__all__ = ["Model", "LayerSpec", "ModelSpec", "PartSpec", "Run"]
