from .durelix import DurelixConfig
from .fubelorn import FubelornConfig
from .gokolix import GokolixConfig
from .larupel import LarupelConfig
from .llama import Llama3RopeScaling, LlamaConfig, UnsupportedModelError
from .radivik import RadivikConfig
from .registry import (Architecture, UnknownArchitectureError, architecture_of, read_model_dir,
                       register_architecture, registered_architectures)
from .zurolorn import ZurolornConfig

__all__ = [
    "Architecture", "DurelixConfig", "FubelornConfig", "GokolixConfig", "LarupelConfig", "Llama3RopeScaling", "LlamaConfig", "RadivikConfig", "UnknownArchitectureError", "UnsupportedModelError",
    "ZurolornConfig",
    "architecture_of", "read_model_dir", "register_architecture", "registered_architectures",
]
