from .base import (BlockSpec, ConfigError, JsonReader, LayerCall, ModelSpec, PartSpec,
                   read_config_json)
from .qwen3 import Qwen3Config
from .defosun import DefosunConfig
from .kosusun import KosusunConfig
from .kunitar import KunitarConfig
from .gimipel import GimipelConfig
from .kapanex import KapanexConfig
from .sinepel import SinepelConfig

__all__ = ["BlockSpec", "ConfigError", "JsonReader", "LayerCall", "ModelSpec", "PartSpec",
           "read_config_json", "Qwen3Config", "SinepelConfig", "KapanexConfig", "GimipelConfig", "DefosunConfig",
           "KosusunConfig", "KunitarConfig"]
