from .base import (ConfigError, Architecture, register_architecture, unregister_architecture,
                   registered_architectures, architecture_of, read_config_json, config_from_folder)
from .llama import LlamaConfig
from .novosun import NovosunConfig
from .ditazen import DitazenConfig
from .noresun import NoresunConfig
from .zovozen import ZovozenConfig
from .guduzen import GuduzenConfig
from .movazen import MovazenConfig
from .presets import preset, preset_names
