from .base import ConfigError, UnsupportedArchitecture, architecture_name, read_config_json
from .qwen3 import Qwen3Config
from .pamevik import PamevikConfig
from .zukinex import ZukinexConfig
from .fosulix import FosulixConfig
from .nogidra import NogidraConfig
from .reverax import ReveraxConfig
from .sonulorn import SonulornConfig
