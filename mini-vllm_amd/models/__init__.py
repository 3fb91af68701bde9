from .registry import (Architecture, config_from_dict, get_architecture, load_config, register_architecture,
                       registered_architectures, unregister_architecture)
from . import qwen3  # registers "Qwen3ForCausalLM"
from . import bolapel  # registers "Bolapel"
from . import dutilix  # registers "Dutilix"
from . import zedudra  # registers "Zedudra"
from . import furanex  # registers "Furanex"
from . import sorulix  # registers "Sorulix"
from . import setirax  # registers "Setirax"
from .causal_lm import CausalLM, expected_tensors
