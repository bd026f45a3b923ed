"""Architectures: name -> configuration class and model assembly."""

from .registry import (ArchitectureEntry, architecture_of, architectures, assemble, read_config, read_model_dir,
                       register_architecture, unregister_architecture)
from . import minimax_m3  # noqa: F401  (registers MiniMaxM3ForCausalLM)
from . import nenotar  # noqa: F401  (registers Nenotar)
from . import bonerax  # noqa: F401  (registers Bonerax)
from . import givozen  # noqa: F401  (registers Givozen)
from . import salipel  # noqa: F401  (registers Salipel)
from . import neruzen  # noqa: F401  (registers Neruzen)
from . import vivulorn  # noqa: F401  (registers Vivulorn)

__all__ = ["ArchitectureEntry", "architecture_of", "architectures", "assemble", "read_config", "read_model_dir",
           "register_architecture", "unregister_architecture"]
