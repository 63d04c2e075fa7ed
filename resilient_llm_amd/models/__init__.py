from .llama import LlamaConfig, LlamaForCausalLM, MODEL_PRESETS  # noqa: F401
from .bolatar import BolatarConfig, BolatarForCausalLM  # noqa: F401
from .fimunex import FimunexConfig, FimunexForCausalLM  # noqa: F401
from .nesizen import NesizenConfig, NesizenForCausalLM  # noqa: F401
from .riruzen import RiruzenConfig, RiruzenForCausalLM  # noqa: F401
from .registry import (  # noqa: F401
    build_model, checkpoint_architecture, get_config, get_model_class,
    model_names,
)
