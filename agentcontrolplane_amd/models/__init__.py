from .fetolix import FetolixForCausalLM  # noqa: F401
from .llama import LlamaForCausalLM  # noqa: F401
from .lobuvik import LobuvikForCausalLM  # noqa: F401
from .mixtral import MixtralForCausalLM  # noqa: F401
from .noganex import NoganexForCausalLM  # noqa: F401
from .tezinex import TezinexForCausalLM  # noqa: F401

#: ModelConfig.architecture -> model class
MODEL_CLASSES = {
    "llama": LlamaForCausalLM,
    "mixtral": MixtralForCausalLM,
    "Fetolix": FetolixForCausalLM,
    "Tezinex": TezinexForCausalLM,
    "Lobuvik": LobuvikForCausalLM,
    "Noganex": NoganexForCausalLM,
}


def create_model(model_config, engine_config, device, tp_rank: int = 0, tp_world: int = 1):
    arch = model_config.architecture or ("mixtral" if model_config.is_moe else "llama")
    if arch not in MODEL_CLASSES:
        raise KeyError(f"unknown architecture {arch!r}; have {sorted(MODEL_CLASSES)}")
    return MODEL_CLASSES[arch](model_config, engine_config, device, tp_rank, tp_world)
