"""Model registry: the architecture a config.json names -> (configuration reader, model class)."""
import warnings

from ..utils.loader import Checkpoint, read_config


def _zobasun():
    from .zobasun import ZobasunConfig, ZobasunForCausalLM
    return ZobasunConfig.from_json, ZobasunForCausalLM


def _galirax():
    from .galirax import GaliraxConfig, GaliraxForCausalLM
    return GaliraxConfig.from_json, GaliraxForCausalLM


def _kekapel():
    from .kekapel import KekapelConfig, KekapelForCausalLM
    return KekapelConfig.from_json, KekapelForCausalLM


def _zaposun():
    from .zaposun import ZaposunConfig, ZaposunForCausalLM
    return ZaposunConfig.from_json, ZaposunForCausalLM


def _qwen():
    from .qwen import ModelConfig, QwenForCausalLM
    return ModelConfig.from_json, QwenForCausalLM


REGISTRY = {"Zobasun": _zobasun, "Galirax": _galirax, "Kekapel": _kekapel, "Zaposun": _zaposun, "Qwen2ForCausalLM": _qwen, "Qwen3ForCausalLM": _qwen}


def architecture(config_json):
    name = config_json.get("architecture") or (config_json.get("architectures") or [None])[0]
    if name not in REGISTRY:
        raise ValueError(f"unknown architecture {name!r}; known: {', '.join(sorted(REGISTRY))}")
    return name


def load_config(path, **overrides):
    """Configuration object of a model folder; overrides set fields of it (dtype, kvcache_block_size, ...)."""
    d = read_config(path)
    return REGISTRY[architecture(d)]()[0](d, **overrides)


def model_class(cfg):
    from .galirax import GaliraxConfig, GaliraxForCausalLM
    from .kekapel import KekapelConfig, KekapelForCausalLM
    from .qwen import ModelConfig, QwenForCausalLM
    from .zaposun import ZaposunConfig, ZaposunForCausalLM
    from .zobasun import ZobasunConfig, ZobasunForCausalLM
    return {ModelConfig: QwenForCausalLM, ZobasunConfig: ZobasunForCausalLM, GaliraxConfig: GaliraxForCausalLM,
            KekapelConfig: KekapelForCausalLM, ZaposunConfig: ZaposunForCausalLM}[type(cfg)]


def build_model(cfg, path=None, seed=0):
    """The model of a configuration with the weights of the folder `path`, or random ones."""
    model = model_class(cfg)(cfg)
    if path is None:
        return model.init_random(seed)
    ckpt = Checkpoint(path)
    model.load_weights(ckpt)
    if ckpt.unread():
        warnings.warn(f"checkpoint tensors no layer of the configuration reads: {', '.join(ckpt.unread()[:8])}")
    return model
