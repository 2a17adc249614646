"""Model registry: config.json -> model class."""
import json
import os

from .berevik import BerevikForCausalLM
from .gopunex import GopunexForCausalLM
from .lefalix import LefalixForCausalLM
from .qwen3 import Qwen3ForCausalLM
from .tafopel import TafopelForCausalLM

MODELS = {
    "Berevik": BerevikForCausalLM,
    "Gopunex": GopunexForCausalLM,
    "Lefalix": LefalixForCausalLM,
    "Qwen3ForCausalLM": Qwen3ForCausalLM,
    "Tafopel": TafopelForCausalLM,
}


def architecture(config):
    """architecture name of a config.json dictionary: `architecture`, else the first of HF's `architectures`, else model_type"""
    if config.get("architecture"):
        return config["architecture"]
    if config.get("architectures"):
        return config["architectures"][0]
    if config.get("model_type") == "qwen3":
        return "Qwen3ForCausalLM"
    raise RuntimeError("config.json names no architecture")


def model_class(model_dir):
    path = os.path.join(model_dir, "config.json")
    try:
        with open(path) as f:
            name = architecture(json.load(f))
    except OSError as e:
        raise RuntimeError(f"Failed to read config {path}: {e}") from e
    except json.JSONDecodeError as e:
        raise RuntimeError(f"Failed to parse config {path}: {e}") from e
    if name not in MODELS:
        raise RuntimeError(f"architecture {name!r} unknown (known: {', '.join(sorted(MODELS))})")
    return MODELS[name]


def load_model(model_dir, ctx=None, dtype="bfloat16"):
    """the model of a checkpoint directory, on the class its config.json names"""
    return model_class(model_dir).from_dir(model_dir, ctx, dtype)
