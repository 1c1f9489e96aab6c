"""Model families by the name a `config.json` gives: `model_type` or `architecture`."""

from __future__ import annotations

from typing import Tuple

from . import checkpoint
from .config import GitipelConfig, GupitarConfig, RavenConfig
from .gitipel import GitipelForCausalLM
from .gupitar import GupitarForCausalLM
from .modeling import RavenForCausalLM

FAMILIES = {
    "huginn_raven": (RavenConfig, RavenForCausalLM),
    "gitipel": (GitipelConfig, GitipelForCausalLM),
    "gupitar": (GupitarConfig, GupitarForCausalLM),
}


def family_of(config: dict) -> Tuple[type, type]:
    """(configuration class, model class) for the contents of a config.json."""
    for key in ("model_type", "architecture"):
        name = config.get(key)
        if isinstance(name, str) and name.lower() in FAMILIES:
            return FAMILIES[name.lower()]
    raise ValueError(f"no model family for model_type {config.get('model_type')!r} / architecture {config.get('architecture')!r}; "
                     f"known: {', '.join(sorted(FAMILIES))}")


def load_model(path: str, device=None, dtype=None):
    """The model in a local checkpoint directory, of whichever family its config.json names."""
    return family_of(checkpoint.read_config(path))[1].from_pretrained(path, device=device, dtype=dtype)
