"""Which configuration and model class a checkpoint directory needs, decided by its ``config.json``:
``architecture`` names a layered decoder, ``model_type`` the EventChat family."""
from __future__ import annotations

import json
import os
from typing import Any, Dict, NamedTuple, Type

import torch

from .config import EventChatConfig
from .event_chat import EventChatModel
from .layered import LayeredConfig, LayeredDecoder


class ModelEntry(NamedTuple):
    config: Type
    model: Type
    modality: str        # "event": takes event frames with its prompt; "text": token ids alone


REGISTRY: Dict[str, ModelEntry] = {
    EventChatConfig.model_type: ModelEntry(EventChatConfig, EventChatModel, "event"),
    "Nusitar": ModelEntry(LayeredConfig, LayeredDecoder, "text"),
    "Zapipel": ModelEntry(LayeredConfig, LayeredDecoder, "text"),
}


def resolve(config: Dict[str, Any]) -> ModelEntry:
    name = config.get("architecture") or config.get("model_type")
    if name is None and "hidden_size" in config:
        name = EventChatConfig.model_type        # checkpoints of that family may omit the field
    if name not in REGISTRY:
        raise ValueError(f"unknown model {name!r}; known: {sorted(REGISTRY)}")
    return REGISTRY[name]


def read_config(path: str):
    """``(entry, configuration object)`` of a checkpoint directory."""
    with open(os.path.join(path, "config.json")) as f:
        d = json.load(f)
    entry = resolve(d)
    return entry, entry.config.from_dict(d)


def load_model(path: str, dtype: torch.dtype, device):
    entry, config = read_config(path)
    return entry.model.from_pretrained(path, torch_dtype=dtype, config=config, device=device)
