"""Python face of ``eventgpt_amd/_D.so``, the gfx950 kernels of the layered decoders (``evlay::`` ops).

Importing this module loads the library and raises if it is not built (``python -m eventgpt_amd.build
--only layered``); there is no other GPU path to fall back to.
"""
from __future__ import annotations

import os

import torch

_SO = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "_D.so")
if not os.path.exists(_SO):
    raise RuntimeError(
        f"{_SO} not found: the HIP extension is not built. Run `python -m eventgpt_amd.build --only layered` "
        "(needs hipcc; cross-compiles for gfx950 without a GPU).")
torch.ops.load_library(_SO)
raw = torch.ops.evlay

GLU_ACTS = {"gelu_tanh": 0, "silu": 1}
