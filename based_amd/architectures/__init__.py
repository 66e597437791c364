"""Model designs with a config.json format and tensor names of their own.  A design is a module with
`stack_config(raw, shapes)` (config.json, and the shapes of the tensors by name for sizes that only they
tell -> StackConfig keywords) and `convert_state(raw, tensors)` (its tensors -> the stack's state dict);
config.json names it under "architecture"."""
from __future__ import annotations

from . import peponex, sozilix

DESIGNS = {"Peponex": peponex, "Sozilix": sozilix}


def find(raw: dict):
    """The design a config.json dictionary names, None for one without an "architecture"."""
    name = raw.get("architecture")
    if name is None:
        return None
    if name not in DESIGNS:
        raise NotImplementedError(f"architecture {name!r}: known are {sorted(DESIGNS)}")
    return DESIGNS[name]
