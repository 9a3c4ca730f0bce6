"""Architectures: the Python mirrors of their typed configurations (the architectures themselves
are registered in the engine library, one file each under csrc/engine/)."""
from . import kezasun, nikasun, piditar, povipel, qwen2, rasodra, sizudra  # noqa: F401
