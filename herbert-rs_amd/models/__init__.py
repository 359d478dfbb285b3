"""Architectures: each module turns its typed configuration into a ModelSpec and registers itself."""
from . import bozasun, figalorn, mefatar, modasun, mutedra, qwen3, vipalorn

__all__ = ["bozasun", "figalorn", "mefatar", "modasun", "mutedra", "qwen3", "vipalorn"]
