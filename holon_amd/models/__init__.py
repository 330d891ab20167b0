"""Architectures. Importing this package registers them by their config.json name."""
from . import dopirax, falisun, nevodra, qwen3, relanex, sopepel, tolurax

__all__ = ["dopirax", "falisun", "nevodra", "qwen3", "relanex", "sopepel", "tolurax"]
