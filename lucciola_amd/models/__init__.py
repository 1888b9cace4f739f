"""Architectures: importing this package registers them."""
from . import kikunex, larupel, pubodra, qwen3, rununex, vasanex  # noqa: F401
