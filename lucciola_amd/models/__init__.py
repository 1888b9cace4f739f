"""Architectures: importing this package registers them."""
from . import kikunex, larupel, nogosun, pubodra, qwen3, rununex, vasanex  # noqa: F401
