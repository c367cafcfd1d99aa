"""Architectures this package provides; importing the package registers them."""
from . import gupitar, kalevik, mapedra, qwen2, siditar, zabozen, zuluvik  # noqa: F401
