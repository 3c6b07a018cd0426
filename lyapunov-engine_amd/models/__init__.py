"""Architectures.  Importing the package registers the built-in one."""
from . import faledra, llama, panodra, pudulorn, ronupel, tonilix, vobotar  # noqa: F401
from .decoder import CacheGroupLayout, CacheLayout, DecoderModel, build_model

__all__ = ["CacheGroupLayout", "CacheLayout", "DecoderModel", "build_model"]
