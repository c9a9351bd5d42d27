"""Architectures. Importing this package registers the built-in ones."""
from . import gurapel, llama, murulorn, niresun, takosun, zevetar, zunilorn  # noqa: F401  (registration)
from .decoder import DecoderModel

__all__ = ["DecoderModel"]
