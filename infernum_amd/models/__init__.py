"""Importing this package registers the built-in architectures."""
from .model import DecoderModel
from . import llama, malinex, mirovik, nesilorn, pamazen, rogizen, sikazen  # noqa: F401  (registration)
