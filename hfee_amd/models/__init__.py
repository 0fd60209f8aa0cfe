"""Architectures.  Importing this package registers every architecture it holds."""
from . import llama, medulorn, ronavik, sabezen, saposun, vofezen  # noqa: F401
