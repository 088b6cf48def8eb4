"""Architectures the framework ships.  Importing a module registers it."""
from . import dogalorn, fikupel, gpt2, nigilorn, pafivik, ridopel   # noqa: F401
