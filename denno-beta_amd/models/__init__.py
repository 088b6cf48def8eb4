"""Architectures the framework ships.  Importing a module registers it."""
from . import dogalorn, fikupel, gpt2, nigilorn, pafivik, pepapel, ridopel   # noqa: F401
