"""Architectures this library knows.  Importing a module registers its architecture."""
from . import bikadra, llama, nizedra, pigodra, refolix, vusenex  # noqa: F401
