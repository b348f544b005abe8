"""Architectures this library knows.  Importing a module registers its architecture."""
from . import bikadra, llama, nizedra, pigodra, pitenex, refolix, vusenex  # noqa: F401
