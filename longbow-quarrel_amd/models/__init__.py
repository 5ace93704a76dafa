"""Architectures.  Importing the package registers them."""
from . import llama, mifidra, puzonex, sofinex, vafodra, vupelorn  # noqa: F401
