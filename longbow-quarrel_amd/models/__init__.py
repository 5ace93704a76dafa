"""Architectures.  Importing the package registers them."""
from . import llama, mifidra, puzonex, sofinex, tukedra, vafodra, vupelorn  # noqa: F401
