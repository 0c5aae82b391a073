"""Architectures; importing this package registers the built-in ones."""
from . import besulix, gemma2, golepel, lutovik, solulix, vogunex   # noqa: F401
