"""Architectures; importing this package registers the built-in ones."""
from . import besulix, gemma2, golepel, kaderax, lutovik, solulix, vogunex   # noqa: F401
