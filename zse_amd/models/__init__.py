"""Importing this package registers every architecture the engine serves."""
from . import bizepel, bumolix, buvuzen, dafotar, gemma2, pubunex, rotalorn  # noqa: F401
