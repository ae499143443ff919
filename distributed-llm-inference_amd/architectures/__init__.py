"""Architectures that ship with the engine. Importing this package registers them."""

from . import betepel, llama, makodra, miberax, pibuvik, rurorax, zarinex  # noqa: F401
