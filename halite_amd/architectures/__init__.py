"""Architectures: each module registers itself in ``config.registry`` on import."""

from . import diporax, divuzen, kavuvik, llama, nodupel, vepitar, zabunex  # noqa: F401
