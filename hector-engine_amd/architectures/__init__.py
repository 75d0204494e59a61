"""Architectures known to the registry."""
from . import butolorn, dofipel, domorax, penasun, qwen2, volonex  # noqa: F401
