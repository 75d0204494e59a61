"""Architectures known to the registry."""
from . import bobevik, butolorn, dofipel, domorax, penasun, qwen2, volonex  # noqa: F401
