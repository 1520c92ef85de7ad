"""Architectures. Importing this package registers them."""
from . import qwen2, goridra, tobozen, mobupel, gitasun, fugevik, lurirax   # noqa: F401
