"""Architectures.  Importing this package registers each of them."""

from tokamak_amd.models import dopirax, gubanex, korazen, mepupel, qwen3, rorosun, supinex  # noqa: F401
