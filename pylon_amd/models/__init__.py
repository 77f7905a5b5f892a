"""Built-in model families; importing this package registers them."""
from . import farorax, gimudra, qwen3, pavitar, ranudra, tukarax, vupuzen  # noqa: F401
