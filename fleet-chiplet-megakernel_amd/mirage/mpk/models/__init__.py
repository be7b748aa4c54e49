"""Model graph builders; importing the package registers them (reference: python/mirage/mpk/models/__init__.py)."""
from .graph_builder import GraphBuilder, MirageModelConfig
from .bukatar import builder as _bukatar_builder  # noqa: F401  (registers BukatarBuilder)
from .dodonex import builder as _dodonex_builder  # noqa: F401  (registers DodonexBuilder)
from .qwen3 import builder as _qwen3_builder  # noqa: F401  (registers Qwen3Builder)
from .suborax import builder as _suborax_builder  # noqa: F401  (registers SuboraxBuilder)
from .vizonex import builder as _vizonex_builder  # noqa: F401  (registers VizonexBuilder)

__all__ = ["GraphBuilder", "MirageModelConfig"]
