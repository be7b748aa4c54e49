from .builder import SuboraxBuilder, SuboraxConfig

__all__ = ["SuboraxBuilder", "SuboraxConfig"]
