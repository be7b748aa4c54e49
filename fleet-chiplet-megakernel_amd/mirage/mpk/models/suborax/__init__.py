from .builder import SuboraxBuilder, SuboraxConfig, random_state_dict

__all__ = ["SuboraxBuilder", "SuboraxConfig", "random_state_dict"]
