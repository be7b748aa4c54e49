from .builder import VizonexBuilder, VizonexConfig, random_state_dict

__all__ = ["VizonexBuilder", "VizonexConfig", "random_state_dict"]
