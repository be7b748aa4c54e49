from .builder import DodonexBuilder, DodonexConfig, random_state_dict

__all__ = ["DodonexBuilder", "DodonexConfig", "random_state_dict"]
