from .builder import BukatarBuilder, BukatarConfig, random_state_dict

__all__ = ["BukatarBuilder", "BukatarConfig", "random_state_dict"]
