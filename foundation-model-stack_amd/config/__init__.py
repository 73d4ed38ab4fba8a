from .base import ModelConfig
from .basopel import BasopelConfig
from .defapel import DefapelConfig
from .kapuvik import KapuvikConfig
from .llama import LLaMAConfig
from .sidalorn import SidalornConfig
from .zimorax import ZimoraxConfig
from .zodolorn import ZodolornConfig

__all__ = ["ModelConfig", "LLaMAConfig", "ZodolornConfig", "DefapelConfig", "SidalornConfig", "BasopelConfig", "ZimoraxConfig", "KapuvikConfig"]
