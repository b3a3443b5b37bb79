"""Registers the Barilix decoder: the name in config.json -> its configuration class."""
from ..config.barilix import BarilixConfig
from ..registry import register

register("architecture", "Barilix")(BarilixConfig)
