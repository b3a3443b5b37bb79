"""Registers the Paluzen decoder: the name in config.json -> its configuration class."""
from ..config.paluzen import PaluzenConfig
from ..registry import register

register("architecture", "Paluzen")(PaluzenConfig)
