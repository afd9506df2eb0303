"""Designs of layer-stack models: architecture name of config.json -> function (config, tensor shape) -> StackSpec."""
from .ganidra import ganidra_spec
from .pabalix import pabalix_spec

DESIGNS = {"Ganidra": ganidra_spec, "Pabalix": pabalix_spec}
