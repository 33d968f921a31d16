from . import (attention, block, combine, diff_attention, ends, head_mix_attention, mlp, norm, recurrent, rope, routed,  # noqa: F401
               sink_attention)  # (they register themselves)
from .model import DecoderModel, build_blocks, expected_tensors
from .registry import PartError, build_part, part_class, register_part

__all__ = ["DecoderModel", "build_blocks", "expected_tensors", "PartError", "build_part", "part_class",
           "register_part"]
