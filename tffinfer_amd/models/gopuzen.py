"""Gopuzen decoder: registration of its configuration and tensor names.

The file names its tensors ``embed``, ``final.norm``, ``head`` and ``l<i>.{norm1, norm1b, norm2, norm2b, mix.*,
mlp.*, ls1, ls2, canon1, canon2}``: a part's single weight carries the part's own name, its other tensors
follow it (``l0.norm1.b``)."""
from ..config.gopuzen import ARCHITECTURE, GopuzenConfig
from .decoder import TensorNames
from .registry import register_architecture

GOPUZEN_NAMES = TensorNames(
    embedding="embed",
    layer="l{i}",
    final_norm="final.norm",
    head="head",
    children={"norm1": "norm1", "norm1_out": "norm1b", "mixer": "mix", "norm2": "norm2", "norm2_out": "norm2b",
              "feed_forward": "mlp"},
    bare_weights=True,
)

register_architecture(ARCHITECTURE, GopuzenConfig, GOPUZEN_NAMES)
