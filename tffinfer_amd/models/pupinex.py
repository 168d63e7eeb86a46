"""Pupinex decoder: registration of its configuration and tensor names.

The file names its tensors ``embed``, ``bigram``, ``final.norm`` and ``l<i>.{norm1, norm2, mix.*, mlp.*}``: a part's
single weight carries the part's own name, its other tensors follow it (``l0.mix.q.b``).  There is no output head: the
embedding serves."""
from ..config.pupinex import ARCHITECTURE, PupinexConfig
from .decoder import TensorNames
from .registry import register_architecture

PUPINEX_NAMES = TensorNames(
    embedding="embed",
    layer="l{i}",
    final_norm="final.norm",
    head="head",
    bigram="bigram",
    children={"norm1": "norm1", "mixer": "mix", "norm2": "norm2", "feed_forward": "mlp"},
    bare_weights=True,
)

register_architecture(ARCHITECTURE, PupinexConfig, PUPINEX_NAMES)
