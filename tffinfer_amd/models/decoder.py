"""The model skeleton every decoder architecture shares: embedding, a list of
blocks run in the order the configuration gives, final norm, output head.

What a layer is made of and in which order layers run is data from the typed
configuration (``layer_specs``, ``layer_schedule``); this file holds no size
and no constant of any architecture.  The reference wires the same sequence as
graph nodes in src/core/model/qwen3/QWen3Creator.cpp:43-165.
"""
from __future__ import annotations

from dataclasses import dataclass, field

import torch

from ..config.base import ModelConfig
from ..parts.base import BLOCKS, FEED_FORWARDS, MIXERS, NORMS, Part, StateSpec, WeightSpec
from ..parts.embedding import BigramTable, Embedding, OutputHead
from ..weights.loader import check_weights, normalize_stored
from ..weights.random_init import FLOAT32_INITS, random_tensor


@dataclass
class TensorNames:
    """How an architecture's files name the tensors of the skeleton's parts."""
    embedding: str = "model.embed_tokens"
    layer: str = "model.layers.{i}"
    final_norm: str = "model.norm"
    head: str = "lm_head"
    #: the table of vectors the run order adds to the stream, for architectures that have one
    stream_offsets: str = "stream_offsets"
    #: the embedding's table for pairs of tokens, for architectures that have one
    bigram: str = "bigram"
    #: the block's children by the name the files use
    children: dict = field(default_factory=dict)
    #: tensors a file may hold that the model has no use for
    ignorable: tuple = ()
    #: True: a part's tensor called "weight" carries the part's own name in the file
    #: ("final.norm", not "final.norm.weight"); a part's other tensors follow the part's name
    bare_weights: bool = False

    def tensor(self, prefix: str, local: str) -> str:
        """The file's name of the tensor ``local`` of the part named ``prefix``."""
        if self.bare_weights and local == "weight":
            return prefix
        return f"{prefix}.{local}"


def _leaves(prefix: str, part: Part, rename: dict):
    """(global name prefix, part) for a part and all its sub-parts."""
    yield prefix, part
    for child_name, child in part.children().items():
        yield from _leaves(f"{prefix}.{rename.get(child_name, child_name)}", child, rename)


class StreamOffsets(Part):
    """A table [rows, hidden] of vectors that the run order adds to the residual stream before
    certain layer calls (``LayerCall.offset`` names the row); float32."""

    graph_safe = True

    def __init__(self, rows: int, hidden_size: int):
        self.rows = int(rows)
        self.hidden_size = int(hidden_size)
        self.weight = None

    def weight_specs(self):
        return {"weight": WeightSpec((self.rows, self.hidden_size), "vector")}

    def load_weights(self, weights, dtype, device):
        self.weight = weights["weight"].to(torch.float32).contiguous().to(device)

    def row(self, i: int) -> torch.Tensor:
        return self.weight[i]


class DecoderModel:
    def __init__(self, config: ModelConfig, names: TensorNames):
        self.config = config
        self.names = names
        self.dtype = None
        self.device = None
        H, V = config.hidden_size, config.vocab_size
        emb_norm = config.embedding_norm_spec() if hasattr(config, "embedding_norm_spec") else None
        pairs = config.bigram_spec() if hasattr(config, "bigram_spec") else None
        self.embedding = Embedding(V, H, scale=getattr(config, "embedding_scale", 1.0),
                                   norm=NORMS.build(emb_norm) if emb_norm is not None else None,
                                   bigram=BigramTable(hidden_size=H, **pairs) if pairs is not None else None)
        n_off = config.stream_offset_rows() if hasattr(config, "stream_offset_rows") else 0
        self.stream_offsets = StreamOffsets(n_off, H) if n_off else None
        self.blocks = []
        for spec in config.layer_specs():
            mixer = MIXERS.build(spec.mixer)
            ffn = FEED_FORWARDS.build(spec.feed_forward)
            norm_spec = spec.norm
            block = BLOCKS.build(spec.block, mixer=mixer, feed_forward=ffn,
                                 make_norm=lambda s=norm_spec: NORMS.build(s))
            self.blocks.append(block)
        # the number each layer with tensors has in the file's names (layers that borrow another
        # layer's tensors are calls of that layer in the run order and have no number here)
        numbers = getattr(config, "layer_numbers", None)
        self.layer_numbers = list(numbers()) if callable(numbers) else list(range(len(self.blocks)))
        if len(self.layer_numbers) != len(self.blocks):
            raise ValueError("the configuration numbers another count of layers than it specifies")
        self.schedule = list(config.layer_schedule())
        for call in self.schedule:
            if not 0 <= call.layer < len(self.blocks):
                raise ValueError(f"layer schedule names layer {call.layer}, the model has {len(self.blocks)}")
            if call.offset >= (self.stream_offsets.rows if self.stream_offsets else 0):
                raise ValueError(f"layer schedule names stream offset {call.offset}, the model has "
                                 f"{self.stream_offsets.rows if self.stream_offsets else 0}")
            if call.add_embedding and call.offset >= 0:
                raise ValueError("a layer call adds the embedding's output or a row of the table of offsets, not both")
        #: some call adds the embedding's output to the stream: it is kept beside it
        self.keeps_embedding = any(call.add_embedding for call in self.schedule)
        self.final_norm = NORMS.build(config.final_norm_spec())
        self.head = OutputHead(V, H, self.embedding if config.tie_word_embeddings else None,
                               softcap=getattr(config, "logit_softcap", None),
                               scale=getattr(config, "logit_scale", None))

    # ---- weights ---------------------------------------------------------
    def _weighted_parts(self):
        yield from _leaves(self.names.embedding, self.embedding, {})
        if self.embedding.bigram is not None:
            yield self.names.bigram, self.embedding.bigram
        if self.stream_offsets is not None:
            yield self.names.stream_offsets, self.stream_offsets
        for i, block in zip(self.layer_numbers, self.blocks):
            yield from _leaves(self.names.layer.format(i=i), block, self.names.children)
        yield self.names.final_norm, self.final_norm
        yield self.names.head, self.head

    def expected_tensors(self) -> dict[str, WeightSpec]:
        out = {}
        for prefix, part in self._weighted_parts():
            for local, spec in part.weight_specs().items():
                out[self.names.tensor(prefix, local)] = spec
        return out

    def load_tensors(self, found: dict[str, torch.Tensor], dtype: torch.dtype, device,
                     where: str = "") -> None:
        """Checks ``found`` against what the parts expect (one error for all
        that is wrong) and hands every part its tensors."""
        ignorable = set(self.names.ignorable)
        if self.config.tie_word_embeddings:
            head = self.names.tensor(self.names.head, "weight")
            ignorable.add(head)
            if head in found:
                from .. import log
                log.warning("%s: '%s' is stored but the configuration ties the head to the embedding; "
                            "the stored copy is not used", where or "weights", head)
        check_weights(self.expected_tensors(), found, ignorable, where)
        self.dtype, self.device = dtype, torch.device(device)
        for prefix, part in self._weighted_parts():
            specs = part.weight_specs()
            if specs:
                part.load_weights({local: normalize_stored(found[self.names.tensor(prefix, local)])
                                   for local in specs if self.names.tensor(prefix, local) in found},
                                  dtype, self.device)

    def init_random(self, seed: int, dtype: torch.dtype, device, on_device: bool = False) -> None:
        """Seeded random weights without a file.  ``on_device`` draws on the GPU
        (another stream of numbers than the host's, for large models)."""
        self.dtype, self.device = dtype, torch.device(device)
        gen_dev = self.device if on_device else "cpu"
        for prefix, part in self._weighted_parts():
            specs = part.weight_specs()
            if specs:
                ws = {}
                for local, spec in specs.items():
                    if spec.optional:
                        continue
                    t = random_tensor(spec, seed, self.names.tensor(prefix, local), device=gen_dev)
                    ws[local] = t if spec.init in FLOAT32_INITS else t.to(torch.bfloat16)
                part.load_weights(ws, dtype, self.device)

    def graph_safe(self) -> bool:
        """True if every part launches only kernels that read the step's sizes
        from device tables, so a whole decode step can be captured in one HIP graph."""
        pieces = self.graph_pieces()
        return pieces is not None and len(pieces) == 1

    def _item_graph_safe(self, item) -> bool:
        if item == "embed":
            parts = [p for _, p in _leaves("", self.embedding, {})]
        elif item == "finish":
            parts = [self.final_norm, self.head]
        else:
            parts = [p for _, p in _leaves("", self.blocks[self.schedule[item].layer], {})]
        return all(getattr(p, "graph_safe", False) for p in parts)

    def graph_pieces(self):
        """The step as a list of pieces ``(capturable, items)``: items are "embed", the
        indices of the run order, and "finish" (final norm and head), in order; consecutive
        items that can all be captured in a HIP graph (or that all cannot: a part that loops
        on the host over the step's entries) form a piece.  None when nothing is gained:
        the embedding cannot be captured, or no layer call can."""
        items = ["embed"] + list(range(len(self.schedule))) + ["finish"]
        if not self._item_graph_safe("embed") or not any(self._item_graph_safe(i) for i in items[1:-1]):
            return None
        pieces = []
        for it in items:
            safe = self._item_graph_safe(it)
            if pieces and pieces[-1][0] == safe:
                pieces[-1][1].append(it)
            else:
                pieces.append((safe, [it]))
        return pieces

    # ---- cache needs -----------------------------------------------------
    def call_requirements(self):
        """For every entry of the run order: (cache id, writes, KVCacheSpec or
        None, StateSpec or None), and the state's id where it is not the cache's.  Where the embedding carries state,
        a row of its own follows those of the run order."""
        out = []
        for call in self.schedule:
            block = self.blocks[call.layer]
            row = (call.cache, call.writes_cache, block.mixer.cache_spec(), self.call_state(block))
            out.append(row if call.state < 0 or call.state == call.cache else row + (call.state,))
        own = self.embedding.state_spec()
        if own is not None:
            out.append((1 + max(max(call.cache, call.state) for call in self.schedule), True, None, own))
        return out

    @staticmethod
    def call_state(block) -> StateSpec | None:
        """The state of a layer call: the mixer's, with what the block itself carries behind it."""
        mixer, own = block.mixer.state_spec(), block.state_spec()
        if own is None:
            return mixer
        n = 0
        if mixer is not None:
            if len(mixer.shape) != 1 or mixer.dtype != own.dtype:
                raise ValueError("a block with state of its own takes a mixer whose state is one row of the same type")
            n = mixer.shape[0]
        block.state_offset = n
        return StateSpec((n + own.shape[0],), own.dtype)

    # ---- one step --------------------------------------------------------
    def forward(self, ctx) -> torch.Tensor:
        """Runs the tokens of ``ctx.batch`` and returns float32 logits
        [len(logit_rows), vocab]."""
        items = ["embed"] + list(range(len(self.schedule))) + ["finish"]
        _, _, logits = self.run_items(ctx, items, None, None)
        return logits

    def run_items(self, ctx, items, resid, pending):
        """Runs some consecutive items of the step (see ``graph_pieces``) and returns
        (residual stream, pending term, logits or None).  The residual stream is one float32
        tensor from the embedding on, added to in place; the pending term is what the last
        block returned for the next norm to add."""
        b = ctx.batch
        logits = None
        for it in items:
            if it == "embed":
                c = ctx.for_call(len(self.schedule)) if self.embedding.state_spec() is not None else ctx
                pending = None
                if self.keeps_embedding:
                    resid, b.embedding_output = self.embedding.forward_kept(c, b.token_ids)
                else:
                    resid = self.embedding.forward(c, b.token_ids)
            elif it == "finish":
                if b.num_logit_rows == 0:
                    logits = torch.empty(0, self.config.vocab_size, dtype=torch.float32, device=resid.device)
                else:
                    y = self.final_norm.forward(ctx, resid, pending, rows=b.logit_rows)
                    logits = self.head.forward(ctx, y)
            else:
                call = self.schedule[it]
                block, c = self.blocks[call.layer], ctx.for_call(it)
                if call.offset >= 0 or call.add_embedding:
                    extra = b.embedding_output if call.add_embedding else self.stream_offsets.row(call.offset)
                    if getattr(block, "takes_stream_offset", False):
                        c.stream_offset = extra
                    else:       # a block that knows nothing of offsets finds them in the stream
                        if pending is not None:
                            resid += ctx.ops.as_tensor(pending)
                            pending = None
                        resid += extra
                pending = block.forward(c, resid, pending)
        return resid, pending, logits
