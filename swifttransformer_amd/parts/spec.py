"""The description of a model as data: which parts each layer is made of, with
what sizes and constants, under which tensor names, and in which order the
layers run.  An architecture module turns its config.json into a ``ModelSpec``;
nothing below this file knows the architecture's name."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional


@dataclass
class PartSpec:
    kind: str                                    # name in the part registry of its category
    params: Dict[str, Any] = field(default_factory=dict)   # sizes and constants
    names: Dict[str, str] = field(default_factory=dict)    # logical tensor -> name in the file


@dataclass
class LayerSpec:
    """The parts of one layer.  The arrangement decides which of them it uses and how; a slot
    that its arrangement does not use is None (a block with one norm, or without feed-forward)."""
    arrangement: PartSpec        # how norms, mixer and feed-forward are wired (pre/post-norm)
    mixer_norm: Optional[PartSpec]
    mixer: PartSpec
    ffn_norm: Optional[PartSpec]
    feed_forward: Optional[PartSpec]
    mixer_conv: Optional[PartSpec] = None   # a short filter over time on what the mixer reads
    ffn_conv: Optional[PartSpec] = None     # the same on what the feed-forward reads
    mixer_out_norm: Optional[PartSpec] = None   # a norm on the mixer's result before it enters the stream
    ffn_out_norm: Optional[PartSpec] = None     # the same for the feed-forward's result
    side_input: Optional[PartSpec] = None       # what the layer adds from an input of the token's own


@dataclass
class ScheduleEntry:
    """One run of a layer.  ``cache`` names the cache this run uses (by default the
    layer's own); a run with ``write=False`` reads a cache that an earlier run of the
    same step has already filled with the step's tokens."""
    layer: int
    cache: int
    write: bool = True
    enter: Optional[int] = None   # index into ``ModelSpec.entries``: that part acts on the stream before this run


@dataclass
class ModelSpec:
    hidden_size: int
    vocab_size: int
    max_positions: int            # longest sequence the model can run
    embedding: PartSpec
    position: PartSpec
    layers: List[LayerSpec]
    schedule: List[ScheduleEntry]
    final_norm: Optional[PartSpec]
    head: PartSpec
    eos_token_id: Optional[int] = None
    # parts of the category "reentry": what happens to the residual stream before the runs that name
    # them (a pass over a group of layers that starts from a mix of the stream and the embedding)
    entries: List[PartSpec] = field(default_factory=list)
    # > 0: the residual stream runs as that many copies side by side, float [T, streams * hidden]: the model
    # makes the copies after the embedding and sums them before the final norm; the layers' arrangements read
    # and write all of them
    streams: int = 0

    def validate(self) -> "ModelSpec":
        n = len(self.layers)
        written = set()
        for e in self.schedule:
            if e.enter is not None and not 0 <= e.enter < len(self.entries):
                raise ValueError(f"the schedule names entry {e.enter}; there are {len(self.entries)}")
            if not 0 <= e.layer < n:
                raise ValueError(f"the schedule names layer {e.layer}; there are {n} layers")
            if e.write:
                if e.cache in written:
                    raise ValueError(f"cache {e.cache} is written by two runs of one step")
                written.add(e.cache)
            elif e.cache not in written:
                raise ValueError(
                    f"layer {e.layer} reads cache {e.cache} before any run has written it")
        return self
