"""Typed hyper-parameters of the Fiterax architecture, read from its config.json.

A Fiterax layer runs its mixer and its feed-forward side by side on one residual stream, x <- x + m (mixer(c1(norm1
x)) + ff(c2(norm2 x))), with a factor m, root-mean-square norms over equal consecutive parts of the vector, and a short
causal filter c over time, added to its input, ahead of each of the two.  Mixers, in any order: grouped softmax
*attention* (biases, rotary positions on the first coordinates of each head in the rotate-half layout, queries and keys
at unit root mean square after the turn, a factor a head on the scores and a smooth cap, a sigmoid gate a head), or an
*mlstm* matrix memory with exponential gates.  The feed-forward is routed experts without gates (exact GELU), chosen by
the sigmoid of their logits plus a correction and weighted by the sigmoids over their sum times a factor, or absent.
The embedding is multiplied by a factor; the head is a matrix of its own.

config.json:
    {"architecture": "Fiterax", "vocab": V, "width": W, "norm": {"eps": e, "groups": g}, "canon": {"taps": t} | absent,
     "embedding": {"scale": f} | absent, "residual_mult": m,
     "layers": [
       {"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "softcap"?,
            "rot": {"dims", "base"}?}, "mlp": ...},
       {"type": "mlstm", "mixer": {"heads", "dim", "vdim", "gate_cap"}, "mlp": ...}]}
    mlp: null | {"kind": "moe", "router": {"experts", "top", "scale"}, "expert": {"ff"}}
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .gisedra_param import _check_rot, _need, _NUM
from .hyper_param import ConfigError

ARCHITECTURE = "Fiterax"
MIXER_TYPES = ("attention", "mlstm")


@dataclass(frozen=True)
class FiteraxHyperParam:
    vocab: int
    width: int
    layers: List[Dict[str, Any]]                 # as in config.json
    norm_groups: int = 1
    norm_eps: float = 1e-5
    taps: int = 0                                # 0: no filter ahead of the sublayers
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    max_positions: int = 65536                   # the design has no limit of its own
    eos_token_id: Optional[int] = None
    torch_dtype: str = "bfloat16"
    architecture: str = ARCHITECTURE
    extra: Dict[str, Any] = field(default_factory=dict, compare=False)

    # ------------------------------------------------------------- validation
    def validate(self) -> "FiteraxHyperParam":
        if self.norm_eps <= 0:
            raise ConfigError(f"norm.eps must be positive, got {self.norm_eps}")
        if self.norm_groups < 1 or self.width % self.norm_groups:
            raise ConfigError(f"norm.groups must divide the width {self.width}, got {self.norm_groups}")
        if not 0 <= self.taps <= 8:
            raise ConfigError(f"canon.taps must be 1 to 8 (or canon absent), got {self.taps}")
        if not self.layers:
            raise ConfigError("config.json: 'layers' is empty")
        for i, L in enumerate(self.layers):
            w = f"layers[{i}]"
            kind = L.get("type") if isinstance(L, dict) else None
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {w}.type must be one of {MIXER_TYPES}, got {kind!r}")
            getattr(self, "_check_" + kind)(L.get("mixer"), f"{w}.mixer")
            self._check_mlp(L.get("mlp"), f"{w}.mlp")
        return self

    @staticmethod
    def _check_attention(m, w: str) -> None:
        heads = _need(m, "heads", w, (int,), 1)
        if heads % _need(m, "kv_heads", w, (int,), 1):
            raise ConfigError(f"config.json: {w}.heads must be a multiple of kv_heads")
        for key in ("dim", "vdim"):
            if _need(m, key, w, (int,), 1) > 256:
                raise ConfigError(f"config.json: {w}.{key}: heads of up to 256, got {m[key]}")
        _need(m, "scale", w, _NUM)
        if m.get("softcap") is not None and _need(m, "softcap", w, _NUM) < 0:
            raise ConfigError(f"config.json: {w}.softcap must not be negative")
        if m.get("rot") is not None:
            _check_rot(m["rot"], f"{w}.rot", m["dim"], False)

    @staticmethod
    def _check_mlstm(m, w: str) -> None:
        _need(m, "heads", w, (int,), 1)
        for key in ("dim", "vdim"):
            if _need(m, key, w, (int,), 1) > 256:
                raise ConfigError(f"config.json: {w}.{key}: up to 256 channels a head, got {m[key]}")
        if _need(m, "gate_cap", w, _NUM) <= 0:
            raise ConfigError(f"config.json: {w}.gate_cap must be positive")

    @staticmethod
    def _check_mlp(mlp, w: str) -> None:
        if mlp is None:
            return
        if not isinstance(mlp, dict) or mlp.get("kind", "moe") != "moe":
            raise ConfigError(f"config.json: {w}.kind must be 'moe'")
        r = mlp.get("router")
        experts = _need(r, "experts", f"{w}.router", (int,), 1)
        if _need(r, "top", f"{w}.router", (int,), 1) > min(experts, 16):
            raise ConfigError(f"config.json: {w}.router.top must be at most the number of experts and 16, got {r['top']}")
        _need(r, "scale", f"{w}.router", _NUM)
        _need(mlp.get("expert"), "ff", f"{w}.expert", (int,), 1)

    # --------------------------------------------------------------- factories
    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "FiteraxHyperParam":
        layers = copy.deepcopy(d.get("layers"))
        if not isinstance(layers, list):
            raise ConfigError("config.json lacks the list 'layers'")
        emb, norm = d.get("embedding") or {}, d.get("norm")
        known = {"architecture", "architectures", "vocab", "width", "layers", "norm", "canon", "embedding", "residual_mult",
                 "max_positions", "eos_token_id", "torch_dtype", "dtype"}
        return cls(
            vocab=_need(d, "vocab", "the top level", (int,), 1),
            width=_need(d, "width", "the top level", (int,), 1),
            layers=layers,
            norm_groups=_need(norm, "groups", "norm", (int,), 1),
            norm_eps=float(_need(norm, "eps", "norm", _NUM)),
            taps=_need(d["canon"], "taps", "canon", (int,), 1) if d.get("canon") is not None else 0,
            embedding_scale=float(emb["scale"]) if emb.get("scale") is not None else 1.0,
            residual_mult=float(_need(d, "residual_mult", "the top level", _NUM)),
            max_positions=int(d.get("max_positions", 65536)),
            eos_token_id=d.get("eos_token_id"),
            torch_dtype=str(d.get("torch_dtype", d.get("dtype", "bfloat16"))).replace("torch.", ""),
            architecture=ARCHITECTURE,
            extra={k: v for k, v in d.items() if k not in known},
        ).validate()

    def to_config_dict(self) -> Dict[str, Any]:
        cfg: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps, "groups": self.norm_groups},
                               "embedding": {"scale": self.embedding_scale}, "residual_mult": self.residual_mult,
                               "layers": copy.deepcopy(self.layers), "torch_dtype": self.torch_dtype}
        if self.taps:
            cfg["canon"] = {"taps": self.taps}
        if self.max_positions != 65536:
            cfg["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            cfg["eos_token_id"] = self.eos_token_id
        return cfg

    def __str__(self) -> str:
        kinds = ", ".join(f"{L['type']}/{'moe' if L.get('mlp') else 'none'}" for L in self.layers)
        return (f"FiteraxHyperParam {{\n\tvocab = {self.vocab}\n\twidth = {self.width}\n\tnorm_eps = {self.norm_eps}\n\t"
                f"norm_groups = {self.norm_groups}\n\ttaps = {self.taps}\n\tlayers = [{kinds}]\n}}")
