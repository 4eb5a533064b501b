"""Typed hyper-parameters of the Fefozen architecture, read from its config.json.

A Fefozen layer has root-mean-square norms (weights stored around zero) before and after its mixer and before and after its
feed-forward.  Mixers, in any order: *delta* (a gated delta rule behind short causal filters, heads sharing queries and keys in
groups), *latent_attention* (queries through a latent of their own, keys and values from one cached latent a token beside a small
turned key part that all heads share, turned pairs of neighbouring coordinates, a learned sink a head, a gate on the heads) and
*latent_attention_2* (the same with turned pairs half the part apart and without a sink; it may read the cache of an earlier layer,
``kv_from``).  The feed-forward is dense (tanh-form GELU), routed experts (clamped gated units, chosen by the softmax over all
plus a correction, weighted by the softmax as it is; the router's last outputs are identity experts), or absent.  The head is the
embedding table.

config.json:
    {"architecture": "Fefozen", "vocab": V, "width": W, "norm": {"eps": e},
     "layers": [
       {"type": "delta", "mixer": {"heads", "kv_heads", "dim", "vdim", "conv"}, "mlp": ...},
       {"type": "latent_attention" | "latent_attention_2", "mixer": {"heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank",
            "scale", "rot": {"dims", "base"}, "kv_from"?}, "mlp": ...}]}
    mlp: null | {"kind": "dense", "ff"} | {"kind": "moe", "router": {"experts", "top", "identity"?}, "expert": {"ff", "limit"}}
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .gisedra_param import _check_rot, _need, _NUM
from .hyper_param import ConfigError

ARCHITECTURE = "Fefozen"
LATENT_TYPES = ("latent_attention", "latent_attention_2")
MIXER_TYPES = ("delta",) + LATENT_TYPES
MAX_ENTRY = 576                  # numbers of a cached entry (latent and turned part) that the attention kernels take


@dataclass(frozen=True)
class FefozenHyperParam:
    vocab: int
    width: int
    layers: List[Dict[str, Any]]                 # as in config.json
    norm_eps: float = 1e-6
    max_positions: int = 65536                   # the design has no limit of its own
    eos_token_id: Optional[int] = None
    torch_dtype: str = "bfloat16"
    architecture: str = ARCHITECTURE
    extra: Dict[str, Any] = field(default_factory=dict, compare=False)

    # ------------------------------------------------------------- validation
    def validate(self) -> "FefozenHyperParam":
        if self.norm_eps <= 0:
            raise ConfigError(f"norm.eps must be positive, got {self.norm_eps}")
        if not self.layers:
            raise ConfigError("config.json: 'layers' is empty")
        for i, L in enumerate(self.layers):
            w = f"layers[{i}]"
            kind = L.get("type") if isinstance(L, dict) else None
            if kind not in MIXER_TYPES:
                raise ConfigError(f"config.json: {w}.type must be one of {MIXER_TYPES}, got {kind!r}")
            m = L.get("mixer")
            if kind == "delta":
                self._check_delta(m, f"{w}.mixer")
            else:
                self._check_latent(m, f"{w}.mixer")
                if m.get("kv_from") is not None:
                    self._check_kv_from(i, kind, m, f"{w}.mixer")
            self._check_mlp(L.get("mlp"), f"{w}.mlp")
        return self

    @staticmethod
    def _check_delta(m, w: str) -> None:
        heads = _need(m, "heads", w, (int,), 1)
        if heads % _need(m, "kv_heads", w, (int,), 1):
            raise ConfigError(f"config.json: {w}.heads must be a multiple of kv_heads")
        if _need(m, "dim", w, (int,), 1) > 256:
            raise ConfigError(f"config.json: {w}.dim: up to 256 key channels a head, got {m['dim']}")
        _need(m, "vdim", w, (int,), 1)
        if _need(m, "conv", w, (int,), 1) > 8:
            raise ConfigError(f"config.json: {w}.conv: 1 to 8 taps, got {m['conv']}")

    @staticmethod
    def _check_latent(m, w: str) -> None:
        for key in ("heads", "dim", "vdim", "q_rank", "kv_rank"):
            _need(m, key, w, (int,), 1)
        r = _need(m, "rot_dim", w, (int,), 0)
        _need(m, "scale", w, _NUM)
        if r % 2 or -(-m["kv_rank"] // 8) * 8 + r > MAX_ENTRY:
            raise ConfigError(f"config.json: {w}.rot_dim must be even and kv_rank + rot_dim at most {MAX_ENTRY}, got "
                              f"{m['kv_rank']} + {r}")
        if r:
            _check_rot(m.get("rot"), f"{w}.rot", r, False)

    def _check_kv_from(self, i: int, kind: str, m, w: str) -> None:
        j = _need(m, "kv_from", w, (int,), 0)
        src = self.layers[j] if j < i else None
        if src is None or src.get("type") != kind or src["mixer"].get("kv_from") is not None:
            raise ConfigError(f"config.json: {w}.kv_from must name an earlier {kind} layer with a latent of its own, got {j}")
        for key in ("kv_rank", "rot_dim", "rot"):
            if src["mixer"].get(key) != m.get(key):
                raise ConfigError(f"config.json: {w}.{key} differs from that of layers[{j}], whose cache it reads")

    @staticmethod
    def _check_mlp(mlp, w: str) -> None:
        if mlp is None:
            return
        kind = mlp.get("kind") if isinstance(mlp, dict) else None
        if kind == "dense":
            _need(mlp, "ff", w, (int,), 1)
            return
        if kind != "moe":
            raise ConfigError(f"config.json: {w}.kind must be 'dense' or 'moe', got {kind!r}")
        r = mlp.get("router")
        outputs = _need(r, "experts", f"{w}.router", (int,), 1)
        if r.get("identity") is not None:
            outputs += _need(r, "identity", f"{w}.router", (int,), 0)
        if _need(r, "top", f"{w}.router", (int,), 1) > min(outputs, 16):
            raise ConfigError(f"config.json: {w}.router.top must be at most the router's outputs and 16, got {r['top']}")
        _need(mlp.get("expert"), "ff", f"{w}.expert", (int,), 1)
        _need(mlp.get("expert"), "limit", f"{w}.expert", _NUM)

    # --------------------------------------------------------------- factories
    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "FefozenHyperParam":
        layers = copy.deepcopy(d.get("layers"))
        if not isinstance(layers, list):
            raise ConfigError("config.json lacks the list 'layers'")
        known = {"architecture", "architectures", "vocab", "width", "layers", "norm", "max_positions", "eos_token_id",
                 "torch_dtype", "dtype"}
        return cls(
            vocab=_need(d, "vocab", "the top level", (int,), 1),
            width=_need(d, "width", "the top level", (int,), 1),
            layers=layers,
            norm_eps=float(_need(d.get("norm"), "eps", "norm", _NUM)),
            max_positions=int(d.get("max_positions", 65536)),
            eos_token_id=d.get("eos_token_id"),
            torch_dtype=str(d.get("torch_dtype", d.get("dtype", "bfloat16"))).replace("torch.", ""),
            architecture=ARCHITECTURE,
            extra={k: v for k, v in d.items() if k not in known},
        ).validate()

    def to_config_dict(self) -> Dict[str, Any]:
        cfg: Dict[str, Any] = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                               "norm": {"eps": self.norm_eps}, "layers": copy.deepcopy(self.layers),
                               "torch_dtype": self.torch_dtype}
        if self.max_positions != 65536:
            cfg["max_positions"] = self.max_positions
        if self.eos_token_id is not None:
            cfg["eos_token_id"] = self.eos_token_id
        return cfg

    def __str__(self) -> str:
        kinds = ", ".join(f"{L['type']}/{(L.get('mlp') or {}).get('kind', 'none')}" for L in self.layers)
        return (f"FefozenHyperParam {{\n\tvocab = {self.vocab}\n\twidth = {self.width}\n\tnorm_eps = {self.norm_eps}\n\t"
                f"layers = [{kinds}]\n}}")
