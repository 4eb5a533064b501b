"""Small Fiterax configurations for the tests, with weights made here, large enough that every mechanism moves the
logits, and a router whose choices rest on no close call.

A: four groups a norm, filters of three taps; an attention whose values are wider than its keys (4 heads on 2 key heads,
   half of each head turned), a matrix memory, an attention whose values are narrower, without feed-forward; 6 experts, 2 a
   token; a branch factor that is no power of two.
B: sizes that no vector load divides (width 90 in 3 groups, filters of five taps, heads of 10 and 6, a memory of 5 x 7
   channels, experts of 20); fully turned heads as many key heads as heads; every expert a token.
C: one group, filters of one tap (no state); 8 heads on one key head, scores without a cap and nothing turned; a memory of
   72 x 40 channels and small gate cap; one expert a token; factors of one.
D: no filters at all; one head everywhere; a memory without feed-forward; three of four experts a token.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict

import torch


def _attention(heads, kv, dim, vdim, scale, softcap=None, rot=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if softcap is not None:
        m["softcap"] = softcap
    if rot is not None:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return {"type": "attention", "mixer": m}


def _mlstm(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _with(layer, experts=0, top=0, scale=1.0, ff=0):
    mlp = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale}, "expert": {"ff": ff}} if experts else None
    return dict(layer, mlp=mlp)


def _cfg(vocab, width, eps, groups, taps, emb, mult, layers):
    c = {"architecture": "Fiterax", "vocab": vocab, "width": width, "max_positions": 1024, "norm": {"eps": eps, "groups": groups},
         "embedding": {"scale": emb}, "residual_mult": mult, "layers": layers}
    if taps:
        c["canon"] = {"taps": taps}
    return c


CONFIGS = {
    "A": _cfg(97, 64, 1e-6, 4, 3, 2.0, 0.6,
              [_with(_attention(4, 2, 16, 24, 0.25, 6.0, (8, 300.0)), 6, 2, 1.5, 24),
               _with(_mlstm(2, 12, 20, 9.0), 6, 2, 1.5, 24),
               _with(_attention(2, 1, 32, 12, 0.2, 20.0, (16, 50.0)))]),
    "B": _cfg(131, 90, 1e-4, 3, 5, 0.5, 1.3,
              [_with(_mlstm(3, 5, 7, 15.0), 5, 5, 2.0, 20),
               _with(_attention(3, 3, 10, 6, 0.3, 3.0, (10, 1000.0)), 5, 5, 0.7, 20)]),
    "C": _cfg(61, 128, 1e-5, 1, 1, 1.0, 1.0,
              [_with(_attention(8, 1, 32, 32, 0.18), 8, 1, 1.0, 40),
               _with(_mlstm(4, 72, 40, 2.0), 8, 1, 1.0, 40)]),
    "D": _cfg(53, 48, 1e-5, 2, 0, 3.0, 0.5,
              [_with(_mlstm(1, 16, 64, 12.0)),
               _with(_attention(1, 1, 48, 16, 0.15, 30.0, (4, 20.0)), 4, 3, 2.5, 16)]),
}
PAGE_SIZE = {"A": 4, "B": 2, "C": 16, "D": 8}


def reserved(cfg: dict) -> int:
    """The first coordinates of the stream hold a code of the token that only the routers read."""
    return max([L["mlp"]["router"]["experts"] for L in cfg["layers"] if L.get("mlp")] or [0])


def make_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors by name.  The embedding's first ``reserved`` coordinates are a code of the token's id (levels from
    1 down to -1, the highest at id % experts); every matrix that writes into the stream is zero there, the filters leave
    them alone, and a router reads nothing else: a token's experts follow from its id by a wide margin.  The corrections
    move an expert past all others, which brings no two close."""
    g = torch.Generator().manual_seed(seed)
    W, V, taps = cfg["width"], cfg["vocab"], (cfg.get("canon") or {}).get("taps", 0)
    R = reserved(cfg)
    rnd = lambda *shape, std=1.0: torch.randn(*shape, generator=g) * std
    mat = lambda out, inp, gain=1.0: rnd(out, inp, std=gain / math.sqrt(inp))

    def writes(t):                # a matrix (or bias) whose result enters the stream: nothing into the reserved coordinates
        t[:R] = 0.0
        return t

    def gain(width):
        w = 1.0 + rnd(width, std=0.2)
        w[:R] = 1.0
        return w

    scale = cfg["embedding"]["scale"]
    emb = rnd(V, W) / scale
    for t in range(V):
        for e in range(R):
            emb[t, e] = (1.0 - 2.0 * ((e - t) % R) / max(R - 1, 1)) / scale
    w = {"embed": emb, "final.norm": gain(W), "head": mat(V, W, 1.0)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        w[p + "norm1"] = gain(W)
        if taps:
            w[p + "canon1"] = rnd(W, taps, std=0.35)
        if L["type"] == "attention":
            G = m["kv_heads"]
            w.update({p + "mix.q": mat(H * d, W, 1.5), p + "mix.q.b": rnd(H * d, std=0.4), p + "mix.k": mat(G * d, W, 1.5),
                      p + "mix.k.b": rnd(G * d, std=0.4), p + "mix.v": mat(G * dv, W, 1.2), p + "mix.v.b": rnd(G * dv, std=0.4),
                      p + "mix.temp": 1.0 + rnd(H, std=0.4), p + "mix.g": mat(H, W, 1.5),
                      p + "mix.o": writes(mat(W, H * dv, 1.2)), p + "mix.o.b": writes(rnd(W, std=0.3))})
        else:
            # a read-out is a sum of v (k . q) and is then normalised: where the k . q of the few tokens that a fast
            # decay leaves cancel, rounding decides the direction.  Keys that lean towards the queries keep them positive.
            rq = mat(H * d, W, 1.5)
            w.update({p + "mix.q": rq, p + "mix.k": 0.8 * rq + mat(H * d, W, 0.5), p + "mix.v": mat(H * dv, W, 1.2),
                      p + "mix.g": mat(H * dv, W, 1.5), p + "mix.i": mat(H, W, 1.5), p + "mix.i.b": rnd(H, std=1.0),
                      p + "mix.f": mat(H, W, 1.0), p + "mix.f.b": 2.5 + rnd(H, std=1.0),
                      p + "mix.norm": 1.0 + rnd(H * dv, std=0.2), p + "mix.o": writes(mat(W, H * dv, 1.0))})
        mlp = L.get("mlp")
        if mlp:
            E, F = mlp["router"]["experts"], mlp["expert"]["ff"]
            w[p + "norm2"] = gain(W)
            if taps:
                w[p + "canon2"] = rnd(W, taps, std=0.35)
                w[p + "canon2"][:R] = 0.0
            router = torch.zeros(E, W)
            for e in range(E):
                router[e, e] = 2.0
            w[p + "mlp.router"] = router
            w[p + "mlp.correction"] = torch.zeros(E)
            if mlp["router"]["top"] < E:                  # one expert is chosen always (of several a token), one never
                w[p + "mlp.correction"][2 % E] = -1.0
                if mlp["router"]["top"] > 1:
                    w[p + "mlp.correction"][1] = 1.0
            for e in range(E):
                w[p + f"mlp.e{e}.up"] = mat(F, W, 1.5)
                w[p + f"mlp.e{e}.down"] = writes(mat(W, F, 1.5))
    return w


def write_folder(cfg: dict, folder: str, seed: int, weights: Dict[str, torch.Tensor] = None) -> str:
    """config.json and model.safetensors (bfloat16) of ``cfg`` in ``folder``."""
    from swifttransformer_amd.weights.safetensors_io import save_safetensors
    os.makedirs(folder, exist_ok=True)
    w = weights if weights is not None else make_weights(cfg, seed)
    save_safetensors(os.path.join(folder, "model.safetensors"),
                     {k: v.to(torch.bfloat16).contiguous() for k, v in w.items()}, {"format": "pt"})
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f, indent=1)
    return folder


def prompt(length: int, vocab: int, seed: int):
    g = torch.Generator().manual_seed(9100 + seed)
    return torch.randint(0, vocab, (length,), generator=g).tolist()
