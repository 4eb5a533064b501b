"""Small Fefozen configurations for the tests, with weights made here, large enough that every mechanism moves the logits,
and a router whose choices rest on no close call.

A: a delta rule (4 heads on 2 query/key heads, four taps, values wider than keys), a latent attention of each kind, the second
   kind once more reading the first one's cache, with other head sizes; dense feed-forwards and 6 experts with 2 identity
   experts, 2 a token; a layer without feed-forward.
B: sizes that no vector load divides (width 90, latents of 37 and 21, heads of 10 and 6, a delta rule of 5 x 7 channels behind
   five taps, experts of 20); the sink first, every expert and identity expert a token.
C: one query/key head for 3 heads, keys wider than values (72 x 40), one tap; 20 heads (more than 16) on a latent of 130 beside a
   turned part of 64 of which 24 turn; one expert a token, no identity experts.
D: one head everywhere, nothing turned, a latent of 16; a borrowing layer beside its lender; three of five choices, three of
   them identity experts.
E: 40 heads (more than 32) on a latent of 270 (entries past 256), two taps, values of 130 channels, and of 264, which the delta
   rule's scan takes; no experts.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict

import torch


def _delta(heads, kv, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def _latent(kind, heads, dim, vdim, q_rank, rank, scale, rot=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot[0] if rot else 0, "vdim": vdim, "q_rank": q_rank, "kv_rank": rank, "scale": scale}
    if rot:
        m["rot"] = {"dims": rot[1], "base": rot[2]}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention" if kind == 1 else "latent_attention_2", "mixer": m}


def _dense(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff})


def _moe(layer, experts, identity, top, ff, limit):
    r = {"experts": experts, "top": top}
    if identity:
        r["identity"] = identity
    return dict(layer, mlp={"kind": "moe", "router": r, "expert": {"ff": ff, "limit": limit}})


def _cfg(vocab, width, eps, layers):
    return {"architecture": "Fefozen", "vocab": vocab, "width": width, "max_positions": 1024, "norm": {"eps": eps},
            "layers": [dict({"mlp": None}, **L) for L in layers]}


CONFIGS = {
    "A": _cfg(97, 64, 1e-5,
              [_dense(_delta(4, 2, 12, 20, 4), 48), _moe(_latent(2, 4, 16, 24, 40, 32, 0.3, (8, 8, 300.0)), 6, 2, 2, 24, 1.5),
               _moe(_latent(1, 6, 24, 16, 24, 48, 0.2, (16, 16, 1000.0)), 6, 2, 2, 24, 0.8),
               _latent(2, 2, 32, 12, 32, 32, 0.25, (8, 8, 300.0), kv_from=1)]),
    "B": _cfg(131, 90, 1e-4,
              [_moe(_latent(1, 3, 10, 6, 37, 21, 0.4, (6, 6, 50.0)), 4, 1, 5, 20, 1.0), _dense(_delta(3, 3, 5, 7, 5), 30),
               _moe(_latent(2, 5, 6, 10, 11, 27, 0.35, (10, 10, 80.0)), 4, 1, 5, 20, 0.6)]),
    "C": _cfg(61, 128, 1e-6,
              [_moe(_delta(3, 1, 72, 40, 1), 8, 0, 1, 40, 2.0), _dense(_latent(1, 20, 8, 8, 64, 130, 0.3, (64, 24, 500.0)), 64),
               _moe(_delta(2, 2, 16, 64, 3), 8, 0, 1, 40, 1.0)]),
    "D": _cfg(53, 48, 1e-5,
              [_moe(_latent(2, 1, 16, 16, 16, 16, 0.5), 2, 3, 3, 16, 1.2), _dense(_latent(2, 1, 20, 8, 24, 16, 0.6, None, kv_from=0), 32),
               _moe(_delta(1, 1, 32, 32, 2), 2, 3, 3, 16, 0.9)]),
    "E": _cfg(59, 96, 1e-5,
              [_dense(_latent(1, 40, 4, 4, 80, 270, 0.5, (16, 16, 200.0)), 64), _dense(_delta(2, 1, 8, 130, 2), 40),
               _delta(2, 2, 12, 264, 3)]),
}
PAGE_SIZE = {"A": 4, "B": 2, "C": 16, "D": 8, "E": 12}


def router_outputs(mlp: dict) -> int:
    return mlp["router"]["experts"] + int(mlp["router"].get("identity") or 0)


def reserved(cfg: dict) -> int:
    """The first coordinates of the stream hold a code of the token that only the routers read."""
    return max([router_outputs(L["mlp"]) for L in cfg["layers"] if (L.get("mlp") or {}).get("kind") == "moe"] or [0])


def make_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors by name.  The embedding's first ``reserved`` coordinates are a code of the token's id (levels from 1
    down to -1, the highest at id % outputs); the norms behind the branches multiply by zero there (their weights are stored
    around zero: -1), and a router reads nothing else: a token's experts follow from its id by a wide margin.  The
    corrections move an expert past all others, which brings no two close."""
    g = torch.Generator().manual_seed(seed)
    W, V, R = cfg["width"], cfg["vocab"], reserved(cfg)
    rnd = lambda *shape, std=1.0: torch.randn(*shape, generator=g) * std
    mat = lambda out, inp, gain=1.0: rnd(out, inp, std=gain / math.sqrt(inp))

    def before():                 # a norm ahead of a branch: the code passes with gain one
        w = rnd(W, std=0.2)
        w[:R] = 0.0
        return w

    def behind():
        w = rnd(W, std=0.2)
        w[:R] = -1.0
        return w

    emb = rnd(V, W)
    for t in range(V):
        for e in range(R):
            emb[t, e] = 1.0 - 2.0 * ((e - t) % R) / max(R - 1, 1)
    w = {"embed": emb, "final.norm": rnd(W, std=0.2)}
    for i, L in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", L["mixer"], L.get("mlp")
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        w[p + "norm1"], w[p + "norm1b"] = before(), behind()
        if L["type"] == "delta":
            G, taps = m["kv_heads"], m["conv"]
            # (keys that lean towards the queries: read-outs whose terms cancel would make a rounding a direction)
            q = mat(G * d, W, 1.5)
            flt = lambda n: torch.cat([rnd(n, taps - 1, std=0.4), 1.0 + rnd(n, 1, std=0.2)], dim=1)
            w.update({p + "mix.q": q, p + "mix.k": 0.8 * q + mat(G * d, W, 0.5), p + "mix.v": mat(H * dv, W, 1.5),
                      p + "mix.q.conv": flt(G * d), p + "mix.k.conv": flt(G * d), p + "mix.v.conv": flt(H * dv),
                      p + "mix.b": mat(H, W, 1.5), p + "mix.a": mat(H, W, 1.0), p + "mix.A_log": rnd(H, std=0.5) - 1.5,
                      p + "mix.dt_bias": rnd(H, std=0.5) - 1.0, p + "mix.norm": 1.0 + rnd(dv, std=0.2),
                      p + "mix.g": mat(H * dv, W, 1.5), p + "mix.o": mat(W, H * dv)})
        else:
            r, R_, q_rank = m["rot_dim"], m["kv_rank"], m["q_rank"]
            w.update({p + "mix.dq": mat(q_rank, W), p + "mix.dq.norm": 1.0 + rnd(q_rank, std=0.2),
                      p + "mix.uq": mat(H * (d + r), q_rank, 1.3), p + "mix.uk": mat(H * d, R_, 1.3), p + "mix.uv": mat(H * dv, R_, 1.3),
                      p + "mix.g": mat(H * dv, W, 1.5), p + "mix.o": mat(W, H * dv)})
            if m.get("kv_from") is None:
                w[p + "mix.dkv"], w[p + "mix.dkv.norm"] = mat(R_ + r, W, 1.2), 1.0 + rnd(R_, std=0.2)
            if L["type"] == "latent_attention":
                w[p + "mix.sink"] = rnd(H, std=1.0) + 1.0
        if mlp is None:
            continue
        w[p + "norm2"], w[p + "norm2b"] = before(), behind()
        if mlp["kind"] == "dense":
            w[p + "mlp.up"], w[p + "mlp.down"] = mat(mlp["ff"], W, 1.5), mat(W, mlp["ff"])
            continue
        E, n, F = mlp["router"]["experts"], router_outputs(mlp), mlp["expert"]["ff"]
        router = torch.zeros(n, W)
        for e in range(n):
            router[e, e] = 2.0
        w[p + "mlp.router"] = router
        corr = torch.zeros(n)
        if mlp["router"]["top"] < n:                      # one is chosen always (of several a token), one never
            corr[2 % n] = -2.0
            if mlp["router"]["top"] > 1:
                corr[1] = 2.0
        w[p + "mlp.correction"] = corr
        for e in range(E):
            w[p + f"mlp.e{e}.gate"], w[p + f"mlp.e{e}.up"] = mat(F, W, 1.5), mat(F, W, 1.5)
            w[p + f"mlp.e{e}.down"] = mat(W, F, 1.5)
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
    g = torch.Generator().manual_seed(7300 + seed)
    return torch.randint(0, vocab, (length,), generator=g).tolist()
