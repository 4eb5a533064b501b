"""A plain, slow Fefozen in float64 on the CPU, one function a mechanism, written from the design's equations
and sharing no code with the engine.  ``PlainFefozen(config, tensors)`` runs whole sequences; ``layers=True``
also returns the residual stream after every layer."""
from __future__ import annotations

import math
from typing import Dict, List

import torch

F = torch.float64


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def shifted_rms(x, w, eps):
    """The norm whose weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def turn(x, dims, base, neighbours):
    """x [T, ..., n]: pairs of the first ``dims`` coordinates turn by position * base^(-2i/dims); pair i is
    (2i, 2i + 1) for ``neighbours``, else (i, i + dims / 2)."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=F).reshape([-1] + [1] * (x.dim() - 2))
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        iu, iv = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        u, v = x[..., iu], x[..., iv]
        out[..., iu] = u * torch.cos(a) - v * torch.sin(a)
        out[..., iv] = v * torch.cos(a) + u * torch.sin(a)
    return out


def turned(x, m, neighbours):
    return turn(x, m["rot"]["dims"], m["rot"]["base"], neighbours) if m["rot_dim"] else x


def latent(h, w, m, eps, neighbours):
    """What a latent attention caches of every token: (latent [T, rank], turned key part [T, rot_dim])."""
    raw = h @ w["dkv"].T
    c = unit_rms(raw[:, :m["kv_rank"]], eps) * w["dkv.norm"]
    return c, turned(raw[:, m["kv_rank"]:], m, neighbours)


def softmax_with_sink(s, sink=None):
    """s [H, T, S]; ``sink`` [H]: one more term exp(sink_h) in the denominator."""
    top = s.max(-1, keepdim=True).values
    if sink is not None:
        top = torch.maximum(top, sink[:, None, None])
    p = torch.exp(s - top)
    total = p.sum(-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink[:, None, None] - top)
    return p / total


def latent_attention(h, w, m, eps, cached, neighbours, sink=None):
    """``cached``: (latent, turned key part), this layer's own or a borrowed one."""
    T = h.shape[0]
    H, d, r, vd = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = ((unit_rms(h @ w["dq"].T, eps) * w["dq.norm"]) @ w["uq"].T).view(T, H, d + r)
    qn, qr = q[..., :d], turned(q[..., d:], m, neighbours)
    c, kr = cached
    kn, v = (c @ w["uk"].T).view(T, H, d), (c @ w["uv"].T).view(T, H, vd)
    s = (torch.matmul(qn.transpose(0, 1), kn.permute(1, 2, 0)) + torch.matmul(qr.transpose(0, 1), kr.T)) * m["scale"]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    p = softmax_with_sink(s.masked_fill(~(j <= i)[None], float("-inf")), sink)
    o = torch.matmul(p, v.transpose(0, 1)).transpose(0, 1).reshape(T, H * vd)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def short_filter(x, w):
    """silu of a causal filter over time a channel; w [channels, taps], the last column meets the token itself."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * x[:T - back]
    return y * torch.sigmoid(y)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_memory(q, k, v, beta, g):
    """q, k [T, H, d], v [T, H, vd], beta, g [T, H] -> read-outs [T, H, vd]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=F)
    out = torch.zeros(T, H, v.shape[2], dtype=F)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def delta(h, w, m, eps):
    T = h.shape[0]
    H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (short_filter(h @ w[n].T, w[n + ".conv"]) for n in "qkv")
    rep = H // G
    q = unit_vector(q.view(T, G, d)).repeat_interleave(rep, dim=1) * d ** -0.5
    k = unit_vector(k.view(T, G, d)).repeat_interleave(rep, dim=1)
    beta = torch.sigmoid(h @ w["b"].T)
    g = torch.exp(-torch.exp(w["A_log"]) * torch.nn.functional.softplus(h @ w["a"].T + w["dt_bias"]))
    o = delta_memory(q, k, v.view(T, H, vd), beta, g)
    gate = (h @ w["g"].T).view(T, H, vd)
    return (unit_rms(o, eps) * w["norm"] * gate * torch.sigmoid(gate)).reshape(T, H * vd) @ w["o"].T


def dense(h, w):
    return gelu_tanh(h @ w["up"].T) @ w["down"].T


def route(z, correction, top):
    """One token's router logits -> [(choice, weight)], best choice first."""
    s = torch.softmax(z, 0)
    return [(e, float(s[e])) for e in torch.topk(s + correction, top).indices.tolist()]


def expert(h, gate, up, down, limit):
    a = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, -limit, limit)
    return (a * torch.sigmoid(1.702 * a) * (u + 1.0)) @ down.T


def moe(h, w, mlp):
    r, limit = mlp["router"], mlp["expert"]["limit"]
    z = h @ w["router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, s in route(z[t], w["correction"], r["top"]):
            if e >= r["experts"]:                        # an identity expert
                out[t] += s * h[t]
            else:
                out[t] += s * expert(h[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], limit)
    return out


class PlainFefozen:
    def __init__(self, cfg: dict, tensors: Dict[str, torch.Tensor]):
        self.cfg = cfg
        self.t = {k: v.to(F) for k, v in tensors.items()}

    def sub(self, prefix):
        n = len(prefix)
        return {k[n:]: v for k, v in self.t.items() if k.startswith(prefix)}

    def forward(self, tokens: List[int], layers: bool = False):
        cfg, t, eps = self.cfg, self.t, self.cfg["norm"]["eps"]
        x = t["embed"][torch.tensor(tokens)]
        after, cached = [], {}
        for i, L in enumerate(cfg["layers"]):
            m, w = L["mixer"], self.sub(f"l{i}.mix.")
            norm = lambda which, y: shifted_rms(y, t[f"l{i}.norm{which}"], eps)
            h = norm("1", x)
            if L["type"] == "delta":
                y = delta(h, w, m, eps)
            else:
                neighbours = L["type"] == "latent_attention"
                j = m.get("kv_from")
                if j is None:
                    cached[i] = latent(h, w, m, eps, neighbours)
                y = latent_attention(h, w, m, eps, cached[i if j is None else j], neighbours,
                                     w["sink"] if L["type"] == "latent_attention" else None)
            x = x + norm("1b", y)
            mlp = L.get("mlp")
            if mlp is not None:
                h, w = norm("2", x), self.sub(f"l{i}.mlp.")
                x = x + norm("2b", dense(h, w) if mlp["kind"] == "dense" else moe(h, w, mlp))
            after.append(x.clone())
        logits = shifted_rms(x, t["final.norm"], eps) @ t["embed"].T
        return (logits, torch.stack(after)) if layers else logits


def load_folder(folder: str):
    """(config, float64 tensors by name) of a model folder, through this file's own reader."""
    import json
    import os
    import struct
    import numpy as np
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    with open(os.path.join(folder, "model.safetensors"), "rb") as f:
        n = struct.unpack("<Q", f.read(8))[0]
        meta = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, m in meta.items():
        if name == "__metadata__":
            continue
        a, b = m["data_offsets"]
        raw = np.frombuffer(data[a:b], dtype=np.uint8)
        if m["dtype"] == "BF16":
            u = raw.view("<u2").astype(np.uint32) << 16
            t = torch.from_numpy(u.view(np.float32).copy())
        elif m["dtype"] == "F32":
            t = torch.from_numpy(raw.view("<f4").copy())
        else:
            raise ValueError(m["dtype"])
        out[name] = t.reshape(m["shape"]).to(F)
    return cfg, out


def logits(cfg, w, tokens):
    with torch.no_grad():
        return PlainFefozen(cfg, w).forward(list(tokens))


def residual_streams(cfg, w, tokens):
    with torch.no_grad():
        return PlainFefozen(cfg, w).forward(list(tokens), layers=True)[1]


def generate(cfg, w, prompt, n):
    seq, out = list(prompt), []
    for _ in range(n):
        tok = int(logits(cfg, w, seq)[-1].argmax())
        out.append(tok)
        seq.append(tok)
    return out
