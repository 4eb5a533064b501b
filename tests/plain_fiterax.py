"""A plain, slow Fiterax in float64 on the CPU, one function a mechanism, written from the design's equations
and sharing no code with the engine.  ``PlainFiterax(config, tensors)`` runs whole sequences; ``layers=True``
also returns the residual stream after every layer."""
from __future__ import annotations

import math
from typing import Dict, List

import torch

F = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_rms(x, gain, groups, eps):
    """Every one of the ``groups`` equal consecutive parts of a row at unit root mean square, then the gain."""
    parts = x.reshape(x.shape[0], groups, -1)
    return rms(parts, eps).reshape(x.shape) * gain


def input_conv(h, w):
    """h + a causal filter over time on each channel; w [width, taps], the last column meets the row itself."""
    T, taps = h.shape[0], w.shape[1]
    out = h.clone()
    for t in range(T):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * h[s]
    return out


def gelu(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def turn_halves(x, dims, base):
    """x [T, heads, dim]: coordinate i of the first ``dims`` turns with i + dims / 2, by position * base^(-2i/dims)."""
    half = dims // 2
    out = x.clone()
    for t in range(x.shape[0]):
        for i in range(half):
            a = t * base ** (-2.0 * i / dims)
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, :, i], x[t, :, i + half]
            out[t, :, i] = u * c - v * s
            out[t, :, i + half] = v * c + u * s
    return out


def attention(h, w, m, eps):
    T = h.shape[0]
    H, G, d, vd = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T + w["q.b"]).view(T, H, d)
    k = (h @ w["k"].T + w["k.b"]).view(T, G, d)
    v = (h @ w["v"].T + w["v.b"]).view(T, G, vd)
    rot = m.get("rot")
    if rot:
        q, k = turn_halves(q, rot["dims"], rot["base"]), turn_halves(k, rot["dims"], rot["base"])
    q, k = rms(q, eps), rms(k, eps)
    rep = H // G
    k, v = k.repeat_interleave(rep, dim=1), v.repeat_interleave(rep, dim=1)
    s = torch.matmul(q.transpose(0, 1), k.permute(1, 2, 0)) * m["scale"] * w["temp"][:, None, None]
    cap = m.get("softcap")
    if cap:
        s = cap * torch.tanh(s / cap)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    p = torch.softmax(s.masked_fill(~(j <= i)[None], float("-inf")), dim=-1)
    o = torch.matmul(p, v.transpose(0, 1)).transpose(0, 1)            # [T, H, vd]
    o = o * torch.sigmoid(h @ w["g"].T)[:, :, None]
    return o.reshape(T, H * vd) @ w["o"].T + w["o.b"]


def log_gates(h, w, cap):
    """(log input gate, log forget gate) [T, heads]."""
    squash = lambda z: cap * torch.tanh(z / cap)
    i = squash(h @ w["i"].T + w["i.b"])
    f = torch.nn.functional.logsigmoid(squash(h @ w["f"].T + w["f.b"]))
    return i, f


def mlstm_memory(q, k, v, i, f):
    """q, k [T, heads, d] (q already scaled), v [T, heads, vd], log gates [T, heads] -> read-outs [T, heads, vd]."""
    T, H, d = q.shape
    vd = v.shape[2]
    S, n, m = torch.zeros(H, d, vd, dtype=F), torch.zeros(H, d, dtype=F), torch.zeros(H, dtype=F)
    out = torch.zeros(T, H, vd, dtype=F)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, add = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep[:, None, None] * S + add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + add[:, None] * k[t]
        m = m_new
        read = (S * q[t][:, :, None]).sum(1)
        den = torch.maximum((n * q[t]).sum(1).abs(), torch.exp(-m)) + 1e-6
        out[t] = read / den[:, None]
    return out


def mlstm(h, w, m, eps):
    T = h.shape[0]
    H, d, vd = m["heads"], m["dim"], m["vdim"]
    q = (h @ w["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).view(T, H, d)
    v = (h @ w["v"].T).view(T, H, vd)
    i, f = log_gates(h, w, m["gate_cap"])
    o = rms(mlstm_memory(q, k, v, i, f), eps).reshape(T, H * vd)
    return (o * w["norm"] * torch.sigmoid(h @ w["g"].T)) @ w["o"].T


def route(z, correction, top, scale):
    """One token's router logits -> [(expert, weight)], best choice first."""
    s = torch.sigmoid(z)
    chosen = torch.topk(s + correction, top).indices.tolist()
    total = sum(float(s[e]) for e in chosen) + 1e-20
    return [(e, float(s[e]) / total * scale) for e in chosen]


def moe(h, w, mlp):
    r = mlp["router"]
    z = h @ w["router"].T
    out = torch.zeros(h.shape[0], w["e0.down"].shape[0], dtype=F)
    for t in range(h.shape[0]):
        for e, s in route(z[t], w["correction"], r["top"], r["scale"]):
            out[t] += s * (gelu(h[t] @ w[f"e{e}.up"].T) @ w[f"e{e}.down"].T)
    return out


class PlainFiterax:
    def __init__(self, cfg: dict, tensors: Dict[str, torch.Tensor]):
        self.cfg = cfg
        self.t = {k: v.to(F) for k, v in tensors.items()}

    def sub(self, prefix):
        n = len(prefix)
        return {k[n:]: v for k, v in self.t.items() if k.startswith(prefix)}

    def forward(self, tokens: List[int], layers: bool = False):
        cfg, t = self.cfg, self.t
        eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
        x = t["embed"][torch.tensor(tokens)] * cfg["embedding"]["scale"]
        after = []
        for i, L in enumerate(cfg["layers"]):
            wm, wf, mlp = self.sub(f"l{i}.mix."), self.sub(f"l{i}.mlp."), L.get("mlp")
            filtered = bool(cfg.get("canon"))
            read = lambda which: (lambda n: input_conv(n, t[f"l{i}.canon{which}"]) if filtered else n)(
                group_rms(x, t[f"l{i}.norm{which}"], groups, eps))
            mixer = {"attention": attention, "mlstm": mlstm}[L["type"]]
            y = mixer(read(1), wm, L["mixer"], eps)
            if mlp is not None:
                y = y + moe(read(2), wf, mlp)
            x = x + cfg["residual_mult"] * y
            after.append(x.clone())
        logits = group_rms(x, t["final.norm"], groups, eps) @ t["head"].T
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
        return PlainFiterax(cfg, w).forward(list(tokens))


def residual_streams(cfg, w, tokens):
    with torch.no_grad():
        return PlainFiterax(cfg, w).forward(list(tokens), layers=True)[1]


def generate(cfg, w, prompt, n):
    seq, out = list(prompt), []
    for _ in range(n):
        tok = int(logits(cfg, w, seq)[-1].argmax())
        out.append(tok)
        seq.append(tok)
    return out
