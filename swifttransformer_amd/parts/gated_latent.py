"""Latent attention whose queries go through a latent of their own and whose heads are gated before the output product.

    c_q = rmsnorm(Wdq x) * gain_q;  q = Wuq c_q                  per head [key_dim plain | rot_dim turned]
    c | r = Wdkv x;  c <- rmsnorm(c) * gain;  r <- turned by the token's position          (both are cached, r shared by heads)
    score_h = (q_plain . Wuk_h c + q_turned . r) * scale;  causal softmax, with a sink: one more term exp(sink_h) in the
    denominator;  o_h = Wuv_h (sum of the c's);  y = Wo (concat(o_h) * sigmoid(Wg x))

Wuk is folded into Wuq when the weights are bound (q'_h = [Wuk_h^T Wuq_h,plain | Wuq_h,turned], in float64, rounded once), so
attention runs against the cached entries themselves, one for all heads, and only c and r are cached.  The gate stands between
Wuv and Wo, so Wuv stays a product of its own, one matrix a head, which also merges the key splits of decoded tokens and
applies the gate (``latent_up``).  Wdq, Wdkv and Wg are one product with float results.

A turned pair is two neighbouring coordinates (2i, 2i + 1) in cache and queries; where a design pairs coordinate i with
i + rot_dims / 2, the rows of Wuq and Wdkv that make the turned part are reordered when the weights are bound: a score is a
sum over coordinates in any order.  A layer may read the entries of an earlier layer (``own_latent`` False).  The reference
has no such mixer."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels as K
from ..weights.loader import TensorSpec
from .attention import _target_workgroups, plan_tiles
from .base import CacheNeed, Mixer
from .position import rotary_frequencies


class GatedLatentAttention(Mixer):
    """params: num_heads, key_dim, value_dim, q_rank, rank, rot_dim (even), scale (float), eps (of both latents' norms), rot_dims
    (default rot_dim: the first coordinates of the turned part that turn), rot_base, rot_scaling (None or a rule of
    ``rotary_frequencies``), rot_layout ("interleaved": pairs (2i, 2i + 1), or "halves": (i, i + rot_dims / 2)), sink (bool),
    gate (bool, default True), own_latent (bool, default True), window (int, default 0), tile_min_len (int, default 8: portions
    from this many tokens on go by tiles).  names: q_down, q_norm, q_up, up_k, up_v, out; gate, sink; down, down_norm with a
    latent of its own."""

    raw_output_ok = True

    def __init__(self, spec, hidden_size, dtype):
        super().__init__(spec, hidden_size, dtype)
        p = spec.params
        self.num_heads = int(self.param("num_heads"))
        self.key_dim, self.value_dim = int(self.param("key_dim")), int(self.param("value_dim"))
        self.q_rank, self.rank, self.rot_dim = int(self.param("q_rank")), int(self.param("rank")), int(p.get("rot_dim", 0) or 0)
        self.scale, self.eps = float(self.param("scale")), float(self.param("eps"))
        self.sink, self.gate = bool(p.get("sink", False)), bool(p.get("gate", True))
        self.own_latent = bool(p.get("own_latent", True))
        self.window = int(p.get("window", 0) or 0)
        self.tile_min_len = int(p.get("tile_min_len", 8))
        self.rot_layout = str(p.get("rot_layout", "interleaved"))
        if self.rot_dim % 2 or self.rot_layout not in ("interleaved", "halves"):
            raise ValueError(f"a turned part of {self.rot_dim} coordinates in the layout {self.rot_layout!r}")
        # an entry: the latent, zeros up to a multiple of 8, the turned part, zeros up to a multiple of 16
        self.tail_off = -(-self.rank // 8) * 8 if self.rot_dim else self.rank
        self.entry = -(-(self.tail_off + self.rot_dim) // 16) * 16
        self.out_dim = -(-self.rank // 16) * 16
        self.q_width = -(-self.q_rank // 16) * 16
        if self.entry > MAX_ENTRY:
            raise ValueError(f"the latent attention kernels take cached entries of up to {MAX_ENTRY} numbers, not {self.entry}")
        self._freq_host, self.rot_mult, self.pair_order = None, 1.0, list(range(self.rot_dim))
        if self.rot_dim:
            dims = int(p.get("rot_dims", self.rot_dim) or self.rot_dim)
            if dims % 2 or not 0 < dims <= self.rot_dim:
                raise ValueError(f"{dims} turning coordinates in a part of {self.rot_dim}")
            freq, self.rot_mult = rotary_frequencies(dims, float(p["rot_base"]), p.get("rot_scaling"))
            self._freq_host = torch.tensor(freq, dtype=torch.float64).to(torch.float32)
            if self.rot_layout == "halves":
                self.pair_order = [c for i in range(dims // 2) for c in (i, i + dims // 2)] + list(range(dims, self.rot_dim))
            if self.rot_mult != 1.0 and dims < self.rot_dim:
                raise ValueError("a factor on cosine and sine goes with a part that turns as a whole")

    def tensor_specs(self) -> List[TensorSpec]:
        H, nh = self.hidden_size, self.num_heads
        specs = [TensorSpec(self.name("q_down"), (self.q_rank, H), "matrix"),
                 TensorSpec(self.name("q_norm"), (self.q_rank,), "vector", init="gain"),
                 TensorSpec(self.name("q_up"), (nh * (self.key_dim + self.rot_dim), self.q_rank), "matrix"),
                 TensorSpec(self.name("up_k"), (nh * self.key_dim, self.rank), "matrix"),
                 TensorSpec(self.name("up_v"), (nh * self.value_dim, self.rank), "matrix"),
                 TensorSpec(self.name("out"), (H, nh * self.value_dim), "matrix")]
        if self.own_latent:
            specs += [TensorSpec(self.name("down"), (self.rank + self.rot_dim, H), "matrix"),
                      TensorSpec(self.name("down_norm"), (self.rank,), "vector", init="gain")]
        if self.gate:
            specs.append(TensorSpec(self.name("gate"), (nh * self.value_dim, H), "matrix"))
        if self.sink:
            specs.append(TensorSpec(self.name("sink"), (nh,), "vector"))
        return specs

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        t = lambda n: tensors[self.name(n)]
        nh, d, r, R, E, wide = self.num_heads, self.key_dim, self.rot_dim, self.rank, self.entry, torch.float64
        q_down = t("q_down")
        dev = q_down.device
        order = torch.tensor(self.pair_order, dtype=torch.long, device=dev)
        uq = t("q_up").to(wide).view(nh, d + r, self.q_rank)
        uk = t("up_k").to(wide).view(nh, d, R)
        w_q = torch.zeros((nh, E, self.q_width), dtype=wide, device=dev)
        for h in range(nh):
            w_q[h, :R, :self.q_rank] = uk[h].T @ uq[h, :d]
        if r:
            w_q[:, self.tail_off:self.tail_off + r, :self.q_rank] = uq[:, d:][:, order]
        self.w_q = w_q.view(nh * E, self.q_width).to(self.dtype).contiguous()
        self.w_v = torch.nn.functional.pad(t("up_v").view(nh, self.value_dim, R), (0, self.out_dim - R)).contiguous()
        rows = [q_down]
        if self.own_latent:
            down = t("down")
            rows += [down[:R], down[R:][order]]
            self.gain = t("down_norm").contiguous()
        used = sum(x.shape[0] for x in rows)
        if self.gate:          # (from a multiple of 4 floats on, so that the gate is read in 16-byte pieces)
            rows.append(torch.zeros((-used % 4, self.hidden_size), dtype=q_down.dtype, device=dev))
            self.gate_off = used + (-used % 4)
            rows.append(t("gate"))
        n = sum(x.shape[0] for x in rows)
        rows.append(torch.zeros((-n % 16, self.hidden_size), dtype=q_down.dtype, device=dev))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        self.gain_q, self.w_out = t("q_norm").contiguous(), t("out")
        self.freq = self._freq_host.to(dev) if self._freq_host is not None else None
        self.shape = K.LatentShape(nh, E, self.out_dim, self.scale, self.tail_off, self.freq, self.rot_mult,
                                   t("sink").contiguous() if self.sink else None, self.window)

    def cache_need(self) -> CacheNeed:
        return CacheNeed("paged_kv", num_kv_heads=1, head_dim=self.entry, window=self.window, values=False)

    def plan_key(self):
        return ("latent_tiles", self.tile_min_len)

    def step_planner(self):
        n = self.tile_min_len
        return self.plan_key(), lambda items, info: plan_tiles(items, n, 64, bucketed=info.bucketed)

    def _splits(self, ctx, rows: int) -> int:
        """Shares of the keys in steps of ``rows`` single tokens: enough workgroups for every compute unit (a workgroup
        takes up to 32 heads), of at least 128 keys each."""
        span = ctx.max_kv_len if self.window <= 0 else min(ctx.max_kv_len, self.window)
        groups = max(1, rows * -(-self.num_heads // 32))
        return max(1, min(-(-_target_workgroups() // groups), -(-span // 128), 32))

    def forward(self, x_t: torch.Tensor, residual32: Optional[torch.Tensor], ctx, cache, write: bool = True) -> torch.Tensor:
        """residual32 + mix(x_t) (``residual32`` None: the second alone)."""
        if write != self.own_latent:
            raise ValueError("a latent attention writes the cache it owns and only reads a borrowed one")
        T, bt = x_t.shape[0], ctx.block_tables[cache.group]
        raw = K.gemm(x_t, self.w_in, out_f32=True)
        gate = raw[:, self.gate_off:self.gate_off + self.num_heads * self.value_dim] if self.gate else None
        own = dict(cache=cache.k, gain=self.gain, rank=self.rank, tail_off=self.tail_off, tail=self.rot_dim, tail_freq=self.freq,
                   tail_mult=self.rot_mult, ctx_arrays=(ctx.token_item, ctx.positions, bt)) if write else {}
        q = K.gemm(K.latent_inputs(raw, self.q_rank, self.q_width, self.gain_q, self.eps, dtype=self.dtype, **own), self.w_q)
        plan = ctx.plans.get(self.plan_key())
        if plan is None:       # single tokens and short portions: the product a head merges the shares
            o = K.latent_rows(q, cache.k, ctx.token_item, ctx.positions, bt, self.shape, self._splits(ctx, T))
            y = K.latent_up(o, self.w_v, gate, ctx.token_item)
        else:
            o = K.empty((T, self.num_heads * self.out_dim), self.dtype, q.device)
            K.latent_tiles(q, cache.k, plan.arrays["tile_item"], plan.arrays["tile_q0"], ctx.item_tok_off, ctx.item_start,
                           ctx.item_len, bt, self.shape, o)
            n = plan.host["num_short_rows"]
            if n > 0:
                rows = plan.arrays["short_rows"]
                part = K.latent_rows(q, cache.k, ctx.token_item, ctx.positions, bt, self.shape, self._splits(ctx, n), rows)
                K.latent_merge(part, o, rows)
            y = K.latent_up(o, self.w_v, gate)
        return K.gemm(y, self.w_out, residual=residual32, out_f32=True)


MAX_ENTRY = 576      # of the kernels (``K.latent_max_entry()`` says the same; a model is laid out without the library)
