"""Grouped softmax attention on unit-length queries and keys, with a factor a head and a cap on the scores and a gate a
head on the results.

    q = Wq x + bq, k = Wk x + bk, v = Wv x + bv          heads x key_dim, kv_heads x key_dim, kv_heads x value_dim
    q, k: the first ``rot_dims`` coordinates of each head turned by the position (i with i + rot_dims / 2), then each
    head divided by its root mean square over key_dim (no gain)
    s = (q_h . k_c(h)) * scale * factor_h;  s <- cap * tanh(s / cap);  softmax over every j <= i
    y = Wo [sigmoid((Wg x)_h) * sum_j p_h(i, j) v_c(h)(j)]_h + bo

One product makes q, k, v and the gate's logits as floats; one kernel turns and normalises queries and keys (with the
head's factor on its queries), rounds to the storage type and writes the pages; the paged attention kernels of
``PagedAttention`` (rows and tiles) run with the cap and multiply by the gate as they store.  Keys and values share one
entry width, the larger of the two sizes padded with zeros to a multiple of 16, and the output matrix gets zero
columns there.  The reference has no such mixer (its attention is src/csrc/layer/attention.cc)."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels as K
from ..weights.loader import TensorSpec
from .attention import PagedAttention, plan_tiles
from .base import CacheNeed
from .position import rotary_frequencies
from .spec import PartSpec


class UnitQueryKeyAttention(PagedAttention):
    """params: num_heads, num_kv_heads, key_dim, value_dim, scale (float), eps (float, of the heads' norm), softcap
    (float, default 0 = none), bias (bool: q, k and v have biases), out_bias (bool), rot_dims (int, 0 = no turn),
    rot_base (float), head_scale (bool: the file holds a factor a head), gate (bool), window (int, default 0), out_scale
    (float, default 1: a factor on the result), tile_min_len (as ``PagedAttention``).  names: q, k, v, out, and
    q_bias, k_bias, v_bias, out_bias, head_scale, gate where asked for."""

    raw_output_ok = True
    accepts_norm = False

    def __init__(self, spec, hidden_size, dtype):
        p = spec.params
        self.key_dim, self.value_dim = int(p["key_dim"]), int(p["value_dim"])
        self.pad = -(-max(self.key_dim, self.value_dim) // 16) * 16
        super().__init__(PartSpec(spec.kind, dict(p, head_dim=self.pad), spec.names), hidden_size, dtype)
        self.spec = spec
        self.bias = bool(p.get("bias", False))
        self.eps = float(p["eps"])
        self.softcap = float(p.get("softcap", 0.0) or 0.0)
        self.out_bias = bool(p.get("out_bias", False))
        self.has_factor = bool(p.get("head_scale", False))
        self.has_gate = bool(p.get("gate", False))
        self.out_scale = float(p.get("out_scale", 1.0))
        rot_dims = int(p.get("rot_dims", 0) or 0)
        if rot_dims % 2 or rot_dims > self.key_dim:
            raise ValueError(f"rotary dims must be even and at most the head size {self.key_dim}, got {rot_dims}")
        self._freq_host = None
        if rot_dims:
            freq, _ = rotary_frequencies(rot_dims, float(self.param("rot_base")))
            self._freq_host = torch.tensor(freq, dtype=torch.float64).to(torch.float32)
        self.freq = self.factor = None

    def tensor_specs(self) -> List[TensorSpec]:
        H = self.hidden_size
        nq, nk, nv = self.num_heads * self.key_dim, self.num_kv_heads * self.key_dim, self.num_kv_heads * self.value_dim
        specs = [TensorSpec(self.name("q"), (nq, H), "matrix"), TensorSpec(self.name("k"), (nk, H), "matrix"),
                 TensorSpec(self.name("v"), (nv, H), "matrix"),
                 TensorSpec(self.name("out"), (H, self.num_heads * self.value_dim), "matrix")]
        if self.bias:
            specs += [TensorSpec(self.name("q_bias"), (nq,), "vector"), TensorSpec(self.name("k_bias"), (nk,), "vector"),
                      TensorSpec(self.name("v_bias"), (nv,), "vector")]
        if self.out_bias:
            specs.append(TensorSpec(self.name("out_bias"), (H,), "vector"))
        if self.has_factor:
            specs.append(TensorSpec(self.name("head_scale"), (self.num_heads,), "vector", init="gain"))
        if self.has_gate:
            specs.append(TensorSpec(self.name("gate"), (self.num_heads, H), "matrix"))
        return specs

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        t = lambda n: tensors[self.name(n)]
        H = self.hidden_size
        # q | k | v | gate, filled up with zero rows to a whole number of the product kernels' tiles
        rows = [t("q"), t("k"), t("v")] + ([t("gate")] if self.has_gate else [])
        self.gate_at = sum(r.shape[0] for r in rows[:3])
        n = sum(r.shape[0] for r in rows)
        dev, total = rows[0].device, -(-n // 16) * 16
        rows.append(torch.zeros((total - n, H), dtype=rows[0].dtype, device=dev))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        self.b_in = None
        if self.bias:
            b = [t("q_bias"), t("k_bias"), t("v_bias")]
            self.b_in = torch.cat(b + [torch.zeros((total - self.gate_at,), dtype=torch.float32, device=dev)]).contiguous()
        w_out = t("out")
        if self.pad != self.value_dim:       # zero columns where the heads are padded
            wide = torch.zeros((H, self.num_heads, self.pad), dtype=w_out.dtype, device=dev)
            wide[:, :, :self.value_dim] = w_out.view(H, self.num_heads, self.value_dim)
            w_out = wide.view(H, self.num_heads * self.pad).contiguous()
        self.w_out = w_out
        # (the bias is multiplied by the factor here: the products add it behind theirs)
        self.b_out = (t("out_bias").to(torch.float64) * self.out_scale).to(torch.float32) if self.out_bias else None
        self.factor = t("head_scale").contiguous() if self.has_factor else None
        self.freq = self._freq_host.to(dev) if self._freq_host is not None else None

    def cache_need(self) -> CacheNeed:
        return CacheNeed("paged_kv", num_kv_heads=self.num_kv_heads, head_dim=self.pad, window=self.window)

    def _tiles_of_64(self) -> bool:
        # capped or gated scores go through the prompt kernel that knows tiles of 64 rows only
        return self.softcap > 0 or self.has_gate

    def plan_key(self):
        return ("attention_tiles", self.tile_min_len, self.num_heads, self.pad, self.dtype, self._tiles_of_64())

    def step_planner(self):
        n, heads, hd, dtype, small = self.tile_min_len, self.num_heads, self.pad, self.dtype, self._tiles_of_64()

        def planner(items, info):
            choose = lambda rows: (K.PREFILL_TILE if small else
                                   K.prefill_tile_rows(hd, info.page_size, info.max_pages, heads, rows, dtype))
            return plan_tiles(items, n, choose, bucketed=info.bucketed)
        return self.plan_key(), planner

    def forward(self, x_t: torch.Tensor, residual32: Optional[torch.Tensor], ctx, cache, write: bool = True) -> torch.Tensor:
        """residual32 + out_scale * mix(x_t) (``residual32`` None: the second alone)."""
        proj = K.gemm(x_t, self.w_in, bias=self.b_in, out_f32=True)
        bt = ctx.block_tables[cache.group]
        q = K.unit_qk_write(proj, self.num_heads, self.num_kv_heads, self.key_dim, self.value_dim, self.eps, self.freq,
                            self.factor, cache.k, cache.v, ctx.token_item, ctx.positions, bt, write=write)
        gate = proj[:, self.gate_at:self.gate_at + self.num_heads] if self.has_gate else None
        T = q.shape[0]
        out = K.empty((T, self.q_size), self.dtype, q.device)
        plan = ctx.plans.get(self.plan_key())
        if plan is not None and K.prefill_available():
            K.attention_prefill(q, cache.k, cache.v, plan.arrays["tile_item"], plan.arrays["tile_q0"],
                                ctx.item_tok_off, ctx.item_start, ctx.item_len, bt, self.num_heads, self.scale,
                                window=self.window, out=out, tile_rows=plan.host["tile_rows"], softcap=self.softcap,
                                head_gate=gate)
            if plan.host["num_short_rows"] > 0:
                splits, waves = self._shape_row_kernel(ctx, plan.host["num_short_rows"])
                K.attention_rows(q, cache.k, cache.v, ctx.token_item, ctx.positions, bt, self.num_heads, self.scale,
                                 window=self.window, row_ids=plan.arrays["short_rows"], num_splits=splits,
                                 num_waves=waves, out=out, softcap=self.softcap, head_gate=gate)
        else:
            splits, waves = self._shape_row_kernel(ctx, T)
            K.attention_rows(q, cache.k, cache.v, ctx.token_item, ctx.positions, bt, self.num_heads, self.scale,
                             window=self.window, num_splits=splits, num_waves=waves, out=out, softcap=self.softcap,
                             head_gate=gate)
        return K.gemm(out, self.w_out, bias=self.b_out, residual=residual32, out_f32=True, out_scale=self.out_scale,
                      bias_unscaled=True)
