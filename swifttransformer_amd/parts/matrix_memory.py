"""Matrix memory with exponential gates (mLSTM): a linear recurrence over a matrix a head whose log gates are kept in
range by a running maximum.

    q = Wq x * key_dim^-1/2, k = Wk x, v = Wv x                         heads x key_dim, heads x value_dim
    i = cap tanh((Wi x + bi) / cap);  f = log sigmoid(cap tanh((Wf x + bf) / cap))          log gates, one a head
    m' = max(f + m, i);  S <- e^(f + m - m') S + e^(i - m') k v^T;  n <- e^(f + m - m') n + e^(i - m') k
    o = S^T q / (max(|n . q|, e^(-m')) + 1e-6)                          S, n and m start at zero
    y = Wo (concat_h(o_h / rms(o_h)) * gain * sigmoid(Wg x))

One product makes q, k, v, the gate's and the log gates' logits as floats.  A step of single tokens then is one kernel
(log gates, state, read-out, norm and gate); other steps go by chunks of rows with products in float on the matrix cores
and a carry of the state between chunks.  State, sums, gates and norm are float; the state (S | n | m, flat) lives in
the request's slot.  The reference has no such mixer."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels as K
from ..weights.loader import TensorSpec
from .base import CacheNeed, Mixer


class MatrixMemory(Mixer):
    """params: num_heads, key_dim, value_dim (up to 256 each), gate_cap (float), eps (float, of the heads' norm),
    out_scale (float, default 1: a factor on the result).  names: q, k, v, gate, in_gate, in_gate_bias, forget_gate,
    forget_gate_bias, norm [heads * value_dim], out."""

    raw_output_ok = True

    def __init__(self, spec, hidden_size, dtype):
        super().__init__(spec, hidden_size, dtype)
        self.num_heads = int(self.param("num_heads"))
        self.key_dim = int(self.param("key_dim"))
        self.value_dim = int(self.param("value_dim"))
        self.gate_cap = float(self.param("gate_cap"))
        self.eps = float(self.param("eps"))
        self.out_scale = float(spec.params.get("out_scale", 1.0))
        if self.key_dim > 256 or self.value_dim > 256:
            raise ValueError(f"a matrix memory has up to 256 key and value channels a head, not {self.key_dim} and "
                             f"{self.value_dim}")
        self.qk_size = self.num_heads * self.key_dim
        self.v_size = self.num_heads * self.value_dim

    def tensor_specs(self) -> List[TensorSpec]:
        H, nh = self.hidden_size, self.num_heads
        return [TensorSpec(self.name("q"), (self.qk_size, H), "matrix"),
                TensorSpec(self.name("k"), (self.qk_size, H), "matrix"),
                TensorSpec(self.name("v"), (self.v_size, H), "matrix"),
                TensorSpec(self.name("gate"), (self.v_size, H), "matrix"),
                TensorSpec(self.name("in_gate"), (nh, H), "matrix"),
                TensorSpec(self.name("in_gate_bias"), (nh,), "vector"),
                TensorSpec(self.name("forget_gate"), (nh, H), "matrix"),
                TensorSpec(self.name("forget_gate_bias"), (nh,), "vector"),
                TensorSpec(self.name("norm"), (self.v_size,), "vector", init="gain"),
                TensorSpec(self.name("out"), (H, self.v_size), "matrix")]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        t = lambda n: tensors[self.name(n)]
        rows = [t(n) for n in ("q", "k", "v", "gate", "in_gate", "forget_gate")]
        n = sum(r.shape[0] for r in rows)
        # (filled up with zero rows to a whole number of the product kernels' tiles)
        rows.append(torch.zeros((-n % 16, self.hidden_size), dtype=rows[0].dtype, device=rows[0].device))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        self.b_i, self.b_f = t("in_gate_bias").contiguous(), t("forget_gate_bias").contiguous()
        self.gain, self.w_out = t("norm").contiguous(), t("out")

    def cache_need(self) -> CacheNeed:
        return CacheNeed("state", state_shape=(K.memory_slot(self.num_heads, self.key_dim, self.value_dim),),
                         state_dtype=torch.float32)

    def forward(self, x_t: torch.Tensor, residual32: Optional[torch.Tensor], ctx, cache, write: bool = True) -> torch.Tensor:
        """residual32 + out_scale * mix(x_t) (``residual32`` None: the second alone)."""
        if not write:
            raise ValueError("a recurrent mixer has no read-only run: its state moves with every token")
        proj = K.gemm(x_t, self.w_in, out_f32=True)
        y = K.matrix_memory(proj, self.b_i, self.b_f, self.gain, cache.state,
                            (ctx.token_item, ctx.item_len, ctx.item_tok_off, ctx.item_slot), self.num_heads, self.key_dim,
                            self.value_dim, self.gate_cap, self.eps, self.dtype, all_single=bool(ctx.all_single))
        return K.gemm(y, self.w_out, residual=residual32, out_f32=True, out_scale=self.out_scale)
