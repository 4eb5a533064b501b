"""The gated delta rule with everything between its two products in few kernels.

    q, k, v = silu(conv(Wq x)), silu(conv(Wk x)), silu(conv(Wv x))       short causal filters a channel over time
    q, k <- unit vectors (eps under the root), q <- q / sqrt(key_dim)     heads share q and k in groups of neighbours
    b = sigmoid(Wb x);   g = exp(-exp(a_log) softplus(Wa x + dt_bias))   one of each a head
    S <- g S;  u = b (v - S^T k);  S <- S + k u^T;  o = S^T q            S [key_dim, value_dim] a head, starts at zero
    y = Wo (concat_h(o_h / rms(o_h) * gain) * silu(Wg x))                gain [value_dim], shared by heads

The same mathematics as ``GatedDeltaRule`` (a kernel a mechanism, the scan over single tokens): here one product makes q, k, v,
the gate and the logits of b and g as floats, a step of single tokens then is one kernel, and other steps go by chunks of rows
with float products on the matrix cores and a carry of the state between chunks.  Filter, unit vectors, gates, state, sums and
norm are float; the state (a ring of the filter's last inputs | S, flat) lives in the request's slot.  The reference has no
such mixer."""
from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import kernels as K
from ..weights.loader import TensorSpec
from .base import CacheNeed, Mixer


class FusedDeltaRule(Mixer):
    """params: num_heads, num_qk_heads (default num_heads), key_dim, value_dim (up to 256 each), taps (1 to 8), eps (of the
    heads' norm), unit_eps (of the unit vectors, default 1e-6).  names: q, k, v, gate, q_conv, k_conv, v_conv [channels, taps],
    write, decay, a_log, dt_bias, norm [value_dim], out."""

    raw_output_ok = True

    def __init__(self, spec, hidden_size, dtype):
        super().__init__(spec, hidden_size, dtype)
        self.num_heads = int(self.param("num_heads"))
        self.num_qk_heads = int(self.param("num_qk_heads", self.num_heads))
        self.key_dim, self.value_dim, self.taps = int(self.param("key_dim")), int(self.param("value_dim")), int(self.param("taps"))
        self.eps, self.unit_eps = float(self.param("eps")), float(spec.params.get("unit_eps", 1e-6))
        if self.num_heads % self.num_qk_heads:
            raise ValueError(f"{self.num_heads} heads do not divide over {self.num_qk_heads} query/key heads")
        if self.key_dim > 256 or self.value_dim > 256 or not 1 <= self.taps <= 8:
            raise ValueError(f"a delta rule has up to 256 key and value channels a head and 1 to 8 taps, not {self.key_dim}, "
                             f"{self.value_dim} and {self.taps}")
        self.qk_size, self.v_size = self.num_qk_heads * self.key_dim, self.num_heads * self.value_dim
        self.sizes = (self.num_heads, self.num_qk_heads, self.key_dim, self.value_dim)

    def tensor_specs(self) -> List[TensorSpec]:
        H, nh = self.hidden_size, self.num_heads
        return [TensorSpec(self.name("q"), (self.qk_size, H), "matrix"),
                TensorSpec(self.name("k"), (self.qk_size, H), "matrix"),
                TensorSpec(self.name("v"), (self.v_size, H), "matrix"),
                TensorSpec(self.name("gate"), (self.v_size, H), "matrix"),
                TensorSpec(self.name("q_conv"), (self.qk_size, self.taps), "vector"),
                TensorSpec(self.name("k_conv"), (self.qk_size, self.taps), "vector"),
                TensorSpec(self.name("v_conv"), (self.v_size, self.taps), "vector"),
                TensorSpec(self.name("write"), (nh, H), "matrix"),
                TensorSpec(self.name("decay"), (nh, H), "matrix"),
                TensorSpec(self.name("a_log"), (nh,), "vector"),
                TensorSpec(self.name("dt_bias"), (nh,), "vector"),
                TensorSpec(self.name("norm"), (self.value_dim,), "vector", init="gain"),
                TensorSpec(self.name("out"), (H, self.v_size), "matrix")]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        t = lambda n: tensors[self.name(n)]
        rows = [t(n) for n in ("q", "k", "v", "gate", "write", "decay")]
        n = sum(r.shape[0] for r in rows)
        # (filled up with zero rows to a whole number of the product kernels' tiles)
        rows.append(torch.zeros((-n % 16, self.hidden_size), dtype=rows[0].dtype, device=rows[0].device))
        self.w_in = torch.cat(rows, dim=0).contiguous()
        self.taps_w = torch.cat([t("q_conv"), t("k_conv"), t("v_conv")], dim=0).T.contiguous()      # by tap
        self.a_log, self.dt_bias, self.gain = t("a_log").contiguous(), t("dt_bias").contiguous(), t("norm").contiguous()
        self.w_out = t("out")

    def cache_need(self) -> CacheNeed:
        return CacheNeed("state", state_shape=(K.delta_slot(*self.sizes, self.taps),), state_dtype=torch.float32)

    def forward(self, x_t: torch.Tensor, residual32: Optional[torch.Tensor], ctx, cache, write: bool = True) -> torch.Tensor:
        """residual32 + mix(x_t) (``residual32`` None: the second alone)."""
        if not write:
            raise ValueError("a recurrent mixer has no read-only run: its state moves with every token")
        proj = K.gemm(x_t, self.w_in, out_f32=True)
        y = K.delta_rule(proj, self.taps_w, self.a_log, self.dt_bias, self.gain, cache.state,
                         (ctx.token_item, ctx.positions, ctx.item_len, ctx.item_tok_off, ctx.item_slot), *self.sizes, self.eps,
                         self.unit_eps, self.dtype, all_single=bool(ctx.all_single))
        return K.gemm(y, self.w_out, residual=residual32, out_f32=True)
