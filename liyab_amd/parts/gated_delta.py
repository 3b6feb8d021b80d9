"""A delta rule whose state decays by one number a head and token, behind a short convolution on its inputs."""

from __future__ import annotations

from typing import Optional

import torch

from ..cache.pages import StateSpec
from ..errors import Unsupported
from ..kernels import ops
from .base import StepContext, settled
from .delta_rule import own_state
from .linear import linear
from .norms import as_tensor
from .registry import register_mixer


class GatedDelta:
    """q, k, v = silu(conv(W h)) a channel over time; q and k of a head to length one, q times q_scale; beta = sigmoid(Wb h), g =
    exp(-exp(A_log) softplus(Wa h + dt_bias)); S <- g S, S <- S + k (beta (v - S^T k))^T, o = S^T q; each head's o brought to unit root
    mean square, times a weight shared by the heads and silu(Wg h), then the output projection. The six projections of h run as one
    product whose 32-bit sums feed everything up to the rows the output projection reads, which are rounded once. A request's slot holds
    the heads' matrices [heads, key, value] and, with more than one tap, the ring of the convolution's inputs (`ops.gated_delta_floats`)."""

    replayable = True
    takes_padding_rows = True  # (the recurrence walks the requests' own rows; rows behind them are computed by the products only)

    def __init__(self, spec, store, dtype: torch.dtype):
        self.dtype = dtype
        self.width, self.n_head, self.n_kv_head = spec.width, spec.n_head, spec.n_kv_head
        self.head_dim, self.value_dim, self.taps = spec.head_dim, spec.value_dim, int(spec.taps)
        self.eps, self.key_eps, self.q_scale = float(spec.eps), float(spec.key_eps), float(spec.q_scale)
        H, G, D, V, d = self.n_head, self.n_kv_head, self.head_dim, self.value_dim, self.width
        if H % G:
            raise ValueError(f"gated delta rule: {H} heads are no multiple of {G}")
        if not ops.gated_delta_takes(D, V) or not 1 <= self.taps <= ops.GATED_DELTA_MAX_TAPS:
            raise Unsupported(f"gated delta rule: keys of {D} / values of {V} / {self.taps} taps are not supported (up to 256 / 256 / {ops.GATED_DELTA_MAX_TAPS})")
        t = spec.tensors
        # [q | k | v | gate | rate | decay] of one input
        self.in_weight = store.fetch_joined([t[c] for c in ("q", "k", "v", "g", "b", "a")],
                                            [(G * D, d), (G * D, d), (H * V, d), (H * V, d), (H, d), (H, d)], "matrix", "rows")
        conv = store.fetch_joined([t[c + "_conv"] for c in "qkv"], [(G * D, self.taps), (G * D, self.taps), (H * V, self.taps)], "vector", "rows")
        # [taps, channels]: a tap's channels side by side, as the kernels read them
        self.conv = store.derived(("taps_first",) + tuple(t[c + "_conv"].name for c in "qkv"), lambda: conv.t().contiguous())
        self.a_log = store.fetch(t["A_log"], (H,), "vector")
        self.dt_bias = store.fetch(t["dt_bias"], (H,), "vector")
        self.norm = store.fetch(t["norm"], (V,), "vector")
        self.out_weight = store.fetch(t["out"], (d, H * V), "matrix")

    def _floats(self) -> int:
        return ops.gated_delta_floats(self.n_head, self.n_kv_head, self.head_dim, self.value_dim, self.taps)

    def cache_spec(self):
        return None

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self._floats(),))

    def forward(self, h, ctx: StepContext, cache, state, residual: Optional[torch.Tensor], writes_cache: bool = True,
                out: Optional[torch.Tensor] = None):
        h = as_tensor(h)
        n, ws = h.shape[0], ctx.workspace
        proj = ws.get("gated_delta_in", (n, self.in_weight.shape[0]), torch.float32)
        linear(h, self.in_weight, None, out=proj)
        y = ws.get("gated_delta_out", (n, self.n_head * self.value_dim), self.dtype)
        ops.gated_delta(y, proj, self.conv, self.a_log, self.dt_bias, self.norm, self.eps, own_state(state, self._floats()), ctx, n_head=self.n_head,
                        n_kv_head=self.n_kv_head, head_dim=self.head_dim, value_dim=self.value_dim, key_eps=self.key_eps, q_scale=self.q_scale)
        if out is not None:
            linear(y, self.out_weight, None, out=out)
        else:
            linear(y, self.out_weight, None, residual=settled(residual))
        return None


register_mixer("gated_delta", GatedDelta)
