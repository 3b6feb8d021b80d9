"""A recurrent mixer with a state of its own for every channel and state number, its decays and inputs selected by the token."""

from __future__ import annotations

import math
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


class SelectiveScan:
    """[x | z] = Win h, one product left in 32 bits; x <- silu(conv(x) + bias) over the request's own rows in time, rounded to the compute dtype
    for the product [low | B | C] = Wx x (kept 32-bit); dt = softplus(Wdt low + bias), a 32-bit product of unrounded rows, since a decay is multiplied by itself
    over hundreds of tokens; S[c, n] <- exp(-dt_c exp(A_log[c, n])) S[c, n] + dt_c x_c B_n, y_c = sum_n S[c, n] C_n + D_c x_c, all 32-bit; the rows y *
    silu(z) are rounded once, for the output projection. A request's slot holds S [states, channels] and behind it the last taps - 1 rows of x before
    the convolution (position p at ring place p % (taps - 1)), 32-bit."""

    replayable = True
    takes_padding_rows = True  # (the recurrence walks the requests' own rows; rows behind them are computed by the products only)

    def __init__(self, spec, store, dtype: torch.dtype):
        self.dtype = dtype
        self.width, self.inner, self.n_state, self.rank, self.taps = spec.width, spec.inner, spec.n_state, spec.dt_rank, int(spec.taps)
        W, N, R, d = self.inner, self.n_state, self.rank, self.width
        if not 1 <= N <= ops.SELECTIVE_MAX_STATES:
            raise Unsupported(f"selective scan: {N} states a channel are not supported (up to {ops.SELECTIVE_MAX_STATES})")
        if self.taps < 1:
            raise ValueError(f"selective scan: a convolution of {self.taps} taps")
        t = spec.tensors
        self.in_weight = store.fetch(t["in"], (2 * W, d), "matrix")
        self.conv = store.fetch(t["conv"], (W, self.taps), "vector")
        self.conv_bias = store.fetch(t["conv_bias"], (W,), "vector")
        self.x_weight = store.fetch(t["x"], (R + 2 * N, W), "matrix")
        dt = store.fetch(t["dt"], (W, R), "matrix")
        # [rank, channels]: a row's channels side by side, as a step of single tokens reads them; and rows of a multiple of eight
        self.dt_weight_t = store.derived(("rank_first", t["dt"].name), lambda: dt.t().contiguous())
        self.dt_weight = store.derived(("rows_of_eights", t["dt"].name), lambda: torch.nn.functional.pad(dt, (0, -R % 8)).contiguous())
        self.low_stride = -(-max(R + 2 * N, self.dt_weight.shape[1]) // 4) * 4
        self.dt_bias = store.fetch(t["dt_bias"], (W,), "vector")
        a_log = store.fetch(t["A_log"], (W, N), "vector")
        # [states, channels], times log2(e): a decay is 2^(dt a)
        self.a2 = store.derived(("decay_rates", t["A_log"].name), lambda: (a_log.double().exp() * -math.log2(math.e)).t().float().contiguous())
        self.skip = store.fetch(t["D"], (W,), "vector")
        self.out_weight = store.fetch(t["out"], (d, W), "matrix")

    def _floats(self) -> int:
        return (self.n_state + self.taps - 1) * self.inner

    def cache_spec(self):
        return None

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self._floats(),))

    def forward(self, h, ctx: StepContext, cache, state, residual: Optional[torch.Tensor], writes_cache: bool = True,
                out: Optional[torch.Tensor] = None):
        if not writes_cache:
            raise Unsupported("selective scan: a run that leaves the state as it found it is not supported")
        h = as_tensor(h)
        n, ws, W, N = h.shape[0], ctx.workspace, self.inner, self.n_state
        own = own_state(state, self._floats())
        proj = ws.get("selective_in", (n, 2 * W), torch.float32)
        linear(h, self.in_weight, None, out=proj)
        raw, z = proj[:, :W], proj[:, W:]
        x = ws.get("selective_x", (n, W), self.dtype)
        ops.conv_act(x, raw, self.conv, self.conv_bias, own.state, own.offset + N * W, ctx)
        low = ws.get("selective_low", (n, self.low_stride), torch.float32)[:, :self.rank + 2 * N]
        linear(x, self.x_weight, None, out=low)
        y = ws.get("selective_out", (n, W), self.dtype)
        # (the walk also keeps the step's last rows of x in the slot's ring: the convolution, which reads the ring, has run)
        ops.selective_scan(y, x, low, z, self.dt_weight, self.dt_weight_t, self.dt_bias, self.a2, self.skip, own, raw, self.taps, ctx)
        if out is not None:
            linear(y, self.out_weight, None, out=out)
        else:
            linear(y, self.out_weight, None, residual=settled(residual))
        return None


register_mixer("selective_scan", SelectiveScan)
