"""A feed-forward that routes each token to a few of many experts."""

from __future__ import annotations

from typing import Optional

import torch

from ..errors import Unsupported
from ..kernels import ops
from .base import StepContext, settled
from .linear import linear
from .norms import as_tensor
from .registry import register_ffn


class RoutedFFN:
    """z = Wr h + b (32-bit sums, kept in 32 bits); a token takes the `top` experts with the largest z,
    weighted by the softmax over those logits alone; expert e gives Wdown_e (silu(Wgate_e h) * (Wup_e
    h)); the result is the weighted sum. The step's (token, choice) entries are listed by expert in
    tiles, and two grouped products run over the tiles: [gate | up] with the activation, then down
    with the router's weight; an entry's row is added to the others of its token by the reader.
    The spec's options: experts without a gate, Wdown_e act(Wup_e h), with act = the square of the positive part; the choice
    among groups of experts (scores by a softmax over all experts, the best groups only, weights divided by their sum:
    `ops.moe_route(groups=)`); scores by the logistic function, or a softmax over all experts, with a correction on the choice
    (`ops.moe_route(scores=)`); gated units whose halves are clamped; identity experts, which are router outputs without tensors: their entries
    stand in no list, and the reader of a token's rows takes the unit's input for them; one more expert of the same form that every token takes, with
    weight one or a logistic weight of its own, whose result is one more row a token for the reader to add."""

    replayable = True
    takes_padding_rows = True  # (they are routed and computed like token 0; nobody reads them)

    def __init__(self, spec, store, dtype: torch.dtype):
        self.dtype = dtype
        self.width, self.inner, self.n_experts, self.top = spec.width, spec.inner, spec.n_experts, spec.top
        self.gated, self.activation = bool(getattr(spec, "gated", True)), spec.activation
        if (self.gated and self.activation not in ("silu", "clamped_glu")) or (not self.gated and self.activation != "relu2"):
            raise ValueError(f"routed feed-forward: activation '{spec.activation}' of {'gated' if self.gated else 'ungated'} experts is not known")
        self.scores = getattr(spec, "scores", "softmax")
        if self.scores not in ("softmax", "logistic", "softmax_all"):
            raise ValueError(f"routed feed-forward: scores '{spec.scores}'")
        corrected = self.scores != "softmax"
        self.groups = tuple(int(v) for v in spec.groups) if getattr(spec, "groups", None) is not None else None
        self.shared_inner = int(getattr(spec, "shared_inner", 0) or 0)
        self.identity, self.scale = int(getattr(spec, "identity", 0) or 0), float(getattr(spec, "scale", 1.0))
        self.weighed = bool(self.shared_inner and getattr(spec, "shared_weighed", False))
        self.clamp = self.shared_clamp = None
        if self.activation == "clamped_glu":
            self.clamp = tuple(float(v) for v in spec.clamp)
            self.shared_clamp = tuple(float(v) for v in (getattr(spec, "shared_clamp", None) or spec.clamp))
            if not (self.clamp[0] > 0 and self.shared_clamp[0] > 0):
                raise ValueError("routed feed-forward: limits must be positive")
        if not corrected and (self.identity or self.weighed or self.scale != 1.0):
            raise Unsupported("routed feed-forward: identity experts, a weighed shared expert and a scale go with corrected scores")
        if self.scale != 1.0 and self.scores != "softmax_all":
            raise Unsupported("routed feed-forward: a scale on the weights goes with softmax scores over all experts")
        if self.weighed and not self.clamp:
            raise Unsupported("routed feed-forward: a weighed shared expert is a clamped gated unit")
        outputs = self.n_experts + self.identity
        if not 1 <= self.top <= min(outputs, ops.MOE_MAX_TOP):
            raise ValueError(f"routed feed-forward: {self.top} of {outputs} experts a token (at most {ops.MOE_MAX_TOP})")
        t, E, F, d, S = spec.tensors, self.n_experts, self.inner, self.width, self.shared_inner
        self.router = store.fetch(t["router"], (outputs, d), "matrix")
        self.router_bias = store.fetch(t["router_bias"], (outputs,), "vector") if "router_bias" in t else None
        self.correction = store.fetch(t["correction"], (outputs,), "vector") if corrected and "correction" in t else None
        # A weighed shared expert of the experts' own form and size stands in their stacks behind the last one: in steps of few rows a token
        # then simply has one entry more, and the shared expert costs no launch of its own.
        self.shared_listed = bool(self.weighed and S == F and self.shared_clamp == self.clamp)
        names = list(range(E)) + (["shared"] if self.shared_listed else [])
        src = lambda what, e: t["shared_" + what] if e == "shared" else t[(what, e)]  # noqa: E731
        self.gate = store.fetch_joined([src("gate", e) for e in names], [(F, d)] * len(names), "matrix", "stack") if self.gated else None
        self.up = store.fetch_joined([src("up", e) for e in names], [(F, d)] * len(names), "matrix", "stack")
        self.down = store.fetch_joined([src("down", e) for e in names], [(d, F)] * len(names), "matrix", "stack")
        self.shared_in = self.shared_down = self.joint_in = None
        self.shared_col = outputs  # the shared expert's columns in the joint product
        if S:
            if self.gated and not self.clamp:
                raise Unsupported("routed feed-forward: a shared expert beside gated experts is a clamped unit")
            parts = ([t["shared_gate"]] if self.gated else []) + [t["shared_up"]]
            self.shared_in = store.fetch_joined(parts, [(S, d)] * len(parts), "matrix", "rows")
            self.shared_down = store.fetch(t["shared_down"], (d, S), "matrix")
            if self.weighed:
                # the shared expert's own logit is one more row of the router
                rw, sw = self.router, store.fetch(t["shared_weight"], (1, d), "matrix")
                self.router = store.derived(("joined_rows", t["router"].name, t["shared_weight"].name), lambda: torch.cat([rw, sw], dim=0).contiguous())
                self.shared_col = -(-(outputs + 1) // 8) * 8
            # the router and the shared expert's first product read the same rows: one product [router | shared], the shared expert's columns
            # on a multiple of eight where something stands between
            if self.router_bias is None and self.router.dtype == self.shared_in.dtype:
                rw, sw, col = self.router, self.shared_in, self.shared_col
                self.joint_in = store.derived(("joined_rows", t["router"].name, t["shared_up"].name),
                                              lambda: torch.cat([rw, torch.zeros((col - rw.shape[0], rw.shape[1]), dtype=rw.dtype, device=rw.device), sw], dim=0).contiguous())

    def take_router(self):
        """(weight [experts, width], bias or None): the router's product handed to a caller that runs it as rows
        of a wider product over the same input and passes the logits to `forward(..., router_logits=)`; this
        part then no longer holds the matrix."""
        w, b = self.router, self.router_bias
        self.router = self.router_bias = self.joint_in = None
        return w, b

    rows_a_token = property(lambda self: self.top + (1 if self.shared_inner else 0))  # rows `forward(..., out=)` leaves for each token

    def forward(self, h, ctx: StepContext, residual: Optional[torch.Tensor], out: Optional[torch.Tensor] = None,
                router_logits: Optional[torch.Tensor] = None):
        """Adds the result into `residual`, or, with `out` (float32 [n * rows_a_token, width]), leaves each token's
        `top` weighted expert outputs (and the shared expert's behind them) there in consecutive rows, for a reader that adds them up; returned
        is then None, or with identity experts the `ops.IdentityEntries` that the reader needs.
        `router_logits` (float32 [n, experts], rows may be strided): the router's logits where the caller
        has computed them already, beside a product of its own over the same rows (`take_router`)."""
        h = as_tensor(h)
        n, ws, E, top = h.shape[0], ctx.workspace, self.n_experts, self.top
        columns = E + self.identity + (1 if self.weighed else 0)
        block = ops.moe_block(n * top, E, self.dtype, self.width, self.inner)
        listed = self.shared_listed and block == ops.SKINNY_ROWS  # the shared expert as one more entry of every token
        logits, shared_pre = router_logits, None
        if logits is None and self.joint_in is not None and not listed:
            z = ws.get("router_shared", (n, self.joint_in.shape[0]), torch.float32)
            linear(h, self.joint_in, None, out=z)
            logits, shared_pre = z[:, :columns], z[:, self.shared_col:]
        if logits is None:
            logits = ws.get("router_logits", (n, columns), torch.float32)
            linear(h, self.router, self.router_bias, out=logits)
        rows = self.rows_a_token
        entries = rows if listed else top  # of a token, as the router lists them
        groups = self.up.shape[0]
        tiles = ops.moe_tiles(n * entries, groups, block)
        ids = ws.get("routed_ids", (n * entries,), torch.int32)
        weights = ws.get("routed_weights", (n * entries,), torch.float32)
        rows_list = ws.get("routed_rows", (tiles * block,), torch.int32)
        tile_group = ws.get("routed_tiles", (tiles,), torch.int32)
        ops.moe_route(logits if listed or not self.weighed else logits[:, :columns - 1], top, ids, weights, rows_list, tile_group, block=block, groups=self.groups,
                      scores=self.scores, correction=self.correction, scale=self.scale, identity=self.identity, extra=listed, n_lists=groups)
        inner = ws.get("routed_inner", (n * entries, self.inner), self.dtype)
        if self.gated:
            ops.moe_product(inner, h, self.gate, self.up, rows_list, tile_group, a_div=entries, block=block, clamp=self.clamp)
        else:
            ops.moe_product(inner, h, self.up, None, rows_list, tile_group, a_div=entries, block=block, act=self.activation)
        y = out if out is not None else ws.get("routed_out", (n * rows, self.width), torch.float32)
        # (the second product's rows are the entries: a_div = 1 for its operand, `entries` for where a token's rows lie in y)
        ops.moe_product(y, inner, self.down, None, rows_list, tile_group, row_scale=weights, block=block, out_div=entries, out_extra=rows - entries)
        if self.shared_inner and not listed:
            S = self.shared_inner
            if shared_pre is None:
                shared_pre = ws.get("shared_in", (n, self.shared_in.shape[0]), torch.float32)
                linear(h, self.shared_in, None, out=shared_pre)
            act = ws.get("shared_inner", (n, S), self.dtype)
            if self.gated:
                ops.glu_clamped(act, shared_pre, *self.shared_clamp, row_gate=logits[:, columns - 1:] if self.weighed else None)
            else:
                ops.activate(act, shared_pre, self.activation)
            # the shared expert's row of each token, behind its `top` rows
            linear(act, self.shared_down, None, out=y.view(n, rows * self.width)[:, top * self.width:])
        identity = ops.IdentityEntries(ids, weights, entries, h) if self.identity else None
        if out is None:
            if identity is None:
                ops.gated_norm_add(settled(residual), y, None, 0.0, n_sum=rows, normalize=False)
            else:
                ops.streams_update(settled(residual).view(n, 1, self.width), y=y, n_sum=rows, identity=identity)
        return identity if out is not None else None


register_ffn("routed_ffn", RoutedFFN)
