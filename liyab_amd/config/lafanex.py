"""Lafanex's typed configuration, read from its own config.json keys.

A decoder of sequential pre-norm layers over several residual streams: a sublayer reads the norm of a learned combination of the streams,
and a learned matrix mixes them when its result is added. No position table: positions enter inside attention. A stretch of layers may run
several times in a row with the same weights, each pass with a cache and state of its own. config.json:

    architecture     "Lafanex"
    vocab, width
    norm.eps         the epsilon of every norm
    streams          the residual streams (optional: without it one plain stream, and no hc tensors)
    loop             optional: {start, stop, times}: layers start .. stop - 1 run that often in a row
    max_positions    optional: the longest context (nothing in the design bounds it; default 32,768)
    layers[i]        type, mixer {...}, mlp (null, {kind "dense", ff} or {kind "moe", expert {ff, limit}, router {experts, top, identity (optional), scale
                     (optional)}, shared {ff, limit} (optional)})
      type "attention": mixer {heads, kv_heads, dim, vdim, scale, rot {dims, base} (optional)}: queries and keys turned, then brought to unit root mean
                     square a head; one added to the softmax's denominator
      type "mamba1":    mixer {inner, state, dt_rank, conv}: a selective scan behind a short convolution (sizes that are left out are read from
                     the tensors' shapes)

Tensors: embed (also the head's matrix), final.norm; layer i's start with "l<i>.": norm1, norm2, hc1.{in, out, mix}, hc2.{in, out, mix}, and
  attention: mix.{q, k, v, o}
  mamba1:    mix.{in, conv, conv.b, x, dt, dt.b, A_log, D, o}
  dense:     mlp.{gate, up, down};  moe: mlp.router, mlp.correction, mlp.e<k>.{gate, up, down}, mlp.shared.{gate, up, down, sg}
Matrices are stored [out, in]; convolutions [channels, taps], the last column the current token's; hc.mix [from, to]; norms around zero.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, List, Optional, Tuple

from ..errors import InvalidModel, Unsupported
from .plan import (
    GatedFFNSpec,
    HeadSpec,
    Init,
    LayerSpec,
    ModelPlan,
    NormSpec,
    OrderEntry,
    RotarySpec,
    RoutedFFNSpec,
    ScoredAttentionSpec,
    SelectiveScanSpec,
    StreamConnectionSpec,
    TensorSource,
    TokenEmbeddingSpec,
)
from .registry import register_architecture

_LIMIT = 1 << 24
DEFAULT_MAX_POSITIONS = 1 << 15
# what the design fixes
SINK = 0.0  # the logit of what is added to the softmax's denominator
GLU_SLOPE, GLU_SHIFT = 1.702, 1.0  # g * sigmoid(1.702 g) * (u + 1)
NORM_OFFSET = 1.0  # norms multiply by 1 + the stored weight


def _int(raw, key: str, what: str, least: int = 1) -> int:
    v = raw.get(key) if isinstance(raw, dict) else None
    if isinstance(v, bool) or not isinstance(v, int) or v < least or v > _LIMIT:
        raise InvalidModel(f"missing or invalid {what}")
    return v


def _number(raw, key: str, what: str, positive: bool = True) -> float:
    v = raw.get(key) if isinstance(raw, dict) else None
    if isinstance(v, bool) or not isinstance(v, (int, float)) or not math.isfinite(v) or (positive and v <= 0):
        raise InvalidModel(f"missing or invalid {what}")
    return float(v)


@dataclass(frozen=True)
class LafanexAttention:
    n_head: int
    n_kv_head: int
    head_dim: int
    value_dim: int
    scale: float
    rot_dims: int  # 0: no rotary encoding
    rot_base: float


@dataclass(frozen=True)
class LafanexScan:
    inner: int
    n_state: int
    dt_rank: int
    taps: int


@dataclass(frozen=True)
class LafanexMLP:
    kind: str  # "dense" | "moe"
    ff: int  # dense: the inner width; moe: an expert's
    limit: float = 0.0  # moe
    experts: int = 0
    top: int = 0
    identity: int = 0
    scale: float = 1.0
    shared_ff: int = 0  # 0: no shared expert
    shared_limit: float = 0.0


@dataclass(frozen=True)
class LafanexLayer:
    kind: str  # "attention" | "mamba1"
    mixer: Any  # LafanexAttention | LafanexScan
    mlp: Optional[LafanexMLP]


@dataclass(frozen=True)
class LafanexLoop:
    start: int
    stop: int
    times: int


def _attention(m, where: str) -> LafanexAttention:
    H, G = _int(m, "heads", where + ".heads"), _int(m, "kv_heads", where + ".kv_heads")
    if H % G:
        raise InvalidModel(f"invalid {where}: {H} heads are no multiple of {G} kv_heads")
    D, dims, base = _int(m, "dim", where + ".dim"), 0, 0.0
    rot = m.get("rot")
    if rot is not None:
        dims, base = _int(rot, "dims", where + ".rot.dims", 0), _number(rot, "base", where + ".rot.base")
        if dims % 2 or dims > D:
            raise InvalidModel(f"invalid {where}.rot: {dims} turned entries of heads of {D}")
    return LafanexAttention(n_head=H, n_kv_head=G, head_dim=D, value_dim=_int(m, "vdim", where + ".vdim"), scale=_number(m, "scale", where + ".scale"),
                            rot_dims=dims, rot_base=base)


def _scan(m, where: str, prefix: str, shapes: dict) -> LafanexScan:
    def size(key: str, tensor: str, axis: int) -> int:
        shape = shapes.get(prefix + tensor)
        if m.get(key) is None and shape is not None and len(shape) == 2:
            return int(shape[axis])
        return _int(m, key, f"{where}.{key}")

    return LafanexScan(inner=size("inner", "A_log", 0), n_state=size("state", "A_log", 1), dt_rank=size("dt_rank", "dt", 1), taps=size("conv", "conv", 1))


def _mlp(raw, where: str) -> Optional[LafanexMLP]:
    if raw is None:
        return None
    kind = raw.get("kind") if isinstance(raw, dict) else None
    if kind == "dense":
        return LafanexMLP(kind="dense", ff=_int(raw, "ff", where + ".ff"))
    if kind == "moe":
        r, e, s = raw.get("router"), raw.get("expert"), raw.get("shared")
        E, top = _int(r, "experts", where + ".router.experts"), _int(r, "top", where + ".router.top")
        identity = _int(r, "identity", where + ".router.identity", 0) if r.get("identity") is not None else 0
        if top > E + identity:
            raise InvalidModel(f"invalid {where}.router: {top} of {E + identity} outputs")
        return LafanexMLP(kind="moe", ff=_int(e, "ff", where + ".expert.ff"), limit=_number(e, "limit", where + ".expert.limit"), experts=E, top=top, identity=identity,
                          scale=_number(r, "scale", where + ".router.scale") if r.get("scale") is not None else 1.0,
                          shared_ff=_int(s, "ff", where + ".shared.ff") if s is not None else 0,
                          shared_limit=_number(s, "limit", where + ".shared.limit") if s is not None else 0.0)
    raise Unsupported(f"{where}.kind '{kind}' is not supported (supported: dense, moe)")


@dataclass(frozen=True)
class LafanexConfig:
    vocab: int
    width: int
    eps: float
    streams: int  # 0: one plain stream
    loop: Optional[LafanexLoop]
    max_positions: int
    layers: Tuple[LafanexLayer, ...]

    architecture = "Lafanex"

    @classmethod
    def from_json(cls, raw: dict, shapes: Optional[dict] = None) -> "LafanexConfig":
        """`shapes`: tensor name -> shape, for sizes of a scan that the file leaves to its tensors."""
        vocab, width = _int(raw, "vocab", "vocab"), _int(raw, "width", "width")
        eps = _number(raw.get("norm"), "eps", "norm.eps")
        streams = _int(raw, "streams", "streams") if raw.get("streams") is not None else 0
        max_positions = _int(raw, "max_positions", "max_positions") if raw.get("max_positions") is not None else DEFAULT_MAX_POSITIONS
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise InvalidModel("missing or invalid layers")
        layers = []
        for i, entry in enumerate(listed):
            if not isinstance(entry, dict):
                raise InvalidModel(f"invalid layers[{i}]")
            kind, m, where = entry.get("type"), entry.get("mixer"), f"layers[{i}].mixer"
            if kind not in ("attention", "mamba1"):
                raise Unsupported(f"layers[{i}].type '{kind}' is not supported (supported: attention, mamba1)")
            if not isinstance(m, dict):
                raise InvalidModel(f"missing or invalid {where}")
            mixer = _attention(m, where) if kind == "attention" else _scan(m, where, f"l{i}.mix.", shapes or {})
            layers.append(LafanexLayer(kind=kind, mixer=mixer, mlp=_mlp(entry.get("mlp"), f"layers[{i}].mlp")))
        loop = None
        if raw.get("loop") is not None:
            lp = raw["loop"]
            loop = LafanexLoop(start=_int(lp, "start", "loop.start", 0), stop=_int(lp, "stop", "loop.stop", 0), times=_int(lp, "times", "loop.times"))
            if not loop.start <= loop.stop <= len(layers):
                raise InvalidModel(f"invalid loop: layers {loop.start} to {loop.stop} of {len(layers)}")
        return cls(vocab=vocab, width=width, eps=eps, streams=streams, loop=loop, max_positions=max_positions, layers=tuple(layers))

    def to_json(self) -> dict:
        layers = []
        for layer in self.layers:
            m, f, mlp = layer.mixer, layer.mlp, None
            if layer.kind == "attention":
                mixer = {"heads": m.n_head, "kv_heads": m.n_kv_head, "dim": m.head_dim, "vdim": m.value_dim, "scale": m.scale}
                if m.rot_dims:
                    mixer["rot"] = {"dims": m.rot_dims, "base": m.rot_base}
            else:
                mixer = {"inner": m.inner, "state": m.n_state, "dt_rank": m.dt_rank, "conv": m.taps}
            if f is not None and f.kind == "dense":
                mlp = {"kind": "dense", "ff": f.ff}
            elif f is not None:
                mlp = {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit},
                       "router": {"experts": f.experts, "top": f.top, "identity": f.identity, "scale": f.scale}}
                if f.shared_ff:
                    mlp["shared"] = {"ff": f.shared_ff, "limit": f.shared_limit}
            layers.append({"type": layer.kind, "mixer": mixer, "mlp": mlp})
        out = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
               "max_positions": self.max_positions, "layers": layers}
        if self.streams:
            out["streams"] = self.streams
        if self.loop is not None:
            out["loop"] = {"start": self.loop.start, "stop": self.loop.stop, "times": self.loop.times}
        return out

    def runs(self) -> List[int]:
        """The layers in the order they run."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return list(range(n))
        return list(range(loop.start)) + loop.times * list(range(loop.start, loop.stop)) + list(range(loop.stop, n))

    def plan(self) -> ModelPlan:
        d, V, S = self.width, self.vocab, self.streams
        wide = Init(1.0 / math.sqrt(d))

        def norm(name: str) -> NormSpec:
            return NormSpec(kind="rmsnorm", width=d, eps=self.eps, weight_offset=NORM_OFFSET, tensors={"weight": TensorSource(name, init=Init(0.1))})

        def connection(name: str):
            return StreamConnectionSpec(kind="stream_connection", streams=S, tensors={
                "take": TensorSource(name + ".in", init=Init(0.3 / S, 1.0 / S)), "give": TensorSource(name + ".out", init=Init(0.2, 1.0)),
                "mix": TensorSource(name + ".mix", init=Init(0.3 / S, 1.0 / S))}) if S else None

        # A layer that runs several times is listed once a run, with the same tensor names (the weights' store hands every
        # run the same device tensors) and a cache and state of its own.
        layers = []
        for i in self.runs():
            layer, p = self.layers[i], f"l{i}"
            mixer = (self._attention_spec if layer.kind == "attention" else self._scan_spec)(p + ".mix", layer.mixer, wide)
            ffn = self._ffn_spec(p + ".mlp", layer.mlp, wide) if layer.mlp is not None else None
            layers.append(LayerSpec(mixer=mixer, ffn=ffn, norm_mixer=norm(p + ".norm1"), norm_ffn=norm(p + ".norm2") if ffn is not None else None,
                                    arrangement="streams", connect_mixer=connection(p + ".hc1"), connect_ffn=connection(p + ".hc2") if ffn is not None else None))
        ignorable = []
        for i, layer in enumerate(self.layers):  # a layer without a feed-forward may still hold the norm and the connection nobody reads
            if layer.mlp is None:
                ignorable += [f"l{i}.norm2", f"l{i}.hc2.*"]
        return ModelPlan(
            architecture=self.architecture, width=d, vocab_size=V, max_positions=self.max_positions,
            embedding=TokenEmbeddingSpec(kind="token_embedding", vocab_size=V, width=d, scale=1.0, tensors={"table": TensorSource("embed", init=Init(1.0))}),
            residual_position=None,
            layers=layers,
            order=[OrderEntry(layer=i) for i in range(len(layers))],
            final_norm=norm("final.norm"),
            head=HeadSpec(kind="lm_head", width=d, vocab_size=V, logit_scale=1.0, tensors={"weight": TensorSource("embed", init=Init(1.0))}),
            ignorable=tuple(ignorable), name_prefixes=("",), eos_token_id=None, streams=S or 1,
        )

    def _attention_spec(self, p: str, m: LafanexAttention, wide: Init) -> ScoredAttentionSpec:
        tensors = {c: TensorSource(f"{p}.{c}", init=wide) for c in "qkv"}
        tensors["out"] = TensorSource(p + ".o", init=Init(1.0 / math.sqrt(m.n_head * m.value_dim)))
        return ScoredAttentionSpec(kind="scored_attention", width=self.width, n_head=m.n_head, n_kv_head=m.n_kv_head, head_dim=m.head_dim,
                                   value_dim=m.value_dim, scale=m.scale, eps=self.eps, qk_norm=True, qk_norm_weights=False, sink_value=SINK,
                                   rotary=RotarySpec(dims=m.rot_dims, base=m.rot_base) if m.rot_dims else None, tensors=tensors)

    def _scan_spec(self, p: str, m: LafanexScan, wide: Init) -> SelectiveScanSpec:
        inner = Init(1.0 / math.sqrt(m.inner))
        return SelectiveScanSpec(kind="selective_scan", width=self.width, inner=m.inner, n_state=m.n_state, dt_rank=m.dt_rank, taps=m.taps, tensors={
            "in": TensorSource(p + ".in", init=wide), "conv": TensorSource(p + ".conv", init=Init(0.5)), "conv_bias": TensorSource(p + ".conv.b", init=Init(0.1)),
            "x": TensorSource(p + ".x", init=inner), "dt": TensorSource(p + ".dt", init=Init(1.0 / math.sqrt(m.dt_rank))),
            "dt_bias": TensorSource(p + ".dt.b", init=Init(1.0, -2.0)), "A_log": TensorSource(p + ".A_log", init=Init(0.7, 0.3)),
            "D": TensorSource(p + ".D", init=Init(0.3, 1.0)), "out": TensorSource(p + ".o", init=inner)})

    def _ffn_spec(self, p: str, f: LafanexMLP, wide: Init):
        down = Init(1.0 / math.sqrt(f.ff))
        if f.kind == "dense":
            return GatedFFNSpec(kind="gated_ffn", width=self.width, inner=f.ff, activation="gelu_tanh", tensors={
                "gate": TensorSource(p + ".gate", init=wide), "up": TensorSource(p + ".up", init=wide), "down": TensorSource(p + ".down", init=down)})
        tensors = {"router": TensorSource(p + ".router", init=Init(2.0 / math.sqrt(self.width))), "correction": TensorSource(p + ".correction", init=Init(0.1))}
        for e in range(f.experts):
            tensors[("gate", e)] = TensorSource(f"{p}.e{e}.gate", init=wide)
            tensors[("up", e)] = TensorSource(f"{p}.e{e}.up", init=wide)
            tensors[("down", e)] = TensorSource(f"{p}.e{e}.down", init=down)
        if f.shared_ff:
            tensors.update({"shared_gate": TensorSource(p + ".shared.gate", init=wide), "shared_up": TensorSource(p + ".shared.up", init=wide),
                            "shared_down": TensorSource(p + ".shared.down", init=Init(1.0 / math.sqrt(f.shared_ff))),
                            "shared_weight": TensorSource(p + ".shared.sg", init=wide)})
        return RoutedFFNSpec(kind="routed_ffn", width=self.width, inner=f.ff, n_experts=f.experts, top=f.top, activation="clamped_glu", scores="softmax_all",
                             identity=f.identity, scale=f.scale, clamp=(f.limit, GLU_SLOPE, GLU_SHIFT), shared_inner=f.shared_ff,
                             shared_clamp=(f.shared_limit, GLU_SLOPE, GLU_SHIFT) if f.shared_ff else None, shared_weighed=bool(f.shared_ff), tensors=tensors)


register_architecture("Lafanex", LafanexConfig)
