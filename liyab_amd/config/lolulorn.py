"""Lolulorn's typed configuration, read from its own config.json keys.

A decoder whose sublayers read the residual stream itself, with a layer norm on each sublayer's result: x <- x + n1(mixer(x)), then
x <- x + n2(ff(x)). No position table: positions enter inside attention. A layer's mixer is one of three kinds, its feed-forward one of
two or none. config.json:

    architecture     "Lolulorn"
    vocab, width
    embedding.scale  the factor on the embedding's rows (optional, default 1)
    norm.eps         the epsilon of every norm
    max_positions    optional: the longest context (nothing in the design bounds it; default 32,768)
    layers[i]        type, mixer {...}, mlp (null, {kind "dense", ff} or {kind "moe", expert {ff}, router {experts, top, groups {count, keep} (optional)}})
      type "attention": mixer {heads, kv_heads, dim, vdim, scale, mask {size, keep_first} (optional), rot {dims, base, scaling {factor} (optional)}
                     (optional), kv_from (optional)}: norms over the whole queries and keys, a sliding window behind which the first
                     keep_first positions stay visible; with kv_from the keys and values of that layer
      type "delta":  mixer {heads, kv_heads, dim, vdim, conv}: a gated delta rule behind a short convolution
      type "gla":    mixer {heads, dim, vdim, tau}: gated linear attention; the decay's rank is the shape of mix.a1 (where no weights say
                     it, the optional key decay_rank, default 16)

Tensors: embed, final.norm, final.norm.b, head; layer i's start with "l<i>.": norm1, norm1.b, norm2, norm2.b, and
  attention: mix.{q, q.norm, o} and, without kv_from, mix.{k, k.norm, v}
  delta:     mix.{q, q.conv, k, k.conv, v, v.conv, b, a, A_log, dt_bias, g, norm, o}
  gla:       mix.{q, k, v, g, a1, a2, a2.b, norm, o}
  dense:     mlp.{gate, up, down};  moe: mlp.router, mlp.correction, mlp.e<k>.{gate, up, down}
Matrices are stored [out, in]; convolutions [channels, taps], the last column the current token's.
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Optional, Tuple

from ..errors import InvalidModel, Unsupported
from .plan import (
    GatedDeltaSpec,
    GatedFFNSpec,
    GatedLinearAttentionSpec,
    HeadSpec,
    Init,
    LayerSpec,
    ModelPlan,
    NormSpec,
    OrderEntry,
    RotarySpec,
    RoutedFFNSpec,
    ScoredAttentionSpec,
    TensorSource,
    TokenEmbeddingSpec,
)
from .registry import register_architecture

_LIMIT = 1 << 24
DEFAULT_MAX_POSITIONS = 1 << 15
DEFAULT_DECAY_RANK = 16
# what the design fixes
KEY_EPS = 1e-6  # under the root that brings the delta rule's queries and keys to length one


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
class LolulornAttention:
    n_head: int
    n_kv_head: int
    head_dim: int
    value_dim: int
    scale: float
    window: int  # 0: every earlier position
    keep_first: int
    rot_dims: int  # 0: no rotary encoding
    rot_base: float
    rot_factor: float
    kv_from: Optional[int] = None


@dataclass(frozen=True)
class LolulornDelta:
    n_head: int
    n_kv_head: int
    head_dim: int
    value_dim: int
    taps: int


@dataclass(frozen=True)
class LolulornGLA:
    n_head: int
    head_dim: int
    value_dim: int
    tau: float
    decay_rank: int


@dataclass(frozen=True)
class LolulornMLP:
    kind: str  # "dense" | "moe"
    ff: int  # dense: the inner width; moe: an expert's
    experts: int = 0
    top: int = 0
    groups: int = 1
    keep: int = 1


@dataclass(frozen=True)
class LolulornLayer:
    kind: str  # "attention" | "delta" | "gla"
    mixer: Any  # LolulornAttention | LolulornDelta | LolulornGLA
    mlp: Optional[LolulornMLP]


def _heads(m, where: str) -> Tuple[int, int, int, int]:
    H, G = _int(m, "heads", where + ".heads"), _int(m, "kv_heads", where + ".kv_heads")
    if H % G:
        raise InvalidModel(f"invalid {where}: {H} heads are no multiple of {G} kv_heads")
    return H, G, _int(m, "dim", where + ".dim"), _int(m, "vdim", where + ".vdim")


def _attention(m, where: str) -> LolulornAttention:
    H, G, D, V = _heads(m, where)
    window, keep = 0, 0
    if m.get("mask") is not None:
        window = _int(m["mask"], "size", where + ".mask.size")
        keep = _int(m["mask"], "keep_first", where + ".mask.keep_first", least=0) if isinstance(m["mask"], dict) and m["mask"].get("keep_first") is not None else 0
    dims, base, factor = 0, 0.0, 1.0
    rot = m.get("rot")
    if rot is not None:
        dims, base = _int(rot, "dims", where + ".rot.dims"), _number(rot, "base", where + ".rot.base")
        if dims % 2 or dims > D:
            raise InvalidModel(f"invalid {where}.rot: {dims} turned entries of heads of {D}")
        if rot.get("scaling") is not None:
            factor = _number(rot["scaling"], "factor", where + ".rot.scaling.factor")
    kv_from = m.get("kv_from")
    if kv_from is not None and (isinstance(kv_from, bool) or not isinstance(kv_from, int) or kv_from < 0):
        raise InvalidModel(f"invalid {where}.kv_from")
    return LolulornAttention(n_head=H, n_kv_head=G, head_dim=D, value_dim=V, scale=_number(m, "scale", where + ".scale"), window=window, keep_first=keep,
                             rot_dims=dims, rot_base=base, rot_factor=factor, kv_from=kv_from)


def _mlp(raw, where: str) -> Optional[LolulornMLP]:
    if raw is None:
        return None
    kind = raw.get("kind") if isinstance(raw, dict) else None
    if kind == "dense":
        return LolulornMLP(kind="dense", ff=_int(raw, "ff", where + ".ff"))
    if kind == "moe":
        r = raw.get("router")
        E, top = _int(r, "experts", where + ".router.experts"), _int(r, "top", where + ".router.top")
        g = r.get("groups") if isinstance(r, dict) else None
        count, keep = (_int(g, "count", where + ".router.groups.count"), _int(g, "keep", where + ".router.groups.keep")) if g is not None else (1, 1)
        if E % count or keep > count or top > keep * (E // count):
            raise InvalidModel(f"invalid {where}.router: {top} of {E} experts in {keep} of {count} groups")
        return LolulornMLP(kind="moe", ff=_int(raw.get("expert"), "ff", where + ".expert.ff"), experts=E, top=top, groups=count, keep=keep)
    raise Unsupported(f"{where}.kind '{kind}' is not supported (supported: dense, moe)")


@dataclass(frozen=True)
class LolulornConfig:
    vocab: int
    width: int
    embedding_scale: float
    eps: float
    max_positions: int
    layers: Tuple[LolulornLayer, ...]

    architecture = "Lolulorn"

    @classmethod
    def from_json(cls, raw: dict, shapes: Optional[dict] = None) -> "LolulornConfig":
        """`shapes`: tensor name -> shape, for the one size that only a tensor's shape gives (the rank of a decay)."""
        vocab, width = _int(raw, "vocab", "vocab"), _int(raw, "width", "width")
        eps = _number(raw.get("norm"), "eps", "norm.eps")
        scale = _number(raw.get("embedding"), "scale", "embedding.scale", positive=False) if raw.get("embedding") is not None else 1.0
        max_positions = _int(raw, "max_positions", "max_positions") if raw.get("max_positions") is not None else DEFAULT_MAX_POSITIONS
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            raise InvalidModel("missing or invalid layers")
        layers = []
        for i, entry in enumerate(listed):
            if not isinstance(entry, dict):
                raise InvalidModel(f"invalid layers[{i}]")
            kind, m, where = entry.get("type"), entry.get("mixer"), f"layers[{i}].mixer"
            if not isinstance(m, dict):
                raise InvalidModel(f"missing or invalid {where}")
            if kind == "attention":
                mixer = _attention(m, where)
                j = mixer.kv_from
                if j is not None:
                    if j >= i or layers[j].kind != "attention" or layers[j].mixer.kv_from is not None:
                        raise InvalidModel(f"invalid {where}.kv_from: layer {j} is no earlier attention layer with keys and values of its own")
                    of = layers[j].mixer
                    if (of.n_kv_head, of.head_dim, of.value_dim) != (mixer.n_kv_head, mixer.head_dim, mixer.value_dim):
                        raise InvalidModel(f"invalid {where}: its keys and values are layer {j}'s, which have another shape")
            elif kind == "delta":
                H, G, D, V = _heads(m, where)
                mixer = LolulornDelta(n_head=H, n_kv_head=G, head_dim=D, value_dim=V, taps=_int(m, "conv", where + ".conv"))
            elif kind == "gla":
                rank = _int(m, "decay_rank", where + ".decay_rank") if m.get("decay_rank") is not None else DEFAULT_DECAY_RANK
                narrow = (shapes or {}).get(f"l{i}.mix.a1")
                if narrow is not None and len(narrow) == 2:
                    rank = int(narrow[0])
                mixer = LolulornGLA(n_head=_int(m, "heads", where + ".heads"), head_dim=_int(m, "dim", where + ".dim"), value_dim=_int(m, "vdim", where + ".vdim"),
                                    tau=_number(m, "tau", where + ".tau"), decay_rank=rank)
            else:
                raise Unsupported(f"layers[{i}].type '{kind}' is not supported (supported: attention, delta, gla)")
            layers.append(LolulornLayer(kind=kind, mixer=mixer, mlp=_mlp(entry.get("mlp"), f"layers[{i}].mlp")))
        return cls(vocab=vocab, width=width, embedding_scale=scale, eps=eps, max_positions=max_positions, layers=tuple(layers))

    def to_json(self) -> dict:
        layers = []
        for layer in self.layers:
            m = layer.mixer
            if layer.kind == "attention":
                mixer = {"heads": m.n_head, "kv_heads": m.n_kv_head, "dim": m.head_dim, "vdim": m.value_dim, "scale": m.scale}
                if m.window:
                    mixer["mask"] = {"size": m.window, "keep_first": m.keep_first}
                if m.rot_dims:
                    mixer["rot"] = {"dims": m.rot_dims, "base": m.rot_base, "scaling": {"factor": m.rot_factor}}
                if m.kv_from is not None:
                    mixer["kv_from"] = m.kv_from
            elif layer.kind == "delta":
                mixer = {"heads": m.n_head, "kv_heads": m.n_kv_head, "dim": m.head_dim, "vdim": m.value_dim, "conv": m.taps}
            else:
                mixer = {"heads": m.n_head, "dim": m.head_dim, "vdim": m.value_dim, "tau": m.tau, "decay_rank": m.decay_rank}
            f, mlp = layer.mlp, None
            if f is not None and f.kind == "dense":
                mlp = {"kind": "dense", "ff": f.ff}
            elif f is not None:
                mlp = {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top, "groups": {"count": f.groups, "keep": f.keep}}}
            layers.append({"type": layer.kind, "mixer": mixer, "mlp": mlp})
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "embedding": {"scale": self.embedding_scale},
                "norm": {"eps": self.eps}, "max_positions": self.max_positions, "layers": layers}

    def plan(self) -> ModelPlan:
        d, V = self.width, self.vocab
        wide = Init(1.0 / math.sqrt(d))

        def norm(name: str) -> NormSpec:
            return NormSpec(kind="layernorm", width=d, eps=self.eps,
                            tensors={"weight": TensorSource(name, init=Init(0.1, 1.0)), "bias": TensorSource(name + ".b", init=Init(0.1))})

        layers, order = [], []
        for i, layer in enumerate(self.layers):
            p = f"l{i}"
            make = {"attention": self._attention_spec, "delta": self._delta_spec, "gla": self._gla_spec}[layer.kind]
            ffn = self._ffn_spec(p + ".mlp", layer.mlp, wide) if layer.mlp is not None else None
            layers.append(LayerSpec(mixer=make(p + ".mix", layer.mixer, wide), ffn=ffn, norm_mixer=norm(p + ".norm1"),
                                    norm_ffn=norm(p + ".norm2") if ffn is not None else None, arrangement="post_norm_gated"))
            shared = layer.mixer.kv_from if layer.kind == "attention" else None
            order.append(OrderEntry(layer=i, cache_of=shared, writes_cache=shared is None))
        return ModelPlan(
            architecture=self.architecture, width=d, vocab_size=V, max_positions=self.max_positions,
            embedding=TokenEmbeddingSpec(kind="token_embedding", vocab_size=V, width=d, scale=self.embedding_scale,
                                         tensors={"table": TensorSource("embed", init=Init(1.0))}),
            residual_position=None,
            layers=layers,
            order=order,
            final_norm=norm("final.norm"),
            head=HeadSpec(kind="lm_head", width=d, vocab_size=V, logit_scale=1.0, tensors={"weight": TensorSource("head", init=wide)}),
            # (a layer without a feed-forward may still carry its norm)
            ignorable=("l*.norm2", "l*.norm2.b"), name_prefixes=("",), eos_token_id=None,
        )

    def _attention_spec(self, p: str, m: LolulornAttention, wide: Init) -> ScoredAttentionSpec:
        tensors = {"q": TensorSource(p + ".q", init=wide), "q_norm": TensorSource(p + ".q.norm", init=Init(0.1, 1.0)),
                   "out": TensorSource(p + ".o", init=Init(1.0 / math.sqrt(m.n_head * m.value_dim)))}
        if m.kv_from is None:
            tensors.update({"k": TensorSource(p + ".k", init=wide), "v": TensorSource(p + ".v", init=wide),
                            "k_norm": TensorSource(p + ".k.norm", init=Init(0.1, 1.0))})
        return ScoredAttentionSpec(kind="scored_attention", width=self.width, n_head=m.n_head, n_kv_head=m.n_kv_head, head_dim=m.head_dim,
                                   value_dim=m.value_dim, scale=m.scale, eps=self.eps, window=m.window, keep_first=m.keep_first, qk_norm_rows=True,
                                   rotary=RotarySpec(dims=m.rot_dims, base=m.rot_base, linear=m.rot_factor) if m.rot_dims else None,
                                   kv_shared=m.kv_from is not None, tensors=tensors)

    def _delta_spec(self, p: str, m: LolulornDelta, wide: Init) -> GatedDeltaSpec:
        tensors = {c: TensorSource(f"{p}.{c}", init=wide) for c in ("q", "k", "v", "g", "b", "a")}
        tensors.update({c + "_conv": TensorSource(f"{p}.{c}.conv", init=Init(0.5)) for c in ("q", "k", "v")})
        tensors.update({"A_log": TensorSource(p + ".A_log", init=Init(0.5, -1.0)), "dt_bias": TensorSource(p + ".dt_bias", init=Init(0.5, -1.0)),
                        "norm": TensorSource(p + ".norm", init=Init(0.1, 1.0)), "out": TensorSource(p + ".o", init=Init(1.0 / math.sqrt(m.n_head * m.value_dim)))})
        return GatedDeltaSpec(kind="gated_delta", width=self.width, n_head=m.n_head, n_kv_head=m.n_kv_head, head_dim=m.head_dim, value_dim=m.value_dim,
                              taps=m.taps, eps=self.eps, q_scale=m.head_dim ** -0.5, key_eps=KEY_EPS, tensors=tensors)

    def _gla_spec(self, p: str, m: LolulornGLA, wide: Init) -> GatedLinearAttentionSpec:
        tensors = {c: TensorSource(f"{p}.{c}", init=wide) for c in ("q", "k", "v", "g")}
        tensors.update({"w1": TensorSource(p + ".a1", init=wide), "w2": TensorSource(p + ".a2", init=Init(1.0 / math.sqrt(m.decay_rank))),
                        "w2_bias": TensorSource(p + ".a2.b", init=Init(0.5, 1.0)), "norm": TensorSource(p + ".norm", init=Init(0.1, 1.0)),
                        "out": TensorSource(p + ".o", init=Init(1.0 / math.sqrt(m.n_head * m.value_dim)))})
        return GatedLinearAttentionSpec(kind="gated_linear_attention", width=self.width, n_head=m.n_head, head_dim=m.head_dim, value_dim=m.value_dim,
                                        decay_rank=m.decay_rank, tau=m.tau, eps=self.eps, q_scale=m.head_dim ** -0.5, tensors=tensors)

    def _ffn_spec(self, p: str, f: LolulornMLP, wide: Init):
        down = Init(1.0 / math.sqrt(f.ff))
        if f.kind == "dense":
            return GatedFFNSpec(kind="gated_ffn", width=self.width, inner=f.ff, activation="gelu_tanh", tensors={
                "gate": TensorSource(p + ".gate", init=wide), "up": TensorSource(p + ".up", init=wide), "down": TensorSource(p + ".down", init=down)})
        tensors = {"router": TensorSource(p + ".router", init=Init(4.0 / math.sqrt(self.width))), "correction": TensorSource(p + ".correction", init=Init(0.3))}
        for e in range(f.experts):
            tensors[("gate", e)] = TensorSource(f"{p}.e{e}.gate", init=wide)
            tensors[("up", e)] = TensorSource(f"{p}.e{e}.up", init=wide)
            tensors[("down", e)] = TensorSource(f"{p}.e{e}.down", init=down)
        return RoutedFFNSpec(kind="routed_ffn", width=self.width, inner=f.ff, n_experts=f.experts, top=f.top, activation="silu", scores="logistic",
                             groups=(f.groups, f.keep), tensors=tensors)


register_architecture("Lolulorn", LolulornConfig)
