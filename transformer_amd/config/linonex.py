"""Typed configuration of the Linonex decoder, read from its own config.json.

A Linonex model is a list of pre-norm layers ``x <- x + mixer(n1(x))``, then ``x <- x + ff(n2(x))``
where the layer has a feed-forward. Two mixers: "mlstm" (a matrix memory with exponential gates, a running
maximum and a normaliser) and "parallel" (grouped-query softmax attention with capped scores over chunks of
the sequence, behind short convolutions on q, k and v, beside a delta rule on a matrix state with one decay
per head; the mean of the two results, each normed over the width). The feed-forward is a gated unit, or
routed: a softmax over experts and identity experts, a correction that takes part in the choice alone. A
learned row per position is added to the embedding; a span of layers can be walked more than once, each
repeat with cache layers and state of its own and with the embedding's rows added once more in front of it.

Keys: ``architecture``, ``vocab``, ``width``, ``max_positions``, ``norm.eps``, ``loop.{start, stop, times}``,
``layers[i].{type, mixer, mlp}``. ``mixer`` by type: mlstm: heads, dim, vdim, gate_cap; parallel: ``left`` with
heads, kv_heads, dim, vdim, conv, scale, softcap, mask.size and ``right`` with heads, kv_heads, dim, vdim, conv.
``mlp``: null, ``{kind: "dense", ff}`` or ``{kind: "moe", expert.ff, router.{experts, identity, scale, top}}``.
Absent keys mean absent mechanisms: no ``mask``: every earlier token is seen; no ``softcap``: plain scores; no
``conv``: none; no ``loop``: every layer once; no ``identity``: no identity experts; ``kv_heads`` defaults to
``heads``, ``vdim`` to ``dim``, ``router.scale`` to 1.
"""
from __future__ import annotations

import dataclasses
from dataclasses import dataclass, field
from typing import Optional, Tuple

from .spec import (BlockSpec, BranchMeanSpec, ConfigError, GatedDeltaSpec, GLUSpec, LearnedPositionSpec, MatrixMemorySpec,
                   ModelSpec, NormSpec, RoutedMLPSpec, RunSpec, SinkAttentionSpec)
from .vametar import _get

LAYER_TYPES = ("mlstm", "parallel")


def _mapping(d, key, where):
    v = d.get(key) if isinstance(d, dict) else None
    if not isinstance(v, dict):
        raise ConfigError(f"config key '{where}{key}' is required")
    return v


@dataclass(frozen=True)
class LinonexHeads:
    """The sizes and constants of one head layout: the matrix memory, or one side of the parallel mixer."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    gate_cap: float = 0.0               # matrix memory
    conv: int = 0                       # both sides of the parallel mixer
    scale: float = 0.0                  # attention
    softcap: Optional[float] = None
    chunk: Optional[int] = None

    @classmethod
    def from_dict(cls, m: dict, w: str, role: str) -> "LinonexHeads":
        heads, dim = _get(m, "heads", int, w), _get(m, "dim", int, w)
        kw = dict(heads=heads, dim=dim, vdim=_get(m, "vdim", int, w, dim))
        if role == "memory":
            return cls(kv_heads=heads, gate_cap=_get(m, "gate_cap", float, w), **kw)
        kw.update(kv_heads=_get(m, "kv_heads", int, w, heads), conv=_get(m, "conv", int, w, 0))
        if role == "delta":
            return cls(**kw)
        mask = m.get("mask")
        return cls(scale=_get(m, "scale", float, w), softcap=_get(m, "softcap", float, w, None),
                   chunk=None if mask is None else _get(mask, "size", int, w + "mask."), **kw)

    def to_dict(self, role: str) -> dict:
        d = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim}
        if role == "memory":
            return {**d, "gate_cap": self.gate_cap}
        d.update(kv_heads=self.kv_heads, conv=self.conv)
        if role == "attention":
            d["scale"] = self.scale
            if self.softcap is not None:
                d["softcap"] = self.softcap
            if self.chunk is not None:
                d["mask"] = {"size": self.chunk}
        return d

    def check(self, w: str, role: str) -> None:
        if min(self.heads, self.dim, self.vdim) < 1:
            raise ConfigError(f"{w}: {self.heads} heads of {self.dim} / {self.vdim}")
        if self.kv_heads < 1 or self.heads % self.kv_heads:
            raise ConfigError(f"{w}: {self.heads} heads do not divide into {self.kv_heads} kv heads")
        if role == "memory" and not self.gate_cap > 0:
            raise ConfigError(f"{w}: gate_cap must be positive, got {self.gate_cap}")
        if self.conv < 0 or (role == "delta" and self.conv < 1):
            raise ConfigError(f"{w}: conv must be at least 1, got {self.conv}")
        if self.softcap is not None and not self.softcap > 0:
            raise ConfigError(f"{w}: softcap must be positive, got {self.softcap}")
        if self.chunk is not None and self.chunk < 1:
            raise ConfigError(f"{w}: mask.size must be at least 1, got {self.chunk}")


@dataclass(frozen=True)
class LinonexMLP:
    """A feed-forward: dense (``experts`` 0) of width ff, or experts of width ff with their router."""
    ff: int
    experts: int = 0
    identity: int = 0
    top: int = 0
    scale: float = 1.0

    @classmethod
    def from_dict(cls, d: dict, w: str) -> "LinonexMLP":
        kind = d.get("kind") if isinstance(d, dict) else None
        if kind == "dense":
            return cls(ff=_get(d, "ff", int, w))
        if kind != "moe":
            raise ConfigError(f"config key '{w}kind' must be 'dense' or 'moe', got {kind!r}")
        e, r = _mapping(d, "expert", w), _mapping(d, "router", w)
        return cls(ff=_get(e, "ff", int, w + "expert."), experts=_get(r, "experts", int, w + "router."),
                   identity=_get(r, "identity", int, w + "router.", 0), top=_get(r, "top", int, w + "router."),
                   scale=_get(r, "scale", float, w + "router.", 1.0))

    def to_dict(self) -> dict:
        if not self.experts:
            return {"kind": "dense", "ff": self.ff}
        return {"kind": "moe", "expert": {"ff": self.ff},
                "router": {"experts": self.experts, "identity": self.identity, "top": self.top, "scale": self.scale}}

    def check(self, w: str) -> None:
        if self.ff < 1 or self.experts < 0 or self.identity < 0:
            raise ConfigError(f"{w}: feed-forward of {self.ff}, {self.experts} experts, {self.identity} identity experts")
        if self.experts and not 1 <= self.top <= self.experts + self.identity:
            raise ConfigError(f"{w}: top {self.top} of {self.experts} + {self.identity} experts")


@dataclass(frozen=True)
class LinonexLayer:
    type: str
    memory: Optional[LinonexHeads] = None      # mlstm
    left: Optional[LinonexHeads] = None        # parallel
    right: Optional[LinonexHeads] = None
    mlp: Optional[LinonexMLP] = None

    @classmethod
    def from_dict(cls, d: dict, i: int) -> "LinonexLayer":
        where = f"layers[{i}]."
        typ = d.get("type") if isinstance(d, dict) else None
        if typ not in LAYER_TYPES:
            raise ConfigError(f"config key '{where}type' must be one of {LAYER_TYPES}, got {typ!r}")
        mlp = d.get("mlp")
        mlp = None if mlp is None else LinonexMLP.from_dict(mlp, where + "mlp.")
        m, w = _mapping(d, "mixer", where), where + "mixer."
        if typ == "mlstm":
            return cls(type=typ, memory=LinonexHeads.from_dict(m, w, "memory"), mlp=mlp)
        return cls(type=typ, left=LinonexHeads.from_dict(_mapping(m, "left", w), w + "left.", "attention"),
                   right=LinonexHeads.from_dict(_mapping(m, "right", w), w + "right.", "delta"), mlp=mlp)

    def to_dict(self) -> dict:
        m = self.memory.to_dict("memory") if self.memory is not None else \
            {"left": self.left.to_dict("attention"), "right": self.right.to_dict("delta")}
        return {"type": self.type, "mixer": m, "mlp": None if self.mlp is None else self.mlp.to_dict()}

    def check(self, w: str) -> None:
        for heads, role, name in ((self.memory, "memory", ""), (self.left, "attention", ".left"), (self.right, "delta", ".right")):
            if heads is not None:
                heads.check(w + name, role)
        if self.mlp is not None:
            self.mlp.check(w)


@dataclass(frozen=True)
class LinonexConfig:
    vocab: int
    width: int
    layers: Tuple[LinonexLayer, ...]
    eps: float
    max_positions: int
    loop: Optional[Tuple[int, int, int]] = None      # start, stop, times
    stop_ids: Tuple[int, ...] = field(default_factory=tuple)
    torch_dtype: Optional[str] = None
    tie_embeddings: Optional[bool] = False
    architecture: str = "Linonex"

    def __post_init__(self):
        if self.vocab <= 0 or self.width <= 0 or not self.layers:
            raise ConfigError("vocab, width and the number of layers must be positive")
        if self.max_positions <= 0:
            raise ConfigError(f"max_positions must be positive, got {self.max_positions}")
        if self.loop is not None:
            a, b, n = self.loop
            if not 0 <= a < b <= len(self.layers) or n < 1:
                raise ConfigError(f"loop: layers {a} to {b} of {len(self.layers)}, {n} times")
        for i, l in enumerate(self.layers):
            l.check(f"layers[{i}]")

    # ------------------------------------------------------------- config.json
    @classmethod
    def from_dict(cls, d: dict) -> "LinonexConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config key 'layers' must be a list with at least one layer")
        eos = d.get("eos_token_id")
        stops = () if eos is None else (eos,) if isinstance(eos, int) else tuple(eos)
        dt, loop = d.get("torch_dtype", d.get("dtype")), d.get("loop")
        return cls(vocab=_get(d, "vocab", int, ""), width=_get(d, "width", int, ""),
                   layers=tuple(LinonexLayer.from_dict(l, i) for i, l in enumerate(layers)),
                   eps=_get(d.get("norm"), "eps", float, "norm."), max_positions=_get(d, "max_positions", int, ""),
                   loop=None if loop is None else tuple(_get(loop, k, int, "loop.") for k in ("start", "stop", "times")),
                   stop_ids=stops, torch_dtype=dt[6:] if isinstance(dt, str) and dt.startswith("torch.") else dt)

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
             "max_positions": self.max_positions, "norm": {"eps": self.eps}, "layers": [l.to_dict() for l in self.layers]}
        if self.loop is not None:
            d["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.torch_dtype is not None:
            d["torch_dtype"] = self.torch_dtype
        if self.stop_ids:
            d["eos_token_id"] = list(self.stop_ids)
        return d

    def default_engine_dtype(self) -> str:
        return "float32" if self.torch_dtype == "float32" else "bfloat16"

    def with_layers(self, n: int) -> "LinonexConfig":
        """The first n layers; a loop keeps the layers of it that stay, or goes with them."""
        n, loop = int(n), self.loop
        if loop is not None:
            loop = None if loop[0] >= n else (loop[0], min(loop[1], n), loop[2])
        return dataclasses.replace(self, layers=self.layers[:n], loop=loop)

    # ------------------------------------------------------------ model layout
    def runs(self) -> Tuple[RunSpec, ...]:
        """The order in which layers run; every pass of the loop but the first begins with the embedding's
        rows. A run owns its cache and state, so every pass of a looped layer has its own."""
        n = len(self.layers)
        if self.loop is None:
            return tuple(RunSpec(block=i) for i in range(n))
        a, b, times = self.loop
        out = [RunSpec(block=i) for i in range(a)]
        for t in range(times):
            out += [RunSpec(block=i, reenter=t > 0 and i == a) for i in range(a, b)]
        return tuple(out + [RunSpec(block=i) for i in range(b, n)])

    def _mixer(self, l: LinonexLayer):
        d = self.width
        if l.type == "mlstm":
            m = l.memory
            return MatrixMemorySpec(hidden=d, num_heads=m.heads, key_dim=m.dim, value_dim=m.vdim, gate_cap=m.gate_cap,
                                    eps=self.eps)
        a, r = l.left, l.right
        left = SinkAttentionSpec(hidden=d, num_heads=a.heads, num_kv_heads=a.kv_heads, key_dim=a.dim, value_dim=a.vdim,
                                 scale=a.scale, softcap=a.softcap, conv_taps=a.conv, chunk=a.chunk)
        right = GatedDeltaSpec(hidden=d, num_heads=r.heads, num_kv_heads=r.kv_heads, key_dim=r.dim, value_dim=r.vdim,
                               taps=r.conv, decay_rank=None, gate_rank=None, eps=self.eps, gate_activation="silu")
        return BranchMeanSpec(hidden=d, eps=self.eps, branches=(left, right), names=("left", "right"))

    def _ffn(self, m: LinonexMLP):
        if not m.experts:
            return GLUSpec(hidden=self.width, intermediate=m.ff, activation="silu")
        return RoutedMLPSpec(hidden=self.width, experts=m.experts, top=m.top, intermediate=m.ff, activation="silu",
                             score="softmax", weight_on="output", form="glu", identity=m.identity, correction=True,
                             factor=m.scale)

    def model_spec(self) -> ModelSpec:
        d = self.width
        norm = NormSpec(size=d, eps=self.eps)
        blocks = tuple(BlockSpec(norm1=norm, mixer=self._mixer(l), norm2=norm if l.mlp is not None else None,
                                 ffn=None if l.mlp is None else self._ffn(l.mlp)) for l in self.layers)
        spec = ModelSpec(vocab=self.vocab, hidden=d, blocks=blocks, schedule=self.runs(), final_norm=norm,
                         tie_embeddings=False, max_position=self.max_positions, stop_ids=self.stop_ids,
                         after_embed=LearnedPositionSpec(hidden=d, positions=self.max_positions))
        spec.validate()
        return spec
