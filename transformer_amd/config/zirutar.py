"""Typed configuration of the Zirutar decoder, read from its own config.json.

A Zirutar model is a list of pre-norm layers ``x <- x + mixer(n1(x))``, then ``x <- x + ff(n2(x))``
where the layer has a feed-forward, then a small input derived from the token itself. Three mixers:
"attention" (grouped-query softmax attention whose values are its keys as projected, heads of q and k
divided by their root mean square, no positions in the scores, a sliding window beside which a
sequence's first tokens stay visible, a gate per head), "latent_attention" (a cached latent per token,
a rotated key part that the heads share, a learned extra term of the softmax denominator per head)
and "channel_delta" (a delta rule on a matrix state with a decay per head and key channel, behind short
convolutions). The feed-forward is a gated unit with limits. The stream's norms have gains stored
around zero; a span of layers can be walked more than once, each repeat with cache layers and state rows
of its own and a learned row added to the stream in front of it; the embedding is scaled and
doubles as the output matrix, whose logits are scaled.

Keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_scale``,
``token_side.dim``, ``loop.{start, stop, times}``, ``layers[i].{type, mixer, mlp}``. ``mixer`` by type:
attention: heads, kv_heads, dim, vdim (= dim), scale, mask.{size, keep_first}; latent_attention: heads,
dim, rot_dim, vdim, kv_rank, scale, rot.{base, dims}; channel_delta: heads, kv_heads, dim, vdim, conv
(the widths of the decay's and the gate's low-rank inputs are tensors' shapes: ``complete_from_file``
reads them; a configuration made by hand may give them as ``decay_rank`` and ``gate_rank``). ``mlp``:
null or ``{kind: "dense", ff, limit}``. Absent keys mean absent mechanisms: no ``mask``: every earlier
token is seen; no ``keep_first``: the window alone; no ``loop``: every layer once; no ``token_side``: no
token input; ``kv_heads`` defaults to ``heads``, ``vdim`` to ``dim``, the scales to 1.
"""
from __future__ import annotations

import dataclasses
from dataclasses import dataclass, field
from typing import Optional, Tuple

from .spec import (BlockSpec, ChainSpec, ConfigError, EmbedScaleSpec, GatedDeltaSpec, GLUSpec, LatentAttentionSpec,
                   LogitScaleSpec, ModelSpec, OffsetNormSpec, RunSpec, SinkAttentionSpec, TokenSideSpec,
                   TokenSideTableSpec)
from .vametar import _get

LAYER_TYPES = ("attention", "latent_attention", "channel_delta")
# fixed by the design: g * sigmoid(GATE_SLOPE * g) * (u + UP_SHIFT) of the feed-forward
GATE_SLOPE = 1.702
UP_SHIFT = 1.0


@dataclass(frozen=True)
class ZirutarLayer:
    type: str
    heads: int
    dim: int
    vdim: int
    kv_heads: int = 0
    # feed-forward: None or its width, and its limit
    ff: Optional[int] = None
    limit: float = 0.0
    # attention, latent attention
    scale: float = 0.0
    window: Optional[int] = None
    keep_first: int = 0
    rot_dim: int = 0
    kv_rank: int = 0
    rot_dims: int = 0
    rot_base: float = 10000.0
    # channel_delta
    conv: int = 0
    decay_rank: Optional[int] = None     # None until a weight file has said them
    gate_rank: Optional[int] = None

    @classmethod
    def from_dict(cls, d: dict, i: int) -> "ZirutarLayer":
        where = f"layers[{i}]."
        typ = d.get("type") if isinstance(d, dict) else None
        if typ not in LAYER_TYPES:
            raise ConfigError(f"config key '{where}type' must be one of {LAYER_TYPES}, got {typ!r}")
        kw = {}
        mlp = d.get("mlp")
        if mlp is not None:
            kind = mlp.get("kind") if isinstance(mlp, dict) else None
            if kind != "dense":
                raise ConfigError(f"config key '{where}mlp.kind' must be 'dense', got {kind!r}")
            kw.update(ff=_get(mlp, "ff", int, where + "mlp."), limit=_get(mlp, "limit", float, where + "mlp."))
        m, w = d.get("mixer"), where + "mixer."
        if not isinstance(m, dict):
            raise ConfigError(f"config key '{where}mixer' is required")
        heads, dim = _get(m, "heads", int, w), _get(m, "dim", int, w)
        vdim = _get(m, "vdim", int, w, dim)
        if typ == "attention":
            mask = m.get("mask")
            return cls(type=typ, heads=heads, kv_heads=_get(m, "kv_heads", int, w, heads), dim=dim, vdim=vdim,
                       scale=_get(m, "scale", float, w),
                       window=None if mask is None else _get(mask, "size", int, w + "mask."),
                       keep_first=0 if mask is None else _get(mask, "keep_first", int, w + "mask.", 0), **kw)
        if typ == "latent_attention":
            rot, rot_dim = m.get("rot"), _get(m, "rot_dim", int, w)
            return cls(type=typ, heads=heads, kv_heads=heads, dim=dim, vdim=vdim, rot_dim=rot_dim,
                       kv_rank=_get(m, "kv_rank", int, w), scale=_get(m, "scale", float, w),
                       rot_dims=_get(rot, "dims", int, w + "rot.", rot_dim) if rot is not None else 0,
                       rot_base=_get(rot, "base", float, w + "rot.") if rot is not None else 10000.0, **kw)
        return cls(type=typ, heads=heads, kv_heads=_get(m, "kv_heads", int, w, heads), dim=dim, vdim=vdim,
                   conv=_get(m, "conv", int, w), decay_rank=_get(m, "decay_rank", int, w, None),
                   gate_rank=_get(m, "gate_rank", int, w, None), **kw)

    def to_dict(self) -> dict:
        m = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim}
        if self.type == "latent_attention":
            m.update(rot_dim=self.rot_dim, kv_rank=self.kv_rank, scale=self.scale)
            if self.rot_dims:
                m["rot"] = {"base": self.rot_base, "dims": self.rot_dims}
        else:
            m["kv_heads"] = self.kv_heads
        if self.type == "attention":
            m["scale"] = self.scale
            if self.window is not None:
                m["mask"] = {"size": self.window, "keep_first": self.keep_first}
        if self.type == "channel_delta":
            m["conv"] = self.conv
            for n in ("decay_rank", "gate_rank"):
                if getattr(self, n) is not None:
                    m[n] = getattr(self, n)
        mlp = None if self.ff is None else {"kind": "dense", "ff": self.ff, "limit": self.limit}
        return {"type": self.type, "mixer": m, "mlp": mlp}

    def check(self, w: str) -> None:
        if min(self.heads, self.dim, self.vdim) < 1:
            raise ConfigError(f"{w}: {self.heads} heads of {self.dim} / {self.vdim}")
        if self.kv_heads < 1 or self.heads % self.kv_heads:
            raise ConfigError(f"{w}: {self.heads} heads do not divide into {self.kv_heads} kv heads")
        if self.ff is not None and (self.ff < 1 or not self.limit > 0):
            raise ConfigError(f"{w}: feed-forward of {self.ff} with limit {self.limit}")
        if self.type == "attention":
            if self.vdim != self.dim:
                raise ConfigError(f"{w}: the values are the keys, so vdim {self.vdim} must equal dim {self.dim}")
            if self.window is not None and self.window < 1:
                raise ConfigError(f"{w}: mask.size must be at least 1, got {self.window}")
            if self.keep_first < 0:
                raise ConfigError(f"{w}: mask.keep_first must not be negative, got {self.keep_first}")
        elif self.type == "latent_attention":
            if self.kv_rank < 1 or self.rot_dim < 0:
                raise ConfigError(f"{w}: kv_rank {self.kv_rank}, rot_dim {self.rot_dim}")
            if self.rot_dims % 2 or not 0 <= self.rot_dims <= self.rot_dim:
                raise ConfigError(f"{w}: rot.dims {self.rot_dims} must be even and at most rot_dim {self.rot_dim}")
        elif self.conv < 1:
            raise ConfigError(f"{w}: conv must be at least 1, got {self.conv}")


@dataclass(frozen=True)
class ZirutarConfig:
    vocab: int
    width: int
    layers: Tuple[ZirutarLayer, ...]
    eps: float
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    side_dim: Optional[int] = None
    loop: Optional[Tuple[int, int, int]] = None      # start, stop, times
    stop_ids: Tuple[int, ...] = field(default_factory=tuple)
    torch_dtype: Optional[str] = None
    tie_embeddings: Optional[bool] = True            # the embedding table is the output matrix
    architecture: str = "Zirutar"

    def __post_init__(self):
        if self.vocab <= 0 or self.width <= 0 or not self.layers:
            raise ConfigError("vocab, width and the number of layers must be positive")
        if self.side_dim is not None and self.side_dim <= 0:
            raise ConfigError(f"token_side.dim must be positive, got {self.side_dim}")
        if self.loop is not None:
            a, b, n = self.loop
            if not 0 <= a < b <= len(self.layers) or n < 1:
                raise ConfigError(f"loop: layers {a} to {b} of {len(self.layers)}, {n} times")
        for i, l in enumerate(self.layers):
            l.check(f"layers[{i}]")

    # ------------------------------------------------------------- config.json
    @classmethod
    def from_dict(cls, d: dict) -> "ZirutarConfig":
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config key 'layers' must be a list with at least one layer")
        eos = d.get("eos_token_id")
        stops = () if eos is None else (eos,) if isinstance(eos, int) else tuple(eos)
        dt = d.get("torch_dtype", d.get("dtype"))
        side, loop = d.get("token_side"), d.get("loop")
        return cls(vocab=_get(d, "vocab", int, ""), width=_get(d, "width", int, ""),
                   layers=tuple(ZirutarLayer.from_dict(l, i) for i, l in enumerate(layers)),
                   eps=_get(d.get("norm"), "eps", float, "norm."),
                   embed_scale=_get(d.get("embedding"), "scale", float, "embedding.", 1.0),
                   logit_scale=_get(d, "logit_scale", float, "", 1.0),
                   side_dim=None if side is None else _get(side, "dim", int, "token_side."),
                   loop=None if loop is None else tuple(_get(loop, k, int, "loop.") for k in ("start", "stop", "times")),
                   stop_ids=stops, torch_dtype=dt[6:] if isinstance(dt, str) and dt.startswith("torch.") else dt)

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
             "norm": {"eps": self.eps}, "embedding": {"scale": self.embed_scale}, "logit_scale": self.logit_scale,
             "layers": [l.to_dict() for l in self.layers]}
        if self.side_dim is not None:
            d["token_side"] = {"dim": self.side_dim}
        if self.loop is not None:
            d["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        if self.torch_dtype is not None:
            d["torch_dtype"] = self.torch_dtype
        if self.stop_ids:
            d["eos_token_id"] = list(self.stop_ids)
        return d

    def complete_from_file(self, file) -> "ZirutarConfig":
        """Sizes that only a tensor's shape gives: the ranks of each channel_delta layer's decay and
        gate inputs."""
        layers = list(self.layers)
        for i, l in enumerate(layers):
            if l.type == "channel_delta":
                found = {n: int(file.shape(t)[0]) for n, t in (("decay_rank", f"l{i}.mix.a1"), ("gate_rank", f"l{i}.mix.g1"))
                         if t in file}
                layers[i] = dataclasses.replace(l, **found)
        return dataclasses.replace(self, layers=tuple(layers))

    def default_engine_dtype(self) -> str:
        return "float32" if self.torch_dtype == "float32" else "bfloat16"

    def with_layers(self, n: int) -> "ZirutarConfig":
        """The first n layers; a loop keeps the layers of it that stay, or goes with them."""
        n, loop = int(n), self.loop
        if loop is not None:
            loop = None if loop[0] >= n else (loop[0], min(loop[1], n), loop[2])
        return dataclasses.replace(self, layers=self.layers[:n], loop=loop)

    # ------------------------------------------------------------ model layout
    def runs(self) -> Tuple[RunSpec, ...]:
        """The order in which layers run; the t-th pass of the loop opens with stream row t. A run owns
        its cache and state, so every pass of a looped layer has its own."""
        n = len(self.layers)
        if self.loop is None:
            return tuple(RunSpec(block=i) for i in range(n))
        a, b, times = self.loop
        out = [RunSpec(block=i) for i in range(a)]
        for t in range(times):
            out += [RunSpec(block=i, opening=t if i == a else None) for i in range(a, b)]
        return tuple(out + [RunSpec(block=i) for i in range(b, n)])

    def _mixer(self, l: ZirutarLayer, i: int):
        d = self.width
        if l.type == "attention":
            return SinkAttentionSpec(hidden=d, num_heads=l.heads, num_kv_heads=l.kv_heads, key_dim=l.dim,
                                     value_dim=l.vdim, scale=l.scale, window=l.window,
                                     keep_first=l.keep_first if l.window is not None else 0, unit_norm=True,
                                     eps=self.eps, values_from_keys=True, head_gate=True)
        if l.type == "latent_attention":
            return LatentAttentionSpec(hidden=d, num_heads=l.heads, nope_dim=l.dim, rope_dim=l.rot_dim,
                                       value_dim=l.vdim, q_rank=None, kv_rank=l.kv_rank, scale=l.scale, eps=self.eps,
                                       rot_dims=l.rot_dims, rot_base=l.rot_base, gated=False, sink=True)
        if l.decay_rank is None or l.gate_rank is None:
            raise ConfigError(f"layers[{i}]: the ranks of the decay and gate inputs are not known: load the model "
                              f"from its folder, or give mixer.decay_rank and mixer.gate_rank")
        return GatedDeltaSpec(hidden=d, num_heads=l.heads, num_kv_heads=l.kv_heads, key_dim=l.dim, value_dim=l.vdim,
                              taps=l.conv, decay_rank=l.decay_rank, gate_rank=l.gate_rank, eps=self.eps)

    def model_spec(self) -> ModelSpec:
        d = self.width
        norm = OffsetNormSpec(size=d, eps=self.eps)
        blocks = []
        for i, l in enumerate(self.layers):
            ffn = None if l.ff is None else GLUSpec(hidden=d, intermediate=l.ff, activation="limited", limit=l.limit,
                                                    gate_slope=GATE_SLOPE, up_shift=UP_SHIFT)
            side = None if self.side_dim is None else TokenSideSpec(hidden=d, dim=self.side_dim,
                                                                    offset=i * self.side_dim, eps=self.eps)
            blocks.append(BlockSpec(norm1=norm, mixer=self._mixer(l, i), norm2=norm if ffn is not None else None,
                                    ffn=ffn, side=side))
        after = [EmbedScaleSpec(scale=self.embed_scale)] if self.embed_scale != 1.0 else []
        if self.side_dim is not None:
            after.append(TokenSideTableSpec(vocab=self.vocab, width=self.side_dim * len(self.layers)))
        spec = ModelSpec(
            vocab=self.vocab, hidden=d, blocks=tuple(blocks), schedule=self.runs(), final_norm=norm,
            tie_embeddings=True, max_position=None, stop_ids=self.stop_ids,
            after_embed=None if not after else after[0] if len(after) == 1 else ChainSpec(parts=tuple(after)),
            on_logits=LogitScaleSpec(scale=self.logit_scale) if self.logit_scale != 1.0 else None,
            stream_rows=0 if self.loop is None else self.loop[2])
        spec.validate()
        return spec
