"""The Linonex decoder as a registry entry: its configuration, its blocks and where its
parameters are found in a safetensors file.

File names: ``embed``, ``pos``, ``head``, ``final.norm``, and per layer i ``l<i>.norm1``, ``l<i>.norm2``, the
mixer under ``l<i>.mix.`` and the feed-forward under ``l<i>.mlp.``. An mlstm mixer has ``q, k, v, g, o, norm``
and the gates ``i, i.b, f, f.b``; a parallel mixer ``left.{q, k, v}`` with taps ``.conv``, ``left.o``,
``right.{q, k, v}`` with taps ``.conv``, ``right.{g, a, b, A_log, dt_bias, norm, o}`` and the branch norms
``left.out``, ``right.out``. A dense feed-forward has ``gate, up, down``, a routed one ``router``,
``correction`` and ``e<j>.{gate, up, down}``. Projections that read the same rows are joined by rows into one
matrix: q, k, v, the output gate and both kinds of gate inputs; q, k, v of the attention (and their taps); q,
k, v, the gate, the decays and the step sizes of the delta rule (and the taps); gate and up, of every expert
one after another; all experts' down matrices.
"""
from __future__ import annotations

from typing import Dict

from ..config.linonex import LinonexConfig
from ..config.registry import Architecture, register_architecture
from ..config.spec import ConfigError
from ..weights.loader import Piece, Source


def _one(name, shape):
    return Source(options=((Piece(name, tuple(shape)),),))


def _join(*pieces):
    return Source(options=(tuple(Piece(n, tuple(s)) for n, s in pieces),))


def _memory(src, q, m, c, d):
    nk, nv = c.heads * c.dim, c.heads * c.vdim
    rows = (("q", nk), ("k", nk), ("v", nv), ("g", nv), ("i", c.heads), ("f", c.heads))
    src[q + "in.weight"] = _join(*[(m + n, (r, d)) for n, r in rows])
    src[q + "i.bias"], src[q + "f.bias"] = _one(m + "i.b", (c.heads,)), _one(m + "f.b", (c.heads,))
    src[q + "norm.weight"] = _one(m + "norm", (nv,))
    src[q + "out.weight"] = _one(m + "o", (d, nv))


def _convolved(src, q, m, rows, taps, more, d):
    """q, k, v of one side with their taps; ``more``: the projections behind them in the same matrix."""
    src[q + "in.weight"] = _join(*[(m + n, (r, d)) for n, r in (*rows, *more)])
    if taps:
        src[q + "conv.weight"] = _join(*[(m + n + ".conv", (r, taps)) for n, r in rows])


def _parallel(src, q, m, left, right, d):
    a, A, B = left, m + "left.", q + "left."
    _convolved(src, B, A, (("q", a.heads * a.dim), ("k", a.kv_heads * a.dim), ("v", a.kv_heads * a.vdim)), a.conv, (), d)
    src[B + "out.weight"] = _one(A + "o", (d, a.heads * a.vdim))
    r, R, B = right, m + "right.", q + "right."
    nv = r.heads * r.vdim
    _convolved(src, B, R, (("q", r.kv_heads * r.dim), ("k", r.kv_heads * r.dim), ("v", nv)), r.conv,
               (("g", nv), ("a", r.heads), ("b", r.heads)), d)
    src[B + "dt_bias"], src[B + "A_log"] = _one(R + "dt_bias", (r.heads,)), _one(R + "A_log", (r.heads,))
    src[B + "norm.weight"], src[B + "out.weight"] = _one(R + "norm", (r.vdim,)), _one(R + "o", (d, nv))
    src[q + "norms.left"], src[q + "norms.right"] = _one(A + "out", (d,)), _one(R + "out", (d,))


def linonex_weight_sources(cfg: LinonexConfig, file_format: str) -> Dict[str, Source]:
    if file_format != "safetensors":
        raise ValueError(f"Linonex weights come as safetensors, not {file_format!r}")
    d, V = cfg.width, cfg.vocab
    src = {"embed.weight": _one("embed", (V, d)), "head.weight": _one("head", (V, d)),
           "after_embed.table": _one("pos", (cfg.max_positions, d)), "final_norm.weight": _one("final.norm", (d,))}
    for i, l in enumerate(cfg.layers):
        f, p = f"l{i}.", f"blocks.{i}."
        src[p + "norm1.weight"] = _one(f + "norm1", (d,))
        if l.type == "mlstm":
            _memory(src, p + "mixer.", f + "mix.", l.memory, d)
        else:
            _parallel(src, p + "mixer.", f + "mix.", l.left, l.right, d)
        e = l.mlp
        if e is None:
            continue
        g, q = f + "mlp.", p + "ffn."
        src[p + "norm2.weight"] = _one(f + "norm2", (d,))
        if not e.experts:
            src[q + "gate_up.weight"] = _join((g + "gate", (e.ff, d)), (g + "up", (e.ff, d)))
            src[q + "down.weight"] = _one(g + "down", (d, e.ff))
            continue
        n = e.experts + e.identity
        src[q + "router.weight"], src[q + "router.correction"] = _one(g + "router", (n, d)), _one(g + "correction", (n,))
        src[q + "experts.gate_up.weight"] = _join(*[(f"{g}e{j}.{k}", (e.ff, d)) for j in range(e.experts)
                                                    for k in ("gate", "up")])
        src[q + "experts.down.weight"] = _join(*[(f"{g}e{j}.down", (d, e.ff)) for j in range(e.experts)])
    return src


def _no_gguf(meta, rows=None):
    raise ConfigError("Linonex models are read from a folder with config.json and model.safetensors")


LINONEX = Architecture(
    name="Linonex",
    config_from_dict=LinonexConfig.from_dict,
    config_from_gguf=_no_gguf,
    model_spec=lambda cfg: cfg.model_spec(),
    weight_sources=linonex_weight_sources,
)

register_architecture(LINONEX, "linonex")
