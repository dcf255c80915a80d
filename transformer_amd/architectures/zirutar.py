"""The Zirutar decoder as a registry entry: its configuration, its blocks and where its
parameters are found in a safetensors file.

File names: ``embed`` (also the output matrix), ``side.embed``, ``loop.step``, ``final.norm``, and per
layer i ``l<i>.norm1``, ``l<i>.norm2``, the mixer under ``l<i>.mix.``, the feed-forward under
``l<i>.mlp.{gate, up, down}`` and ``l<i>.side.{gate, proj, norm}``. An attention mixer has ``q, k, g, o``;
latent attention ``q, dkv, dkv.norm, uk, uv, sink, o``; a delta mixer ``q, k, v`` with taps ``.conv``,
``a1, a2, g1, g2, b, A_log, dt_bias, norm, o``. Projections that read the same rows are joined by rows into
one matrix: q, k and the heads' gates; the queries and the key/value latent; q, k, v, the low-rank
inputs and the step sizes (and their taps); gate and up.
"""
from __future__ import annotations

from typing import Dict

from ..config.registry import Architecture, register_architecture
from ..config.spec import ConfigError
from ..config.zirutar import ZirutarConfig
from ..weights.loader import Piece, Source


def _one(name, shape):
    return Source(options=((Piece(name, tuple(shape)),),))


def _join(*pieces):
    return Source(options=(tuple(Piece(n, tuple(s)) for n, s in pieces),))


def zirutar_weight_sources(cfg: ZirutarConfig, file_format: str) -> Dict[str, Source]:
    if file_format != "safetensors":
        raise ValueError(f"Zirutar weights come as safetensors, not {file_format!r}")
    d, V = cfg.width, cfg.vocab
    src = {"embed.weight": _one("embed", (V, d)),
           "head.weight": Source(options=(), stand_in="embed.weight"),
           "final_norm.weight": _one("final.norm", (d,))}
    if cfg.loop is not None:
        src["stream_rows"] = _one("loop.step", (cfg.loop[2], d))
    if cfg.side_dim is not None:
        name = "after_embed.1.table" if cfg.embed_scale != 1.0 else "after_embed.table"
        src[name] = _one("side.embed", (V, cfg.side_dim * len(cfg.layers)))
    for i, l in enumerate(cfg.layers):
        f, p = f"l{i}.", f"blocks.{i}."
        src[p + "norm1.weight"] = _one(f + "norm1", (d,))
        m, q = f + "mix.", p + "mixer."
        H, G = l.heads, l.kv_heads
        src[q + "out.weight"] = _one(m + "o", (d, H * l.vdim))
        if l.type == "attention":
            src[q + "in.weight"] = _join((m + "q", (H * l.dim, d)), (m + "k", (G * l.dim, d)), (m + "g", (H, d)))
        elif l.type == "latent_attention":
            src[q + "in.weight"] = _join((m + "q", (H * (l.dim + l.rot_dim), d)), (m + "dkv", (l.kv_rank + l.rot_dim, d)))
            src[q + "kv_norm.weight"] = _one(m + "dkv.norm", (l.kv_rank,))
            src[q + "uk.weight"] = _one(m + "uk", (H * l.dim, l.kv_rank))
            src[q + "uv.weight"] = _one(m + "uv", (H * l.vdim, l.kv_rank))
            src[q + "sink"] = _one(m + "sink", (H,))
        else:
            ra, rg = l.decay_rank, l.gate_rank
            if ra is None or rg is None:
                raise ConfigError(f"layers[{i}]: the ranks of the decay and gate inputs are not known")
            rows = [("q", G * l.dim), ("k", G * l.dim), ("v", H * l.vdim)]
            src[q + "in.weight"] = _join(*[(m + n, (r, d)) for n, r in rows + [("a1", ra), ("g1", rg), ("b", H)]])
            src[q + "conv.weight"] = _join(*[(m + n + ".conv", (r, l.conv)) for n, r in rows])
            src[q + "decay.weight"], src[q + "gate.weight"] = _one(m + "a2", (H * l.dim, ra)), _one(m + "g2", (H * l.vdim, rg))
            src[q + "dt_bias"], src[q + "A_log"] = _one(m + "dt_bias", (H * l.dim,)), _one(m + "A_log", (H,))
            src[q + "norm.weight"] = _one(m + "norm", (l.vdim,))
        if l.ff is not None:
            g, q = f + "mlp.", p + "ffn."
            src[p + "norm2.weight"] = _one(f + "norm2", (d,))
            src[q + "gate_up.weight"] = _join((g + "gate", (l.ff, d)), (g + "up", (l.ff, d)))
            src[q + "down.weight"] = _one(g + "down", (d, l.ff))
        if cfg.side_dim is not None:
            s, q = f + "side.", p + "side."
            src[q + "gate.weight"] = _one(s + "gate", (cfg.side_dim, d))
            src[q + "proj.weight"] = _one(s + "proj", (d, cfg.side_dim))
            src[q + "norm.weight"] = _one(s + "norm", (d,))
    return src


def _no_gguf(meta, rows=None):
    raise ConfigError("Zirutar models are read from a folder with config.json and model.safetensors")


ZIRUTAR = Architecture(
    name="Zirutar",
    config_from_dict=ZirutarConfig.from_dict,
    config_from_gguf=_no_gguf,
    model_spec=lambda cfg: cfg.model_spec(),
    weight_sources=zirutar_weight_sources,
    complete_config=lambda cfg, file: cfg.complete_from_file(file),
)

register_architecture(ZIRUTAR, "zirutar")
