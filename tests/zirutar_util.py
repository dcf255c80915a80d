"""Tiny Zirutar configurations and helpers shared by the Zirutar tests. Sizes differ between the
configurations and from one another inside each (heads and kv heads, widths, ranks, windows, kept first
tokens, taps, token input), few are powers of two, and the corners (one head, as many kv heads as heads,
a window of one token, no window, nothing kept, more kept than a page, kept tokens beyond the window,
no rotated part, one tap, no feed-forward, no token input, no loop, a loop of one layer, of all layers,
of one pass) each appear somewhere."""
import functools
import tempfile

import numpy as np

import plain_zirutar as P


def _dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _att(heads, kv_heads, dim, scale, window=None, keep=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window} if keep is None else {"size": window, "keep_first": keep}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def _lat(heads, dim, rot_dim, vdim, kv_rank, scale, base=1000.0, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim}}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def _delta(heads, kv_heads, dim, vdim, conv, ranks, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "ranks": ranks}
    return {"type": "channel_delta", "mixer": m, "mlp": mlp}


# three query heads per kv head, windows shorter and longer than a page, a loop over the middle in three
# passes, a delta rule whose heads share q and k, a token input of an odd width
CFG_A = {
    "architecture": "Zirutar", "vocab": 211, "width": 72, "norm": {"eps": 1e-5}, "embedding": {"scale": 3.0},
    "logit_scale": 0.7, "token_side": {"dim": 10}, "loop": {"start": 1, "stop": 4, "times": 3},
    "layers": [
        _att(6, 2, 20, 0.6, 50, 7, _dense(48, 1.2)),
        _delta(6, 3, 24, 12, 4, (8, 5), _dense(40, 0.9)),
        _att(4, 1, 32, 0.4, 90, 70, _dense(56, 2.0)),
        _lat(5, 12, 6, 9, 20, 0.3, 500.0, _dense(33, 1.5)),
        _delta(2, 2, 10, 14, 3, (3, 6)),
    ],
}
# the corners: one head, no window, a window of one token, nothing kept, no feed-forward, no token input,
# a loop over all layers, scales left out
CFG_B = {
    "architecture": "Zirutar", "vocab": 50, "width": 64, "norm": {"eps": 1e-6}, "loop": {"start": 0, "stop": 4, "times": 2},
    "layers": [
        _att(1, 1, 32, 0.4),
        _lat(1, 16, 2, 16, 8, 0.25, 20.0),
        _delta(1, 1, 64, 8, 1, (1, 2), _dense(24, 0.5)),
        _att(4, 4, 16, 0.7, 1, 3, _dense(24, 4.0)),
    ],
}
# wide enough for the library's products of many rows and the matrix-core attention: heads of 128, a
# latent of 128 + 32, delta heads of 64 x 96, windows of several pages, a loop of one layer
CFG_C = {
    "architecture": "Zirutar", "vocab": 1200, "width": 512, "norm": {"eps": 1e-5}, "embedding": {"scale": 8.0},
    "logit_scale": 0.4, "token_side": {"dim": 24}, "loop": {"start": 2, "stop": 3, "times": 2},
    "layers": [
        _att(8, 2, 128, 0.09, 200, 130, _dense(704, 1.4)),
        _lat(8, 64, 32, 64, 128, 0.12, 50000.0, _dense(640, 1.1)),
        _delta(8, 4, 64, 96, 4, (32, 16), _dense(512, 0.8)),
        _att(16, 16, 32, 0.35, 70, 0, _dense(704, 1.4)),
    ],
}
# a width that is no multiple of four, odd sizes everywhere, a loop of one pass at the end
CFG_D = {
    "architecture": "Zirutar", "vocab": 77, "width": 90, "norm": {"eps": 1e-4}, "embedding": {"scale": 5.0},
    "logit_scale": 1.3, "token_side": {"dim": 7}, "loop": {"start": 3, "stop": 5, "times": 1},
    "layers": [
        _delta(3, 1, 33, 7, 9, (5, 3), _dense(30, 0.7)),
        _att(5, 5, 7, 1.2, 65, 64, _dense(21, 1.0)),
        _lat(3, 5, 4, 11, 13, 0.4, 100.0),
        _att(3, 1, 40, 0.3, 33, 100, _dense(50, 3.0)),
        _delta(2, 1, 6, 66, 2, (9, 16), _dense(18, 1.1)),
    ],
}
CONFIGS = {"A": (CFG_A, 51), "B": (CFG_B, 52), "C": (CFG_C, 53), "D": (CFG_D, 54)}
STORAGE = {"float32": "F32", "bfloat16": "BF16"}
# largest allowed rms(engine - plain) / rms(plain) over a row of logits
TOL = {"float32": 2e-4, "bfloat16": 1e-1}

_keep = []


def _sharp(w):
    """Peaked softmax in the latent layers (those of "attention" norm their queries and keys; their scale
    says how peaked they are): one key stands out, so a fault in any single one moves the logits."""
    for n in list(w):
        if n.endswith("mix.q") and n[:-1] + "dkv" in w:
            w[n] = w[n] * 4.0


EDITS = {None: None, "sharp": _sharp}


@functools.lru_cache(maxsize=None)
def folder(name, dtype, edit=None):
    cfg, seed = CONFIGS[name]
    d = tempfile.TemporaryDirectory(prefix=f"zi_{name}_{dtype}_")
    _keep.append(d)
    P.make_model_folder(d.name, cfg, seed, storage=STORAGE[dtype], edit=EDITS[edit])
    return d.name


@functools.lru_cache(maxsize=None)
def plain(name, dtype, edit=None):
    return P.PlainZirutar(folder(name, dtype, edit))


@functools.lru_cache(maxsize=None)
def engine(name, dtype, edit=None):
    import transformer_amd as ta
    return ta.load_model(folder(name, dtype, edit), dtype, "cuda:0")


def tokens(name, n, seed):
    cfg, _ = CONFIGS[name]
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


@functools.lru_cache(maxsize=None)
def plain_logits(name, dtype, edit, toks):
    return plain(name, dtype, edit).forward(list(toks))


def row_error(got, want):
    """rms of the difference (mean taken off) over rms of the expected row, per row."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    d = got - want
    d = d - d.mean(axis=-1, keepdims=True)
    return np.sqrt((d ** 2).mean(axis=-1)) / np.sqrt((want ** 2).mean(axis=-1))


def run_cuts(model, cache, slot, toks, cuts):
    """Feeds ``toks`` into ``slot`` in portions of the given sizes (the rest one by one) and
    returns the logits of every position, [len(toks), vocab]."""
    from transformer_amd import Entry
    out, at, sizes = [], 0, list(cuts)
    while at < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - at)
        out.append(model.step(cache, [Entry(slot, toks[at:at + n], list(range(n)))]).detach().cpu().numpy().copy())
        at += n
    return np.concatenate(out, 0)


def check_against_plain(name, dtype, edit, toks, got, what=""):
    """The engine's logits of a sequence's first len(got) tokens against the plain model's."""
    want = plain_logits(name, dtype, edit, tuple(toks))[:len(got)]
    err = row_error(got, want).max()
    assert err < TOL[dtype], f"{what}: {err}"
