"""Tiny Linonex configurations and helpers shared by the Linonex tests. Sizes differ between the
configurations and from one another inside each (heads and kv heads, widths, chunks, taps, experts), few are
powers of two, and the corners (one head, as many kv heads as heads, chunks of one token, of a page, no
chunks, no cap, one tap, no identity experts, one expert, top 1, every expert chosen, no feed-forward, no loop,
a loop of one layer, of all layers, of one pass) each appear somewhere."""
import functools
import tempfile

import numpy as np

import plain_linonex as P


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, identity=0, scale=1.0):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "identity": identity, "scale": scale, "top": top}}


def _mem(heads, dim, vdim, cap, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def _left(heads, kv_heads, dim, vdim, conv, scale, chunk=None, softcap=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale}
    if chunk is not None:
        m["mask"] = {"size": chunk}
    if softcap is not None:
        m["softcap"] = softcap
    return m


def _right(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def _par(left, right, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": mlp}


# query heads that share keys, chunks shorter and longer than a page, delta heads that share q and k, a loop over
# the middle in three passes, identity experts
CFG_A = {
    "architecture": "Linonex", "vocab": 211, "width": 72, "max_positions": 600, "norm": {"eps": 1e-5},
    "loop": {"start": 1, "stop": 4, "times": 3},
    "layers": [
        _mem(3, 20, 12, 8.0, _dense(48)),
        _par(_left(6, 2, 20, 20, 3, 0.3, 50, 12.0), _right(6, 3, 24, 12, 4), _moe(6, 2, 20, 3, 1.7)),
        _mem(2, 10, 33, 15.0, _moe(5, 3, 17, 1, 0.8)),
        _par(_left(4, 1, 32, 24, 4, 0.2, 90, 30.0), _right(2, 2, 10, 14, 3), _dense(56)),
        _mem(4, 16, 24, 4.0),
    ],
}
# the corners: one head, no chunks, no cap, one tap, chunks of one token, no feed-forward, every expert chosen, a
# single expert, a loop over all layers
CFG_B = {
    "architecture": "Linonex", "vocab": 50, "width": 64, "max_positions": 400, "norm": {"eps": 1e-6},
    "loop": {"start": 0, "stop": 4, "times": 2},
    "layers": [
        _par(_left(1, 1, 32, 32, 1, 0.2), _right(1, 1, 64, 8, 1)),
        _mem(1, 40, 8, 3.0, _moe(3, 5, 24, 2, 1.0)),
        _par(_left(4, 4, 16, 16, 2, 0.3, 1, 5.0), _right(3, 1, 8, 20, 2), _moe(1, 1, 30)),
        _mem(5, 4, 4, 20.0, _dense(24)),
    ],
}
# wide enough for the library's products of many rows and the matrix-core attention: heads of 128, chunks of
# several pages and of exactly one, memory heads of 64 x 96, a loop of one layer
CFG_C = {
    "architecture": "Linonex", "vocab": 1200, "width": 512, "max_positions": 700, "norm": {"eps": 1e-5},
    "loop": {"start": 2, "stop": 3, "times": 2},
    "layers": [
        _par(_left(8, 2, 128, 128, 4, 0.05, 130, 20.0), _right(8, 4, 64, 96, 4), _moe(12, 3, 256, 4, 2.0)),
        _mem(6, 64, 96, 12.0, _dense(704)),
        _par(_left(16, 16, 32, 32, 3, 0.15, 64, 50.0), _right(4, 4, 128, 64, 3), _dense(640)),
        _mem(4, 128, 160, 10.0, _moe(8, 2, 352, 0, 1.3)),
    ],
}
# a width that is no multiple of four, odd sizes everywhere, values wider than keys, many taps, a loop of one
# pass at the end
CFG_D = {
    "architecture": "Linonex", "vocab": 77, "width": 90, "max_positions": 350, "norm": {"eps": 1e-4},
    "loop": {"start": 2, "stop": 4, "times": 1},
    "layers": [
        _par(_left(5, 5, 7, 11, 9, 0.5, 65, 7.0), _right(3, 1, 33, 7, 9), _moe(7, 4, 13, 5, 0.6)),
        _mem(3, 33, 7, 6.0, _dense(30)),
        _par(_left(3, 1, 40, 6, 2, 0.25, 33), _right(2, 1, 6, 66, 2)),
        _mem(2, 5, 130, 9.0, _dense(18)),
    ],
}
CONFIGS = {"A": (CFG_A, 61), "B": (CFG_B, 62), "C": (CFG_C, 63), "D": (CFG_D, 64)}
STORAGE = {"float32": "F32", "bfloat16": "BF16"}
# a bfloat16 engine may choose another expert than the plain model where the two choice scores are this close
SLACK = 0.06
# largest allowed rms(engine - plain) / rms(plain) over a row of logits
TOL = {"float32": 2e-4, "bfloat16": 1e-1}

_keep = []


def _sharp(w):
    """Peaked softmax and long memories: larger queries make one key stand out, forget gates near one keep
    what was written long ago, so a fault in a single key or a lost state moves the logits."""
    for n in list(w):
        if n.endswith("left.q"):
            w[n] = w[n] * 2.0
        elif n.endswith("mix.f.b"):
            w[n] = w[n] + 3.0
        elif n.endswith("right.A_log"):
            w[n] = w[n] - 2.0


EDITS = {None: None, "sharp": _sharp}


@functools.lru_cache(maxsize=None)
def folder(name, dtype, edit=None):
    cfg, seed = CONFIGS[name]
    d = tempfile.TemporaryDirectory(prefix=f"li_{name}_{dtype}_")
    _keep.append(d)
    P.make_model_folder(d.name, cfg, seed, storage=STORAGE[dtype], edit=EDITS[edit])
    return d.name


@functools.lru_cache(maxsize=None)
def plain(name, dtype, edit=None):
    return P.PlainLinonex(folder(name, dtype, edit))


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


class Routes:
    """Collects the experts that the engine's routed feed-forwards choose, step by step: ``with
    Routes(model) as r`` ... ``r.steps`` is a list of {layer run: [tokens of the step, top]}. A bfloat16 engine
    decides a close call between two experts differently from the float64 plain model now and then; the plain
    model is then told the engine's choice, checks that it was a close call indeed, and follows it. Steps run
    eagerly meanwhile."""

    def __init__(self, model):
        self.model, self.steps = model, []

    def __enter__(self):
        self.steps.append({})
        self.model.dump = self._take
        return self

    def __exit__(self, *exc):
        self.model.dump = None
        return False

    def _take(self, name, t):
        if name.endswith(".experts"):
            self.steps[-1][int(name.split(".")[1])] = t.detach().cpu().numpy().copy()

    def next_step(self):
        self.steps.append({})

    def of_rows(self, rows_of_step):
        """{layer run: [T, top]} of one sequence: rows_of_step[i] = slice of its rows in step i (or None)."""
        out = {}
        for step, rows in zip(self.steps, rows_of_step):
            if rows is None:
                continue
            for run, chosen in step.items():
                out.setdefault(run, []).append(chosen[rows])
        return {run: np.concatenate(parts) for run, parts in out.items()}


def run_cuts(model, cache, slot, toks, cuts, routes=False):
    """Feeds ``toks`` into ``slot`` in portions of the given sizes (the rest one by one) and returns the
    logits of every position, [len(toks), vocab]; with ``routes`` also the experts the engine chose."""
    import contextlib
    from transformer_amd import Entry
    out, at, sizes = [], 0, list(cuts)
    rec = Routes(model) if routes else None
    with rec if rec is not None else contextlib.nullcontext():
        while at < len(toks):
            n = min(sizes.pop(0) if sizes else 1, len(toks) - at)
            out.append(model.step(cache, [Entry(slot, toks[at:at + n], list(range(n)))]).detach().cpu().numpy().copy())
            at += n
            if rec is not None:
                rec.next_step()
    logits = np.concatenate(out, 0)
    return (logits, rec.of_rows([slice(None)] * len(rec.steps))) if routes else logits


def check_against_plain(name, dtype, edit, toks, got, routes=None, what=""):
    """The engine's logits of a sequence's first len(got) tokens against the plain model's; float32: with the
    plain model's own routing, bfloat16: with the engine's, where given."""
    toks = list(toks)[:len(got)]
    if dtype == "float32" or not routes:
        want = plain_logits(name, dtype, edit, tuple(toks))
    else:
        want = plain(name, dtype, edit).forward(toks, routes=routes, slack=SLACK)
    err = row_error(got, want[:len(got)])
    if dtype == "float32":
        assert err.max() < TOL[dtype], f"{what}: {err.max()}"
    else:
        # (a row now and then is badly conditioned: a norm of a readout near zero)
        assert np.quantile(err, 0.98) < TOL[dtype] and err.max() < 2 * TOL[dtype], f"{what}: {np.quantile(err, [0.5, 0.98])} {err.max()}"
