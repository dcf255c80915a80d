"""Plain, slow Linonex decoder: the oracle of the Linonex tests.

Whole sequences, no cache, NumPy float64, one function per mechanism. It shares no code
with ``transformer_amd``: it reads config.json and the safetensors file itself (through the
test-suite's own reader) and states every formula once more.

Notation: T tokens, d the model's width, x the residual stream [T, d]. A weight ``W`` is
stored [out, in] and used as ``h @ W.T``.

A layer is ``x <- x + mixer(n1(x))``, then ``x <- x + ff(n2(x))`` where it has a feed-forward. A range
of layers may run several times in a row; what the embedding gave is added once more in front of
every pass but the first. Mixers: "mlstm" (a matrix memory with exponential gates, a running maximum
and a normaliser) and "parallel" (chunked softmax attention behind short convolutions beside a delta
rule with one decay per head; the mean of their normed results).
"""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np

from plain_llama import read_safetensors, round_bf16  # noqa: F401  (the suite's own file code)
from plain_vametar import write_safetensors  # noqa: F401

UNIT_EPS = 1e-6             # under the root of the unit vectors' length
READ_EPS = 1e-6             # beside the matrix memory's normaliser


# --------------------------------------------------------------------------
# small functions
# --------------------------------------------------------------------------
def sigmoid(z):
    z = np.asarray(z, dtype=np.float64)
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0, e) / (1.0 + e)


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    z = np.asarray(z, dtype=np.float64)
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def cap(z, bound):
    return bound * np.tanh(z / bound)


def unit_rms(x, eps):
    x = np.asarray(x, dtype=np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rms_norm(x, weight, eps):
    return unit_rms(x, eps) * weight


def unit_length(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


def causal_conv(x, taps):
    """x [T, C], taps [C, n]: y_t = sum_j taps[:, n - 1 - j] x_(t-j), zeros before the start."""
    n = taps.shape[1]
    padded = np.vstack([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n))


# --------------------------------------------------------------------------
# the matrix memory
# --------------------------------------------------------------------------
def matrix_memory(q, k, v, i, f, state=None):
    """q, k [T, H, dk], v [T, H, dv], i, f [T, H] the logarithms of the input and the forget gates.
    Returns (o [T, H, dv], (S [H, dk, dv], n [H, dk], m [H]))."""
    T, H, dk = q.shape
    if state is None:
        state = np.zeros((H, dk, v.shape[2])), np.zeros((H, dk)), np.zeros(H)
    S, n, m = (np.array(a, dtype=np.float64) for a in state)
    o = np.zeros(v.shape)
    for t in range(T):
        new = np.maximum(f[t] + m, i[t])
        keep, write = np.exp(f[t] + m - new), np.exp(i[t] - new)
        m = new
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + write[:, None] * k[t]
        below = np.maximum(np.abs(np.sum(n * q[t], axis=-1)), np.exp(-m)) + READ_EPS
        o[t] = np.einsum("hkv,hk->hv", S, q[t]) / below[:, None]
    return o, (S, n, m)


def matrix_memory_sum(q, k, v, i, f):
    """The same readout as a sum over earlier tokens (no state, no running maximum), for cross-checks:
    with F the running sum of f, token j weighs exp(i_j + F_t - F_j), and the floor of the denominator
    is 1 where the memory has not been scaled."""
    T = q.shape[0]
    F = np.cumsum(f, axis=0)
    m = np.zeros(q.shape[1])
    o = np.zeros(v.shape)
    for t in range(T):
        m = np.maximum(f[t] + m, i[t])
        w = np.exp(i[:t + 1] + F[t] - F[:t + 1]) * np.einsum("hk,jhk->jh", q[t], k[:t + 1])
        below = np.maximum(np.abs(w.sum(0)), 1.0) + READ_EPS * np.exp(m)
        o[t] = np.einsum("jh,jhv->hv", w, v[:t + 1]) / below[:, None]
    return o


def mlstm(h, w, p, m, eps):
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dk) * dk ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, dk)
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    i = cap(h @ w[p + "i"].T + w[p + "i.b"], m["gate_cap"])
    f = -softplus(-cap(h @ w[p + "f"].T + w[p + "f.b"], m["gate_cap"]))
    o, _ = matrix_memory(q, k, v, i, f)
    o = unit_rms(o, eps).reshape(T, H * dv) * w[p + "norm"]
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# --------------------------------------------------------------------------
# the two branches
# --------------------------------------------------------------------------
def same_chunk(T, size):
    """[T, T] booleans: row i marks the keys that position i sees. size None: every earlier one."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    see = j <= i
    return see if size is None else see & (i // size == j // size)


def softmax_rows(scores, see):
    s = np.where(see, scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def chunked_attention(h, w, p, m):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])

    def stream(n, heads, width):
        return causal_conv(h @ w[p + n].T, w[p + n + ".conv"]).reshape(T, heads, width)

    q, k, v = stream("q", H, dk), stream("k", G, dk), stream("v", G, dv)
    see = same_chunk(T, (m.get("mask") or {}).get("size"))
    out = np.zeros((T, H, dv))
    for a in range(H):
        g = a // (H // G)
        s = q[:, a] @ k[:, g].T * m["scale"]
        if m.get("softcap") is not None:
            s = cap(s, m["softcap"])
        out[:, a] = softmax_rows(s, see) @ v[:, g]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def delta_rule(q, k, v, decay, beta, state=None):
    """Per head a state S [dk, dv]; every token: S <- decay S, u = beta (v - S^T k), S <- S + k u^T,
    o = S^T q. q, k [T, H, dk]; v [T, H, dv]; decay, beta [T, H]. Returns (o, last S [H, dk, dv])."""
    T, H, dk = q.shape
    S = np.zeros((H, dk, v.shape[2])) if state is None else np.array(state, dtype=np.float64)
    o = np.zeros(v.shape)
    for t in range(T):
        S = S * decay[t][:, None, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o, S


def head_delta(h, w, p, m, eps):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])

    def stream(n, heads, width):
        return silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])).reshape(T, heads, width)

    q = unit_length(stream("q", G, dk)) * dk ** -0.5
    k = unit_length(stream("k", G, dk))
    v = stream("v", H, dv)
    beta = sigmoid(h @ w[p + "b"].T)
    decay = np.exp(-np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o, _ = delta_rule(np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1), v, decay, beta)
    gate = silu(h @ w[p + "g"].T).reshape(T, H, dv)
    return (unit_rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * dv) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps):
    left = chunked_attention(h, w, p + "left.", m["left"])
    right = head_delta(h, w, p + "right.", m["right"], eps)
    return 0.5 * (rms_norm(left, w[p + "left.out"], eps) + rms_norm(right, w[p + "right.out"], eps))


# --------------------------------------------------------------------------
# feed-forwards
# --------------------------------------------------------------------------
def glu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h, w, p, r):
    """(scores [T, E + identity], choice scores): softmax of the router's logits, and what is compared."""
    z = h @ w[p + "router"].T
    e = np.exp(z - z.max(axis=-1, keepdims=True))
    s = e / e.sum(axis=-1, keepdims=True)
    return s, s + w[p + "correction"]


def moe(h, w, p, mlp, forced=None, slack=0.0):
    """forced [T, top]: experts that another implementation chose. Where they differ from this
    function's own choice they must be as good within ``slack`` (a close call that rounding
    decides); the function then goes on with them."""
    r = mlp["router"]
    E, top, factor = r["experts"], r["top"], r.get("scale", 1.0)
    s, choice = route(h, w, p, r)
    chosen = np.argsort(-choice, axis=-1, kind="stable")[:, :top]
    if forced is not None:
        forced = np.asarray(forced, dtype=np.int64)
        for t in range(len(h)):
            if set(forced[t]) != set(chosen[t]):
                assert len(set(forced[t])) == len(forced[t]), f"token {t}: an expert chosen twice"
                assert choice[t, forced[t]].min() >= choice[t, chosen[t]].min() - slack, \
                    f"token {t}: experts {forced[t]} chosen, {chosen[t]} have the largest scores: {choice[t]}"
        chosen = forced
    out = np.zeros(h.shape)
    for t in range(len(h)):
        for e in chosen[t]:
            y = h[t] if e >= E else glu(h[t][None], w, f"{p}e{int(e)}.")[0]
            out[t] += factor * s[t, e] * y
    return out


# --------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------
def schedule(c):
    """[(layer, whether the embedding's rows are added in front of it)] in the order in which layers run."""
    n, loop = len(c["layers"]), c.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, False) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


class PlainLinonex:
    def __init__(self, folder=None, config=None, weights=None):
        if folder is not None:
            config = json.loads((Path(folder) / "config.json").read_text())
            weights = read_safetensors(Path(folder) / "model.safetensors")
        self.c, self.w = config, weights

    def forward(self, tokens, layers_out=None, routes=None, slack=0.02):
        """Logits [T, vocab] of a whole sequence from position 0. ``layers_out``: a list that
        receives the residual stream after every layer run. ``routes``: {layer run: experts [T, top]}
        chosen elsewhere (see ``moe``)."""
        c, w = self.c, self.w
        eps = c["norm"]["eps"]
        tokens = np.asarray(tokens, dtype=np.int64)
        first = w["embed"][tokens] + w["pos"][:len(tokens)]
        x = np.array(first, dtype=np.float64)
        mixers = {"mlstm": mlstm, "parallel": parallel_mixer}
        for run, (li, again) in enumerate(schedule(c)):
            layer, L = c["layers"][li], f"l{li}."
            if again:
                x = x + first
            x = x + mixers[layer["type"]](rms_norm(x, w[L + "norm1"], eps), w, L + "mix.", layer["mixer"], eps)
            mlp = layer.get("mlp")
            if mlp is not None:
                h = rms_norm(x, w[L + "norm2"], eps)
                if mlp["kind"] == "dense":
                    x = x + glu(h, w, L + "mlp.")
                else:
                    x = x + moe(h, w, L + "mlp.", mlp, None if routes is None else routes.get(run), slack)
            if layers_out is not None:
                layers_out.append(x.copy())
        return rms_norm(x, w["final.norm"], eps) @ w["head"].T


# --------------------------------------------------------------------------
# random models for the tests
# --------------------------------------------------------------------------
def tensor_shapes(c):
    """{tensor name: shape} of a configuration, in the file's own names."""
    d, V = c["width"], c["vocab"]
    s = {"embed": (V, d), "pos": (c["max_positions"], d), "final.norm": (d,), "head": (V, d)}
    for li, layer in enumerate(c["layers"]):
        L, m, M = f"l{li}.", layer["mixer"], f"l{li}.mix."
        s[L + "norm1"] = (d,)
        if layer["type"] == "mlstm":
            H, nk, nv = m["heads"], m["heads"] * m["dim"], m["heads"] * m["vdim"]
            s[M + "q"], s[M + "k"], s[M + "v"], s[M + "g"] = (nk, d), (nk, d), (nv, d), (nv, d)
            s[M + "o"], s[M + "norm"] = (d, nv), (nv,)
            for n in "if":
                s[M + n], s[M + n + ".b"] = (H, d), (H,)
        else:
            for side in ("left", "right"):
                b, B = m[side], M + side + "."
                H, G = b["heads"], b.get("kv_heads", b["heads"])
                dk, dv = b["dim"], b.get("vdim", b["dim"])
                rows = {"q": (H if side == "left" else G) * dk, "k": G * dk, "v": (G if side == "left" else H) * dv}
                for n, r in rows.items():
                    s[B + n], s[B + n + ".conv"] = (r, d), (r, b["conv"])
                s[B + "o"], s[B + "out"] = (d, H * dv), (d,)
                if side == "right":
                    s[B + "b"], s[B + "a"], s[B + "g"] = (H, d), (H, d), (H * dv, d)
                    s[B + "A_log"], s[B + "dt_bias"], s[B + "norm"] = (H,), (H,), (dv,)
        mlp, F = layer.get("mlp"), L + "mlp."
        if mlp is None:
            continue
        s[L + "norm2"] = (d,)
        if mlp["kind"] == "dense":
            units = [(F, mlp["ff"])]
        else:
            r = mlp["router"]
            units = [(f"{F}e{e}.", mlp["expert"]["ff"]) for e in range(r["experts"])]
            n = r["experts"] + r.get("identity", 0)
            s[F + "router"], s[F + "correction"] = (n, d), (n,)
        for u, ff in units:
            s[u + "gate"], s[u + "up"], s[u + "down"] = (ff, d), (ff, d), (d, ff)
    return s


def random_weights(c, seed, edit=None):
    """float64 weights, already rounded to bfloat16 values so that a bfloat16 file holds them
    exactly. Matrices ~ N(0, 1/sqrt(in)); gains near 1; queries large enough that the softmax is peaked
    and the cap bites; the matrix memory's gates spread over most of their range (some heads write with
    weights far above one, some forget within a few tokens, some hardly); the delta rule's decays between
    about 0.3 and 0.999 a token; router rows large enough that the chosen experts are seldom a close
    call, corrections that change the choice."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_shapes(c).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2", "norm", "out"):
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif name in ("embed", "pos"):
            a = rng.standard_normal(shape) * (1.0 if name == "embed" else 0.5)
        elif last == "A_log":
            a = rng.uniform(-1.0, 1.0, shape)
        elif last == "dt_bias":
            a = rng.uniform(-5.0, 0.0, shape)
        elif name.endswith("mix.i.b"):
            a = rng.uniform(-3.0, 3.0, shape)
        elif name.endswith("mix.f.b"):
            a = rng.uniform(0.0, 6.0, shape)
        elif last == "conv":
            a = rng.standard_normal(shape) / np.sqrt(shape[-1])
        elif last == "router":
            a = 3.0 * rng.standard_normal(shape) / np.sqrt(shape[-1])
        elif last == "correction":
            a = 0.2 * rng.standard_normal(shape)
        elif name.endswith("left.q"):
            a = 3.0 * rng.standard_normal(shape) / np.sqrt(shape[-1])
        else:
            a = rng.standard_normal(shape) / np.sqrt(shape[-1])
        w[name] = round_bf16(a)
    if edit is not None:
        edit(w)
        for n in w:
            w[n] = round_bf16(w[n].reshape(-1)).reshape(w[n].shape)
    return w


def make_model_folder(folder, c, seed, storage="BF16", edit=None):
    folder = Path(folder)
    folder.mkdir(parents=True, exist_ok=True)
    w = random_weights(c, seed, edit)
    write_safetensors(folder / "model.safetensors", w, dtype=storage)
    (folder / "config.json").write_text(json.dumps(c, indent=1))
    return w
