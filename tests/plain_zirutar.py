"""Plain, slow Zirutar decoder: the oracle of the Zirutar tests.

Whole sequences, no cache, NumPy float64, one function per mechanism. It shares no code
with ``transformer_amd``: it reads config.json and the safetensors file itself (through the
test-suite's own reader) and states every formula once more.

Notation: T tokens, d the model's width, x the residual stream [T, d]. A weight ``W`` is
stored [out, in] and used as ``h @ W.T``.

A layer is ``x <- x + mixer(n1(x))``, then ``x <- x + ff(n2(x))`` where it has a feed-forward, then
the token's own input of that layer. The gains of n1, n2 and of the last norm are stored around
zero. A range of layers may run several times in a row; a row of ``loop.step`` opens each pass.
Mixers: "attention" (keys and values from one projection, normed queries and keys, a window that
keeps the first tokens, a gate per head), "latent_attention" (a cached latent, rotated parts, a
learned extra denominator term per head) and "channel_delta" (a delta rule on a matrix state with
a decay per head and key channel, behind short convolutions).
"""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np

from plain_llama import read_safetensors, round_bf16  # noqa: F401  (the suite's own file code)
from plain_vametar import write_safetensors  # noqa: F401

UNIT_EPS = 1e-6             # under the root of the unit vectors' length
GATE_SLOPE = 1.702          # of the feed-forward's gate


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


def gelu_tanh(z):
    z = np.asarray(z, dtype=np.float64)
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def unit_rms(x, eps):
    x = np.asarray(x, dtype=np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def offset_norm(x, weight, eps):
    """The stream's norm: a gain of 1 + weight."""
    return unit_rms(x, eps) * (1.0 + weight)


def unit_length(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + UNIT_EPS)


# --------------------------------------------------------------------------
# softmax mixers
# --------------------------------------------------------------------------
def visible(T, size, keep_first):
    """[T, T] booleans: row i marks the keys that position i sees. size None: every earlier one."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    see = j <= i
    if size is not None:
        see &= (i - j < size) | (j < keep_first)
    return see


def softmax_rows(scores, see, sink=None):
    """Softmax over the visible keys of every row; sink: a further term exp(sink) below the line."""
    s = np.where(see, scores, -np.inf)
    top = s.max(axis=-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, sink)
    e = np.exp(s - top)
    den = e.sum(axis=-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink - top)
    return e / den


def shared_kv_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, G, dh = m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[p + "q"].T).reshape(T, H, dh)
    k = (h @ w[p + "k"].T).reshape(T, G, dh)
    v = k                                                   # the keys before their norm
    qn, kn = unit_rms(q, eps), unit_rms(k, eps)
    mask = m.get("mask") or {}
    see = visible(T, mask.get("size"), mask.get("keep_first", 0))
    out = np.zeros((T, H, dh))
    for a in range(H):
        g = a // (H // G)
        out[:, a] = softmax_rows(qn[:, a] @ kn[:, g].T * m["scale"], see) @ v[:, g]
    out *= sigmoid(h @ w[p + "g"].T)[:, :, None]
    return out.reshape(T, H * dh) @ w[p + "o"].T


def rotate_neighbours(t, positions, base, dims):
    """t: [T, heads, n]. Coordinates (2i, 2i + 1), i < dims / 2, turn by position * base^(-2i/dims)."""
    out = np.array(t, dtype=np.float64)
    i = np.arange(dims // 2, dtype=np.float64)
    ang = np.asarray(positions, dtype=np.float64)[:, None] * float(base) ** (-2.0 * i / dims)
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    u, v = t[..., 0:dims:2], t[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def latent_attention(h, w, p, m, eps):
    T = h.shape[0]
    H, dn, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos, rot = np.arange(T), m["rot"]
    q = (h @ w[p + "q"].T).reshape(T, H, dn + dr)
    qr = rotate_neighbours(q[..., dn:], pos, rot["base"], rot["dims"])
    both = h @ w[p + "dkv"].T
    c = unit_rms(both[:, :r], eps) * w[p + "dkv.norm"]
    kr = rotate_neighbours(both[:, None, r:], pos, rot["base"], rot["dims"])[:, 0]
    kn = (c @ w[p + "uk"].T).reshape(T, H, dn)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    see = visible(T, None, 0)
    out = np.zeros((T, H, dv))
    for a in range(H):
        s = (q[:, a, :dn] @ kn[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out[:, a] = softmax_rows(s, see, w[p + "sink"][a]) @ v[:, a]
    return out.reshape(T, H * dv) @ w[p + "o"].T


# --------------------------------------------------------------------------
# the delta rule
# --------------------------------------------------------------------------
def causal_conv(x, taps):
    """x [T, C], taps [C, n]: y_t = sum_j taps[:, n - 1 - j] x_(t-j), zeros before the start."""
    n = taps.shape[1]
    padded = np.vstack([np.zeros((n - 1, x.shape[1])), x])
    return sum(padded[j:j + x.shape[0]] * taps[:, j] for j in range(n))


def delta_rule(q, k, v, decay, beta, state=None):
    """Per head a state S [dk, dv]; every token: S <- diag(decay) S, u = beta (v - S^T k),
    S <- S + k u^T, o = S^T q. q, k, decay [T, H, dk]; v [T, H, dv]; beta [T, H].
    Returns (o [T, H, dv], S [H, dk, dv])."""
    T, H, dk = q.shape
    S = np.zeros((H, dk, v.shape[2])) if state is None else np.array(state, dtype=np.float64)
    o = np.zeros(v.shape)
    for t in range(T):
        S = S * decay[t][:, :, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = np.einsum("hkv,hk->hv", S, q[t])
    return o, S


def delta_decay(h, w, p, m):
    """[T, H, dk]: what the rows of the state are multiplied by."""
    T, H = h.shape[0], m["heads"]
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    rate = np.exp(w[p + "A_log"])[None, :, None]
    return np.exp(-rate * softplus(z).reshape(T, H, m["dim"]))


def channel_delta(h, w, p, m, eps):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m["vdim"]

    def stream(n, heads, width):
        return silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])).reshape(T, heads, width)

    q = unit_length(stream("q", G, dk)) * dk ** -0.5
    k = unit_length(stream("k", G, dk))
    v = stream("v", H, dv)
    beta = sigmoid(h @ w[p + "b"].T)
    o, _ = delta_rule(np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1), v, delta_decay(h, w, p, m), beta)
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, dv)
    return (unit_rms(o, eps) * w[p + "norm"] * gate).reshape(T, H * dv) @ w[p + "o"].T


# --------------------------------------------------------------------------
# feed-forward, token input
# --------------------------------------------------------------------------
def limited_glu(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w[p + "down"].T


def token_side(x, tokens, w, layer, dim, eps):
    """What the layer's token input adds to the stream."""
    e = w["side.embed"][np.asarray(tokens), layer * dim:(layer + 1) * dim]
    y = (gelu_tanh(x @ w[f"l{layer}.side.gate"].T) * e) @ w[f"l{layer}.side.proj"].T
    return unit_rms(y, eps) * w[f"l{layer}.side.norm"]


# --------------------------------------------------------------------------
# the model
# --------------------------------------------------------------------------
def schedule(c):
    """[(layer, pass that it opens or None)] in the order in which layers run."""
    n, loop = len(c["layers"]), c.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


class PlainZirutar:
    def __init__(self, folder=None, config=None, weights=None):
        if folder is not None:
            config = json.loads((Path(folder) / "config.json").read_text())
            weights = read_safetensors(Path(folder) / "model.safetensors")
        self.c, self.w = config, weights

    def forward(self, tokens, layers_out=None):
        """Logits [T, vocab] of a whole sequence from position 0. ``layers_out``: a list that
        receives the residual stream after every layer run."""
        c, w = self.c, self.w
        eps = c["norm"]["eps"]
        tokens = np.asarray(tokens, dtype=np.int64)
        x = w["embed"][tokens] * (c.get("embedding") or {}).get("scale", 1.0)
        side = (c.get("token_side") or {}).get("dim")
        mixers = {"attention": shared_kv_attention, "latent_attention": latent_attention,
                  "channel_delta": channel_delta}
        for li, opens in schedule(c):
            layer, L = c["layers"][li], f"l{li}."
            if opens is not None:
                x = x + w["loop.step"][opens]
            x = x + mixers[layer["type"]](offset_norm(x, w[L + "norm1"], eps), w, L + "mix.", layer["mixer"], eps)
            mlp = layer.get("mlp")
            if mlp is not None:
                assert mlp["kind"] == "dense"
                x = x + limited_glu(offset_norm(x, w[L + "norm2"], eps), w, L + "mlp.", mlp["limit"])
            if side:
                x = x + token_side(x, tokens, w, li, side, eps)
            if layers_out is not None:
                layers_out.append(x.copy())
        return offset_norm(x, w["final.norm"], eps) @ w["embed"].T * c.get("logit_scale", 1.0)


# --------------------------------------------------------------------------
# random models for the tests
# --------------------------------------------------------------------------
def tensor_shapes(c, ranks=(3, 5)):
    """{tensor name: shape} of a configuration, in the file's own names. ranks: the widths of
    the low-rank inputs of a channel_delta mixer's decay and gate, which no config key gives (a
    layer's mixer may name its own as "ranks")."""
    d, V = c["width"], c["vocab"]
    s = {"embed": (V, d), "final.norm": (d,)}
    side = (c.get("token_side") or {}).get("dim")
    if side:
        s["side.embed"] = (V, side * len(c["layers"]))
    if c.get("loop"):
        s["loop.step"] = (c["loop"]["times"], d)
    for li, layer in enumerate(c["layers"]):
        L, m, M = f"l{li}.", layer["mixer"], f"l{li}.mix."
        s[L + "norm1"] = (d,)
        H = m["heads"]
        G = m.get("kv_heads", H)
        if layer["type"] == "attention":
            s[M + "q"], s[M + "k"] = (H * m["dim"], d), (G * m["dim"], d)
            s[M + "g"], s[M + "o"] = (H, d), (d, H * m["dim"])
        elif layer["type"] == "latent_attention":
            dn, dr, dv, r = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            s[M + "q"], s[M + "dkv"], s[M + "dkv.norm"] = (H * (dn + dr), d), (r + dr, d), (r,)
            s[M + "uk"], s[M + "uv"], s[M + "sink"], s[M + "o"] = (H * dn, r), (H * dv, r), (H,), (d, H * dv)
        else:
            dk, dv, n = m["dim"], m["vdim"], m["conv"]
            ra, rg = m.get("ranks", ranks)
            for name, rows in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
                s[M + name], s[M + name + ".conv"] = (rows, d), (rows, n)
            s[M + "b"], s[M + "A_log"], s[M + "norm"] = (H, d), (H,), (dv,)
            s[M + "a1"], s[M + "a2"], s[M + "dt_bias"] = (ra, d), (H * dk, ra), (H * dk,)
            s[M + "g1"], s[M + "g2"], s[M + "o"] = (rg, d), (H * dv, rg), (d, H * dv)
        if layer.get("mlp") is not None:
            ff, F = layer["mlp"]["ff"], L + "mlp."
            s[L + "norm2"] = (d,)
            s[F + "gate"], s[F + "up"], s[F + "down"] = (ff, d), (ff, d), (d, ff)
        if side:
            s[L + "side.gate"], s[L + "side.proj"], s[L + "side.norm"] = (side, d), (d, side), (d,)
    return s


def random_weights(c, seed, edit=None):
    """float64 weights, already rounded to bfloat16 values so that a bfloat16 file holds them
    exactly. Matrices ~ N(0, 1/sqrt(in)), the feed-forward's gate and up matrices larger so that
    their limits are met, the token input's gate smaller (far down gelu's tail all its numbers are near
    zero, and the norm behind them would blow up their rounding); stored-around-zero gains near 0, the others near 1; decays between about
    0.3 and 0.999 a token, so that a state forgets and also remembers."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_shapes(c).items():
        last = name.rsplit(".", 1)[-1]
        if last in ("norm1", "norm2") or name == "final.norm":
            a = 0.2 * rng.standard_normal(shape)
        elif last == "norm":
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif last == "sink":
            a = 1.0 + rng.standard_normal(shape)
        elif last == "A_log":
            a = rng.uniform(-1.0, 1.0, shape)
        elif last == "dt_bias":
            a = rng.uniform(-5.0, 0.0, shape)
        elif last == "conv":
            a = rng.standard_normal(shape) / np.sqrt(shape[-1])
        elif name in ("embed", "side.embed"):
            a = rng.standard_normal(shape) * (0.3 if name == "embed" else 1.0)
        elif name == "loop.step":
            a = 0.7 * rng.standard_normal(shape)
        elif name.endswith("side.gate"):
            a = 0.3 * rng.standard_normal(shape) / np.sqrt(shape[-1])
        elif ".mlp." in name and last in ("gate", "up"):
            a = 1.5 * rng.standard_normal(shape) / np.sqrt(shape[-1])
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
    cfg = json.loads(json.dumps(c))
    for layer in cfg["layers"]:                       # the file says it: a tensor's shape
        layer["mixer"].pop("ranks", None)
    (folder / "config.json").write_text(json.dumps(cfg, indent=1))
    return w
