"""The Linonex decoder on the GPU against the plain implementation in ``plain_linonex``.

Each mechanism alone (its kernels against the plain function, with cache and state carried over
cuts), then the engine: layers, whole prompts, portions, token-by-token decoding, unequal batches, slots
and pages used again, recorded steps, far keys and keys at the borders of pages and chunks, long decoding,
greedy generation, the replayer and the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import linonex_util as U
import plain_linonex as P

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
TD = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def _t(a, dtype=torch.float32):
    return torch.tensor(np.asarray(a), dtype=dtype, device=DEV)


def _bf(a, dtype="bfloat16"):
    from plain_llama import round_bf16
    a = np.asarray(a, dtype=np.float64)
    return round_bf16(a) if dtype == "bfloat16" else a.astype(np.float32).astype(np.float64)


def _f32(a):
    return np.asarray(a, dtype=np.float32).astype(np.float64)


def _np(t):
    return t.detach().float().cpu().numpy().astype(np.float64)


def _close(got, want, dtype, what="", scale=1.0):
    tol = (3e-5 if dtype == "float32" else 2.5e-2) * scale
    assert np.isfinite(got).all() and np.abs(got - want).max() <= tol * max(1.0, np.abs(want).max()), \
        (what, np.abs(got - want).max())


def _selectors(sizes):
    """Matrices that cut consecutive column ranges of the given sizes out of a row."""
    total, at, out = sum(sizes), 0, []
    for n in sizes:
        m = np.zeros((n, total))
        m[np.arange(n), at + np.arange(n)] = 1.0
        out.append(m)
        at += n
    return out


def _run_part(part, hs, cuts, dtype, layers=None, max_slots=5):
    """Runs a mixer over sequences ``hs`` in the given cuts (one size per sequence, 0: left out), in slots that held
    something else; returns (results per sequence, the cache, the slots)."""
    from transformer_amd.cache.storage import SequenceCache
    from transformer_amd.engine.batch import Entry, Uploader, plan_step
    from transformer_amd.parts.linear import Workspace
    need = part.cache_need()
    needs = need if isinstance(need, list) else [need]
    planner = getattr(part, "step_planner", lambda: None)()
    cache = SequenceCache(needs, 2048, max_slots, TD[dtype], DEV, planners=[planner] * len(needs))
    for t in cache.states:
        t.fill_(3.0)
    for t in cache.keys + cache.values:
        t.fill_(float("nan"))
    slots = [cache.alloc_slot() for _ in range(len(hs) + 1)][1:]
    ws, up = Workspace(DEV), Uploader(DEV)
    got, at = [[] for _ in hs], [0] * len(hs)
    for cut in cuts:
        live = [i for i, n in enumerate(cut) if n]
        ctx = plan_step([Entry(slots[i], [0] * cut[i]) for i in live], cache, 10, up, ws)
        h = np.concatenate([hs[i][at[i]:at[i] + cut[i]] for i in live])
        delta, bias = part.run(_t(h, TD[dtype]), ctx, cache, tuple(range(len(needs))) if isinstance(need, list) else 0)
        assert bias is None
        out, o = _np(delta), 0
        out = out.sum(0) if out.ndim == 3 else out
        for i in live:
            got[i].append(out[o:o + cut[i]])
            o += cut[i]
            at[i] += cut[i]
            cache.pool.advance(slots[i], cut[i])
            cache.release_outside_windows(slots[i])
    for t in cache.states:                                  # slots of others stay as they are
        assert float(t[:, 0].abs().max()) == 0.0 and float(t[:, max_slots].min()) == 3.0
    return [np.concatenate(g) for g in got], cache, slots


# ----------------------------------------------------------------------------- mechanisms alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d", [72, 90, 1024])
def test_learned_positions(d, dtype):
    from transformer_amd import kernels as K
    rng = np.random.default_rng(d)
    table, x0 = _bf(rng.standard_normal((50, d)), dtype), rng.standard_normal((9, d)).astype(np.float32)
    at = [0, 49, 7, 7, 13, 1, 2, 50, -1]
    x = K.rows_add(_t(table, TD[dtype]), _t(at, torch.int32), _t(x0))
    np.testing.assert_allclose(_np(x)[:7], x0[:7] + table[at[:7]], atol=1e-6)
    assert torch.isnan(x[7:]).all()                         # a position outside the table


ATT_GEOMS = [(6, 2, 20, 20, 37, 9.0), (4, 4, 16, 24, None, None), (1, 1, 33, 7, 64, None), (5, 5, 7, 11, 65, 3.0), (2, 1, 34, 50, 1, 6.0),
             (4, 1, 40, 40, 200, 30.0), (8, 2, 96, 64, 128, None), (3, 1, 256, 256, 90, 15.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", ATT_GEOMS)
def test_chunked_attention_part_over_cuts(dtype, geom):
    """The softmax side as the mixer runs it: convolution of q, k and v, capped scores, chunks; one sequence in
    cuts beside another, into pages that held NaN, pages of chunks left behind given back meanwhile."""
    from transformer_amd.config.spec import SinkAttentionSpec
    from transformer_amd.parts.base import build_part
    H, G, dk, dv, chunk, cap = geom
    rng = np.random.default_rng(H * 7 + dk)
    d, taps, T = 48, 1 + H % 4, 330
    rows = (("q", H * dk), ("k", G * dk), ("v", G * dv))
    w = {n: _bf((2.5 if n == "q" else 1.0) * rng.standard_normal((r, d)) / np.sqrt(d)) for n, r in rows}
    w.update({n + ".conv": _bf(rng.standard_normal((r, taps)) / np.sqrt(taps)) for n, r in rows})
    w["o"] = _bf(rng.standard_normal((d, H * dv)) / np.sqrt(H * dv))
    m = {"heads": H, "kv_heads": G, "dim": dk, "vdim": dv, "scale": 2.0 * dk ** -0.5}
    if chunk is not None:
        m["mask"] = {"size": chunk}
    if cap is not None:
        m["softcap"] = cap
    part = build_part(SinkAttentionSpec(hidden=d, num_heads=H, num_kv_heads=G, key_dim=dk, value_dim=dv, scale=m["scale"],
                                        softcap=cap, conv_taps=taps, chunk=chunk), TD[dtype], DEV)
    part.bind({"in.weight": _t(np.concatenate([w[n] for n, _ in rows]), TD[dtype]),
               "conv.weight": _t(np.concatenate([w[n + ".conv"] for n, _ in rows])), "out.weight": _t(w["o"], TD[dtype])})
    hs = [_bf(rng.standard_normal((T, d))), _bf(rng.standard_normal((90, d)))]
    cuts = [(70, 3), (120, 60), (1, 1), (1, 1), (2, 2), (8, 0), (1, 1), (1, 1), (2, 0), (124, 21)]
    got, cache, _ = _run_part(part, hs, cuts, dtype)
    for g, h in zip(got, hs):
        _close(g, P.chunked_attention(h, w, "", m), dtype, scale=2.0)
    cache.pool.check()


EDGES = [(0, None), (63, None), (298, None), (200, 100), (199, 100), (256, 64), (255, 64), (258, 129), (257, 129), (299, 1), (298, 1),
         (150, 150), (149, 150), (0, 300), (297, 27), (296, 27), (280, 70), (279, 70)]


@pytest.mark.parametrize("where,kernel", [(w, k) for k in ("vector32", "vector16", "matrix") for w in ("prompt", "decode")] +
                         [("prompt", "matrix_lds"), ("planned", "matrix")])
@pytest.mark.parametrize("mark,chunk", EDGES)
def test_one_key_stands_out(where, kernel, mark, chunk):
    """The last query points at ONE earlier key (the first, the last and the first of a page, the first of its
    own chunk and the last of the one before): its score stands out, so the result is that key's value where the
    mask shows it, and something else where not."""
    from transformer_amd import kernels as K
    from transformer_amd.kernels import PAGE
    dtype = "float32" if kernel == "vector32" else "bfloat16"
    H, G, dh, T = 4, 2, 32, 300
    rng = np.random.default_rng(mark)
    q, k = 0.05 * rng.standard_normal((T, H * dh)), 0.3 * rng.standard_normal((T, G * dh))
    v = rng.standard_normal((T, G * dh))
    k.reshape(T, G, dh)[mark, :, 0] = 5.0
    q.reshape(T, H, dh)[T - 1, :, 0] = 3.0
    rows = _bf(np.concatenate([q, k, v], 1), dtype)
    pages = np.array([4, 1, 3, 0, 5])
    kc = torch.full((6, G, PAGE, dh), float("nan"), dtype=TD[dtype], device=DEV)
    vc = torch.full((6, G, dh, PAGE), float("nan"), dtype=TD[dtype], device=DEV)
    nq = 130 if where == "prompt" else 1
    for p in (np.arange(0, T - nq), np.arange(T - nq, T)):
        proj = _t(rows[p], TD[dtype])
        dest = _t(pages[p // PAGE] * PAGE + p % PAGE, torch.int32)
        K.qk_rotate_store(proj, H, G, dh, dh, dest=dest, kcache=kc, vcache=vc)
    o = torch.empty(nq, H * dh, dtype=TD[dtype], device=DEV)
    args = (proj, o, kc, vc, _t([pages], torch.int32), _t([0, nq], torch.int32), _t([T - nq], torch.int32))
    opts = dict(softcap=20.0, chunk=chunk)
    if kernel.startswith("vector"):
        K.attention_sink(*args, nq, H, G, dh, dh, 1.0, **opts)
    elif where == "prompt":
        K.attention_rows_sink(*args, nq, H, G, dh, 1.0, through_lds=int(kernel == "matrix_lds"), **opts)
    else:
        plan = {}
        if where == "planned":
            u, s = K.plan_key_units([T], 7, tables=[pages], chunk=chunk)
            plan = dict(units=_t(u, torch.int32), seq_units=_t(s, torch.int32))
        K.attention_keys_sink(*args, T, H, G, dh, 1.0, **opts, **plan)
    marked = np.repeat(rows[mark, (H + G) * dh:].reshape(G, dh), H // G, axis=0).reshape(-1)
    err = np.abs(_np(o[-1]) - marked).max()
    if bool(P.same_chunk(T, chunk)[T - 1, mark]):
        assert err < (0.02 if dtype == "float32" else 4e-2)
    else:
        assert err > 0.5


@pytest.mark.parametrize("geom", [(8, 2, 128, 100), (4, 4, 32, 64), (16, 4, 64, 129), (2, 1, 96, 300), (6, 1, 160, 1), (64, 2, 64, 200),
                                  (5, 5, 32, 65), (8, 1, 256, 150)])
def test_chunks_on_matrix_cores(geom):
    """Prompts through the kernel that reads pages directly and the one that shares them through LDS, single tokens
    planned with and without the chunks, against each other's plain result over 700 tokens."""
    from transformer_amd import kernels as K
    from transformer_amd.kernels import PAGE
    H, G, dh, chunk = geom
    rng = np.random.default_rng(H * 7 + dh)
    T, scale, cap = 700, 2.0 * dh ** -0.5, 8.0
    rows = _bf(rng.standard_normal((T, (H + 2 * G) * dh)) * 1.3)
    q, k, v = (rows[:, a:b].reshape(T, -1, dh) for a, b in ((0, H * dh), (H * dh, (H + G) * dh), ((H + G) * dh, (H + 2 * G) * dh)))
    see, want = P.same_chunk(T, chunk), np.zeros((T, H, dh))
    for a in range(H):
        g = a // (H // G)
        want[:, a] = P.softmax_rows(P.cap(q[:, a] @ k[:, g].T * scale, cap), see) @ v[:, g]
    want = want.reshape(T, H * dh)
    kc = torch.full((12, G, PAGE, dh), float("nan"), dtype=torch.bfloat16, device=DEV)
    vc = torch.full((12, G, dh, PAGE), float("nan"), dtype=torch.bfloat16, device=DEV)
    pages = np.array([7, 2, 5, 11, 0, 9, 4, 1, 3, 10, 8, 0])
    got, at = [], 0
    for n, how in ((70, 0), (300, 1), (1, "planned"), (1, None), (28, 0), (1, "planned"), (199, 1), (99, 1), (1, "planned")):
        p = np.arange(at, at + n)
        qkv = _t(rows[p], torch.bfloat16)
        K.qk_rotate_store(qkv, H, G, dh, dh, dest=_t(pages[p // PAGE] * PAGE + p % PAGE, torch.int32), kcache=kc, vcache=vc)
        o = torch.empty(n, H * dh, dtype=torch.bfloat16, device=DEV)
        args = (qkv, o, kc, vc, _t([pages], torch.int32), _t([0, n], torch.int32), _t([at], torch.int32))
        opts = dict(softcap=cap, chunk=chunk)
        if how in (0, 1):
            K.attention_rows_sink(*args, n, H, G, dh, scale, through_lds=how if dh <= 192 else 0, **opts)
        elif not K.keys_sink_fits(H, G, dh):
            K.attention_rows_sink(*args, n, H, G, dh, scale, **opts)
        else:
            plan = {}
            if how == "planned":
                u, s = K.plan_key_units([at + 1], 7, tables=[pages], chunk=chunk)
                plan = dict(units=_t(u, torch.int32), seq_units=_t(s, torch.int32))
            K.attention_keys_sink(*args, at + 1, H, G, dh, scale, **opts, **plan)
        got.append(_np(o))
        at += n
    _close(np.concatenate(got), want, "bfloat16", scale=1.5)


def _memory_case(geom, rng, lens, spread=3.0):
    H, dk, dv, cap = geom
    d = 40
    shapes = {"q": (H * dk, d), "k": (H * dk, d), "v": (H * dv, d), "g": (H * dv, d), "i": (H, d), "f": (H, d), "o": (d, H * dv)}
    w = {n: _bf((spread if n in "if" else 1.0) * rng.standard_normal(s) / np.sqrt(s[-1])) for n, s in shapes.items()}
    w["i.b"], w["f.b"], w["norm"] = _f32(rng.uniform(-3, 3, H)), _f32(rng.uniform(-1, 6, H)), _f32(1 + 0.2 * rng.standard_normal(H * dv))
    return w, {"heads": H, "dim": dk, "vdim": dv, "gate_cap": cap}, [_bf(rng.standard_normal((L, d))) for L in lens]


def _memory_part(w, m, dtype):
    from transformer_amd.config.spec import MatrixMemorySpec
    from transformer_amd.parts.base import build_part
    part = build_part(MatrixMemorySpec(hidden=w["q"].shape[1], num_heads=m["heads"], key_dim=m["dim"], value_dim=m["vdim"],
                                       gate_cap=m["gate_cap"], eps=1e-5), TD[dtype], DEV)
    part.bind({"in.weight": _t(np.concatenate([w[n] for n in ("q", "k", "v", "g", "i", "f")]), TD[dtype]), "i.bias": _t(w["i.b"]),
               "f.bias": _t(w["f.b"]), "norm.weight": _t(w["norm"]), "out.weight": _t(w["o"], TD[dtype])})
    return part


CUTS = [(37, 1, 18), (1, 1, 1), (2, 2, 2), (2, 2, 2), (1, 1, 1), (18, 1, 16)]
MEMORY_GEOMS = [(2, 32, 64, 10.0), (3, 20, 12, 4.0), (1, 1, 1, 5.0), (5, 33, 7, 15.0), (2, 6, 66, 2.0), (4, 128, 128, 12.0), (1, 64, 200, 8.0),
                (2, 256, 512, 15.0), (3, 16, 100, 7.0), (1, 300, 40, 9.0), (2, 40, 127, 3.0), (1, 100, 1202, 6.0), (1, 1000, 1111, 5.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", MEMORY_GEOMS)
def test_matrix_memory_part_over_cuts(dtype, geom):
    """The whole mixer over three sequences of unequal lengths in slots that held something else, in cuts of many,
    one, two and two tokens: gates, running maximum, state, normaliser, the readout's denominator, norm and gate,
    prompts through the walking kernel and single tokens through the fused one (where the heads fit it)."""
    rng = np.random.default_rng(geom[1] * 10 + geom[2])
    lens = [61, 8, 40]
    w, m, hs = _memory_case(geom, rng, lens)
    got, _, _ = _run_part(_memory_part(w, m, dtype), hs, CUTS, dtype)
    for g, h in zip(got, hs):
        _close(g, P.mlstm(h, w, "", m, 1e-5), dtype, scale=6.0)


@pytest.mark.parametrize("lens", [[1, 64, 65, 200], [257, 1024, 1], [1025, 2100]])
def test_memory_gates_alone(lens):
    """The gates' scan over one wave, four and sixteen (several turns of them), from a maximum that is not zero,
    with input gates near the cap, forget gates near zero and one: every maximum, and the weights' products with
    what the maximum has divided out."""
    from transformer_amd import kernels as K
    rng = np.random.default_rng(lens[0])
    H, nt, cap = 5, sum(lens), 9.0
    raw = 6.0 * rng.standard_normal((nt, 2 * H + 3)).astype(np.float32)
    raw[::7] *= 5.0
    bi, bf = rng.uniform(-2, 2, H), np.array([-4.0, 0.0, 3.0, 9.0, 30.0])
    m0 = rng.uniform(-3, 3, (len(lens), H)).astype(np.float32)
    slots = [3, 0, 2, 1][:len(lens)]
    state = torch.full((5, H), 7.0, device=DEV)
    for s, a in zip(slots, m0):
        state[s] = _t(a)
    cu = np.concatenate([[0], np.cumsum(lens)])
    keep, write, floor = (torch.full((nt, H), float("nan"), device=DEV) for _ in range(3))
    K.memory_gates(_t(raw), 1, H + 2, _t(bi), _t(bf), cap, state, _t(cu, torch.int32), _t(slots, torch.int32), max(lens), keep, write, floor)
    i = P.cap(raw[:, 1:1 + H] + np.float32(bi), cap)
    f = -P.softplus(-P.cap(raw[:, H + 2:2 * H + 2] + np.float32(bf), cap))
    for b in range(len(lens)):
        m = m0[b].astype(np.float64)
        for t in range(cu[b], cu[b + 1]):
            new = np.maximum(f[t] + m, i[t])
            np.testing.assert_allclose(_np(floor[t]), np.exp(-new), rtol=3e-5)
            np.testing.assert_allclose(_np(write[t]), np.exp(i[t] - new), rtol=3e-5, atol=1e-30)
            np.testing.assert_allclose(_np(keep[t]), np.exp(f[t] + m - new), rtol=5e-5, atol=1e-30)
            m = new
        np.testing.assert_allclose(_np(state[slots[b]]), m, atol=3e-5)
    assert float(state[4].min()) == 7.0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lanes", [0, 16, 32])
@pytest.mark.parametrize("geom", [(3, 32, 16), (2, 128, 40), (2, 47, 5), (2, 192, 33), (1, 256, 70), (8, 64, 64), (1, 300, 9), (1, 1000, 6), (2, 3, 15)])
def test_matrix_memory_recurrence_alone(geom, lanes, dtype):
    """The recurrence's kernel on weights of its own (keep down to 0 and up to 1), rows whose heads do and do not
    start on whole pieces, sequences that end inside, at and behind the edge of a chunk of tokens."""
    from transformer_amd import kernels as K
    H, dk, dv = geom
    rng = np.random.default_rng(dk)
    lens = [1, 16, 17, 50, 3]
    nt, n = sum(lens), 2 * H * dk + H * dv
    rows = _bf(rng.standard_normal((nt, n + 5)), dtype)
    keep, write = rng.uniform(0.5, 1.0, (nt, H)), rng.uniform(0, 1, (nt, H))
    keep[::3], keep[::5], write[::4] = 1.0, 0.0, 0.0
    S0, n0 = rng.standard_normal((len(lens), H, dk, dv)), rng.standard_normal((len(lens), H, dk))
    state, norm = torch.zeros((7, H, dk, dv), device=DEV), torch.zeros((7, H, dk), device=DEV)
    slots = [4, 0, 5, 2, 6]
    for s, a, c in zip(slots, S0, n0):
        state[s], norm[s] = _t(a), _t(c)
    cu = np.concatenate([[0], np.cumsum(lens)])
    o, den = torch.full((nt, H, dv), float("nan"), device=DEV), torch.full((nt, H), float("nan"), device=DEV)
    off, scale = (1 if H == 2 else 4), dk ** -0.5
    K.memory_recurrent(_t(rows, TD[dtype]), off, off + H * dk, off + 2 * H * dk, scale, _t(keep), _t(write), state, norm,
                       _t(cu, torch.int32), _t(slots, torch.int32), o, den, lanes=lanes)
    q, k, v = (rows[:, a:b].reshape(nt, H, -1) for a, b in ((off, off + H * dk), (off + H * dk, off + 2 * H * dk), (off + 2 * H * dk, off + n)))
    for i in range(len(lens)):
        S, nn = S0[i], n0[i]
        for t in range(cu[i], cu[i + 1]):
            S = keep[t][:, None, None] * S + write[t][:, None, None] * k[t][:, :, None] * v[t][:, None, :]
            nn = keep[t][:, None] * nn + write[t][:, None] * k[t]
            np.testing.assert_allclose(_np(o[t]), scale * np.einsum("hkv,hk->hv", S, q[t]), atol=1e-3)
            np.testing.assert_allclose(_np(den[t]), scale * (nn * q[t]).sum(-1), atol=1e-3)
        np.testing.assert_allclose(_np(state[slots[i]]), S, atol=1e-3)
        np.testing.assert_allclose(_np(norm[slots[i]]), nn, atol=1e-3)
    assert float(state[[1, 3]].abs().max()) == 0.0 and float(norm[[1, 3]].abs().max()) == 0.0


@pytest.mark.parametrize("where", ["prompt", "decode"])
def test_a_far_token_in_the_matrix_memory(where):
    """A token 497 steps back wrote its value under a key that nobody touched since: head 0, which never forgets,
    gives it back, head 1 has forgotten it, and in head 2 it weighs as much as its input gate said."""
    H, dk, dv, T, far = 3, 8, 5, 500, 2
    rng = np.random.default_rng(5)
    d = dk * 2 + H * dv + 1
    w, m, _ = _memory_case((H, dk, dv, 15.0), rng, [1])
    for n, c in (("q", 0), ("k", dk)):
        w[n] = np.zeros((H * dk, d)); w[n].reshape(H, dk, d)[:, :, c:c + dk] = np.eye(dk)
    w["v"] = np.zeros((H * dv, d)); w["v"][:, 2 * dk:2 * dk + H * dv] = np.eye(H * dv)
    w["i"], w["f"], w["g"] = np.zeros((H, d)), np.zeros((H, d)), np.zeros((H * dv, d))
    w["i"][2, -1] = 1.0                                       # head 2: the far token writes with exp(4)
    w["i.b"], w["f.b"] = np.array([0.0, 0.0, -2.0]), np.array([60.0, -1.0, 60.0])
    w["norm"], w["o"] = np.ones(H * dv), np.eye(d, H * dv)
    h = np.zeros((T, d))
    h[:, dk + 1], h[:, 1] = 3.0, 3.0
    h[far, dk + 1], h[far, dk], h[far, -1] = 0.0, 3.0, 6.0
    h[T - 1, 1], h[T - 1, 0] = 0.0, 3.0
    h[:, 2 * dk:2 * dk + H * dv] = 0.01 * rng.standard_normal((T, H * dv))
    h[far, 2 * dk:2 * dk + H * dv] = 4.0
    part = _memory_part(w, m, "float32")
    nq = 1 if where == "decode" else 33
    got, cache, slots = _run_part(part, [h], [(T - nq,), (nq,)], "float32")
    want = P.mlstm(h, w, "", m, 1e-5)
    np.testing.assert_allclose(got[0][-1], want[-1], atol=2e-3)
    S, n, mx = (_np(cache.layer_state(i)[slots[0]]) for i in range(3))
    np.testing.assert_allclose(S[0, 0], 12.0, rtol=1e-3)                    # 3 * 4, kept
    assert np.abs(S[1, 0]).max() < 1e-20 and abs(n[1, 0]) < 1e-20           # sigmoid(-1)^497
    np.testing.assert_allclose(S[2, 0] * np.exp(mx[2]), 12.0 * np.exp(P.cap(4.0, 15.0)), rtol=1e-3)


def _delta_case(geom, rng, lens):
    H, G, dk, dv, taps = geom
    d = 40
    shapes = {"q": (G * dk, d), "k": (G * dk, d), "v": (H * dv, d), "g": (H * dv, d), "a": (H, d), "b": (H, d), "o": (d, H * dv)}
    w = {n: _bf(rng.standard_normal(s) / np.sqrt(s[-1])) for n, s in shapes.items()}
    for n in "qkv":
        w[n + ".conv"] = _bf(rng.standard_normal((shapes[n][0], taps)))
    w["A_log"], w["dt_bias"], w["norm"] = _f32(rng.uniform(-1, 1, H)), _f32(rng.uniform(-5, 0, H)), _f32(1 + 0.2 * rng.standard_normal(dv))
    return w, {"heads": H, "kv_heads": G, "dim": dk, "vdim": dv, "conv": taps}, [_bf(rng.standard_normal((L, d))) for L in lens]


def _delta_part(w, m, dtype):
    from transformer_amd.config.spec import GatedDeltaSpec
    from transformer_amd.parts.base import build_part
    part = build_part(GatedDeltaSpec(hidden=40, num_heads=m["heads"], num_kv_heads=m["kv_heads"], key_dim=m["dim"],
                                     value_dim=m["vdim"], taps=m["conv"], decay_rank=None, gate_rank=None, eps=1e-5,
                                     gate_activation="silu"), TD[dtype], DEV)
    part.bind({"in.weight": _t(np.concatenate([w[n] for n in ("q", "k", "v", "g", "a", "b")]), TD[dtype]),
               "conv.weight": _t(np.concatenate([w[n + ".conv"] for n in "qkv"])), "dt_bias": _t(w["dt_bias"]), "A_log": _t(w["A_log"]),
               "norm.weight": _t(w["norm"]), "out.weight": _t(w["o"], TD[dtype])})
    return part


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", [(2, 2, 32, 64, 3), (6, 3, 24, 12, 4), (1, 1, 64, 8, 1), (3, 1, 33, 7, 9), (2, 1, 6, 66, 2), (4, 2, 128, 128, 4),
                                  (2, 1, 160, 40, 2), (2, 2, 250, 20, 3), (1, 1, 200, 256, 4), (3, 3, 16, 100, 4)])
def test_head_delta_part_over_cuts(dtype, geom):
    rng = np.random.default_rng(geom[2] * 10 + geom[3])
    w, m, hs = _delta_case(geom, rng, [61, 8, 40])
    got, _, _ = _run_part(_delta_part(w, m, dtype), hs, CUTS, dtype)
    for g, h in zip(got, hs):
        _close(g, P.head_delta(h, w, "", m, 1e-5), dtype, scale=3.0)


@pytest.mark.parametrize("lanes", [0, 16, 32])
@pytest.mark.parametrize("geom", [(3, 3, 32, 16), (4, 2, 128, 40), (2, 1, 47, 5), (2, 2, 192, 33), (1, 1, 256, 70), (16, 4, 64, 64)])
def test_head_delta_recurrence_alone(geom, lanes):
    """The recurrence's kernel with one decay per head (0 and 1 among them), sequences that end inside and at the
    edge of a chunk of tokens."""
    from transformer_amd import kernels as K
    H, G, dk, dv = geom
    rng = np.random.default_rng(dk)
    lens = [1, 16, 17, 50]
    nt = sum(lens)
    q, k = 0.3 * rng.standard_normal((nt, G, dk)), rng.standard_normal((nt, G, dk)) / np.sqrt(dk)
    g, b = rng.uniform(0.5, 1.0, (nt, H)), rng.uniform(0, 1, (nt, H))
    g[::3], g[::5] = 1.0, 0.0
    b[::7], b[1::7] = 0.0, 1.0
    v = rng.standard_normal((nt, H, dv))
    S0 = rng.standard_normal((len(lens), H, dk, dv))
    state = torch.zeros((6, H, dk, dv), device=DEV)
    slots = [4, 0, 5, 2]
    for s, a in zip(slots, S0):
        state[s] = _t(a)
    cu = np.concatenate([[0], np.cumsum(lens)])
    o = torch.full((nt, H, dv), float("nan"), device=DEV)
    f = lambda a: _t(np.asarray(a, dtype=np.float32))
    K.delta_recurrent(f(q), f(k), f(g), f(v.reshape(nt, -1)), f(b), f((q * k).sum(-1)), state, _t(cu, torch.int32),
                      _t(slots, torch.int32), o, lanes=lanes)
    rep = lambda a: np.repeat(a, H // G, axis=1)
    for i, n in enumerate(lens):
        r = slice(cu[i], cu[i + 1])
        want, S = P.delta_rule(rep(q[r]), rep(k[r]), v[r], g[r], b[r], S0[i])
        np.testing.assert_allclose(_np(o[r]), want, atol=3e-4)
        np.testing.assert_allclose(_np(state[slots[i]]), S, atol=3e-4)
    assert float(state[1].abs().max()) == 0.0 and float(state[3].abs().max()) == 0.0


@pytest.mark.parametrize("ranks", [(None, 5), (6, None)])
def test_delta_rule_with_one_of_its_inputs_low_rank(ranks):
    """The step's kernel and the prompt's agree where the decay is per head and the gate a low-rank product, and the
    other way round."""
    from transformer_amd.config.spec import GatedDeltaSpec
    from transformer_amd.parts.base import build_part
    ra, rg = ranks
    H, G, dk, dv, d = 4, 2, 24, 20, 40
    rng = np.random.default_rng(3)
    part = build_part(GatedDeltaSpec(hidden=d, num_heads=H, num_kv_heads=G, key_dim=dk, value_dim=dv, taps=3, decay_rank=ra,
                                     gate_rank=rg, eps=1e-5, gate_activation="silu"), torch.float32, DEV)
    part.bind({n: _t(rng.standard_normal(p.shape) / np.sqrt(p.shape[-1])) for n, p in part.params().items()})
    h = _f32(rng.standard_normal((40, d)))
    whole, _, _ = _run_part(part, [h], [(40,)], "float32")
    single, _, _ = _run_part(part, [h], [(1,)] * 40, "float32")
    np.testing.assert_allclose(single[0], whole[0], atol=1e-4)


MOE_GEOMS = [(6, 2, 20, 40, 3, 1.7), (5, 5, 17, 33, 0, 1.0), (3, 5, 24, 64, 2, 0.6), (1, 1, 30, 48, 0, 2.0), (1, 2, 8, 72, 4, 1.1),
             (12, 3, 80, 264, 4, 2.0), (64, 6, 48, 128, 8, 1.5)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("geom", MOE_GEOMS)
def test_routed_part_with_identity_experts(dtype, geom):
    """Scores over experts and identity experts, a correction that changes the choice and not the weights, weights
    that are not renormalised, identity experts beside the others, alone, and not at all."""
    from transformer_amd.config.spec import RoutedMLPSpec
    from transformer_amd.parts.base import build_part
    from transformer_amd.parts.linear import Workspace
    E, top, ff, d, identity, factor = geom
    rng = np.random.default_rng(E + top + ff)
    mlp = {"router": {"experts": E, "top": top, "identity": identity, "scale": factor}, "expert": {"ff": ff}}
    w = {"router": _bf(3.0 * rng.standard_normal((E + identity, d)) / np.sqrt(d), dtype),
         "correction": _f32(0.2 * rng.standard_normal(E + identity))}
    for e in range(E):
        for n, s in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff))):
            w[f"e{e}.{n}"] = _bf(rng.standard_normal(s) / np.sqrt(s[-1]), dtype)
    part = build_part(RoutedMLPSpec(hidden=d, experts=E, top=top, intermediate=ff, activation="silu", score="softmax",
                                    weight_on="output", form="glu", identity=identity, correction=True, factor=factor), TD[dtype], DEV)
    mat = lambda a: _t(a, TD[dtype])

    class Ctx:
        ws, dump = Workspace(DEV), None
    for what in ("drawn", "all identity", "no identity"):
        if what != "drawn" and not identity:
            continue
        c = w["correction"].copy()
        c[E:] += {"drawn": 0.0, "all identity": 50.0, "no identity": -50.0}[what]
        if what == "no identity" and top > E or what == "all identity" and top > identity:
            continue
        part.bind({"router.weight": mat(w["router"]), "router.correction": _t(c),
                   "experts.gate_up.weight": mat(np.concatenate([w[f"e{e}.{n}"] for e in range(E) for n in ("gate", "up")])),
                   "experts.down.weight": mat(np.concatenate([w[f"e{e}.down"] for e in range(E)]))})
        for nt in (1, 9, 150):
            h = _bf(rng.standard_normal((nt, d)), dtype)
            chosen = {}
            Ctx.dump = lambda name, t: chosen.__setitem__(name, t.cpu().numpy().astype(np.int64))
            delta, bias = part.run(mat(h), Ctx)
            assert bias is None
            if what == "all identity":
                assert (chosen["experts"] >= E).all()
            want = P.moe(h, {**w, "correction": c}, "", mlp, forced=None if dtype == "float32" else chosen["experts"], slack=0.02)
            _close(_np(delta), want, dtype, f"{what} {nt} rows")


@pytest.mark.parametrize("dtype", DTYPES)
def test_parallel_mixer_over_cuts(dtype):
    """Both sides and the mean of their normed results, as the block runs them."""
    from transformer_amd.config.linonex import LinonexConfig
    from transformer_amd.parts.base import build_part
    from transformer_amd.architectures.linonex import linonex_weight_sources
    cfg_dict = {**U.CFG_A, "layers": [U.CFG_A["layers"][1]], "loop": None}
    cfg = LinonexConfig.from_dict(cfg_dict)
    w = P.random_weights(cfg_dict, 9)
    part = build_part(cfg.model_spec().blocks[0].mixer, TD[dtype], DEV)
    src = linonex_weight_sources(cfg, "safetensors")
    params = part.all_params("blocks.0.mixer.")
    part.bind_all({n: _t(np.concatenate([w[p.name] for p in src[n].options[0]]), TD[dtype] if params[n].role == "matrix" else torch.float32)
                   for n in params}, "blocks.0.mixer.")
    rng = np.random.default_rng(4)
    hs = [_bf(rng.standard_normal((L, cfg.width))) for L in (61, 8, 40)]
    got, _, _ = _run_part(part, hs, CUTS, dtype)
    for g, h in zip(got, hs):
        _close(g, P.parallel_mixer(h, w, "l0.mix.", cfg_dict["layers"][0]["mixer"], cfg.eps), dtype, scale=3.0)


# ----------------------------------------------------------------------------- the engine
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_layers_and_whole_prompt(name, dtype):
    from transformer_amd import Entry
    model, toks = U.engine(name, dtype), U.tokens(name, 140, 1)
    dumps = {}
    model.dump = lambda n, t: dumps.__setitem__(n, t.detach().float().cpu().numpy().copy())
    try:
        cache = model.new_cache(256)
        got = model.step(cache, [Entry(cache.alloc_slot(), toks, list(range(len(toks))))]).cpu().numpy()
    finally:
        model.dump = None
    routes = None if dtype == "float32" else {int(n.split(".")[1]): a.astype(np.int64) for n, a in dumps.items() if n.endswith(".experts")}
    layers = []
    want = U.plain(name, dtype).forward(toks, layers, routes=routes, slack=U.SLACK)
    assert len(layers) == len(model.spec.schedule)
    for i, l in enumerate(layers):
        d = np.abs(dumps[f"run.{i}"] - l)
        if dtype == "float32":
            assert d.max() < 1e-4 * max(1.0, np.abs(l).max()), f"layer run {i}"
        else:
            assert np.quantile(d, 0.99) < 0.06 * max(1.0, np.sqrt((l ** 2).mean())), f"layer run {i}"
    U.check_against_plain(name, dtype, None, toks, got, routes)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,edit", [("A", None), ("B", None), ("D", None), ("A", "sharp"), ("D", "sharp")])
def test_cuts_agree_with_plain(name, edit, dtype):
    """Whole, portions down to two tokens, and every token alone: all against the plain model."""
    model, toks = U.engine(name, dtype, edit), U.tokens(name, 150, 2)
    cache = model.new_cache(512, max_slots=3)
    for cuts in ([150], [2, 2, 61, 3, 64, 17], [130], []):
        slot = cache.alloc_slot()
        got, routes = U.run_cuts(model, cache, slot, toks, cuts, routes=True)
        cache.free_slot(slot)                      # the next cut takes the same slot and pages
        U.check_against_plain(name, dtype, edit, toks, got, routes, f"cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_prompt_in_portions_over_pages_and_chunks(dtype):
    """400 tokens with peaked softmax and long memories: portions end at and around the borders of pages, of the
    chunks and of the recurrences' runs; pages of chunks left behind are given back meanwhile."""
    name, edit = "A", "sharp"
    model, toks = U.engine(name, dtype, edit), U.tokens(name, 400, 7)
    cache = model.new_cache(512, max_slots=1)
    for cuts in ([400], [257, 63, 65, 15], [64, 256, 33, 31, 16], [255, 129, 8, 7, 1], [50, 50, 40, 10, 90, 90, 70], [49, 2, 38, 2, 179, 2]):
        slot = cache.alloc_slot()
        got, routes = U.run_cuts(model, cache, slot, toks, cuts, routes=True)
        for g, need in enumerate(cache.kv_groups):
            gone = [p < 0 for p in cache.pool.pages(slot, g)]
            n = (400 // need.chunk * need.chunk) // 64
            assert gone == [True] * n + [False] * (len(gone) - n)
        cache.free_slot(slot)
        U.check_against_plain(name, dtype, edit, toks, got, routes, f"cuts {cuts}")
        cache.pool.check()


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batch_then_decoding_in_used_slots(dtype):
    """The second batch lives in slots and pages that a first one left dirty; a sequence leaves early and its slot
    is taken again; another joins while the rest decode."""
    from transformer_amd import Entry
    name = "A"
    model = U.engine(name, dtype)
    cache = model.new_cache(1024, max_slots=4)
    old = [cache.alloc_slot() for _ in range(4)]
    model.step(cache, [Entry(s, U.tokens(name, 100 + 7 * s, 50 + s), [0]) for s in old])
    for s in old:
        cache.free_slot(s)
    lens = [1, 70, 131, 2]
    seqs = [U.tokens(name, n + 45, 10 + i) for i, n in enumerate(lens)]
    slots = [cache.alloc_slot() for _ in seqs]
    late = U.tokens(name, 33, 99)
    got, rows, tail = [[] for _ in seqs], [[] for _ in seqs], []
    with U.Routes(model) as rec:
        def step(entries):
            out = model.step(cache, entries).cpu().numpy().copy()
            rec.next_step()
            return out
        lg = step([Entry(sl, s[:n], list(range(n))) for sl, s, n in zip(slots, seqs, lens)])
        at = 0
        for i, n in enumerate(lens):
            got[i].append(lg[at:at + n])
            rows[i].append(slice(at, at + n))
            at += n
        live = list(range(len(seqs)))
        for t in range(40):
            if t == 25:
                cache.free_slot(slots[1])
                live.remove(1)
                slots[1] = cache.alloc_slot()
            lg = step([Entry(slots[i], [seqs[i][lens[i] + t]], [0]) for i in live])
            for i in range(len(seqs)):
                rows[i].append(slice(live.index(i), live.index(i) + 1) if i in live else None)
            for j, i in enumerate(live):
                got[i].append(lg[j:j + 1])
        # the slot that came back: a prompt beside single tokens and a portion of two
        lg = step([Entry(slots[0], [seqs[0][lens[0] + 40]], [0]), Entry(slots[1], late[:31], list(range(31))),
                   Entry(slots[2], seqs[2][lens[2] + 40:lens[2] + 42], [0, 1])])
        got[0].append(lg[:1]); rows[0].append(slice(0, 1))
        got[2].append(lg[32:34]); rows[2].append(slice(32, 34))
        last = step([Entry(slots[1], late[31:], [0, 1])])
        late_rows = [None] * 41 + [slice(1, 32), slice(0, 2)]
    U.check_against_plain(name, dtype, None, late, np.concatenate([lg[1:32], last]), rec.of_rows(late_rows), "the late sequence")
    for i in range(len(seqs)):
        U.check_against_plain(name, dtype, None, seqs[i], np.concatenate(got[i]), rec.of_rows(rows[i]), f"sequence {i}")
    cache.pool.check()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "D"])
def test_recorded_steps_match_eager_steps(name, dtype):
    from transformer_amd import Entry
    model = U.engine(name, dtype)
    seqs = [U.tokens(name, 60, 20 + i) for i in range(3)]
    outs = []
    for graphs in (True, False):
        model.use_graphs = graphs
        try:
            cache = model.new_cache(512, max_slots=4)
            slots = [cache.alloc_slot() for _ in seqs]
            rows = []
            for t in range(60):
                lg = model.step(cache, [Entry(sl, [s[t]], [0]) for sl, s in zip(slots, seqs)])
                rows.append(lg.cpu().numpy().copy())
            outs.append(np.stack(rows))
            assert bool(cache.graphs) == graphs and not cache.graphs_failed
        finally:
            model.use_graphs = True
    assert np.abs(outs[0] - outs[1]).max() < (1e-5 if dtype == "float32" else 3e-2) * np.abs(outs[1]).max()
    if dtype == "float32":
        want = np.stack([U.plain_logits(name, dtype, None, tuple(s)) for s in seqs], 1)
        assert U.row_error(outs[0], want).max() < U.TOL[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_wide_model_in_three_cuts(dtype):
    """Width 512: heads of 128 on the matrix cores, memory heads of 64 x 96 and 128 x 160, delta heads of 64 x 96,
    products of 17 to 64 rows, prompts through the library and single tokens through the few-rows products; 330
    tokens pass the borders of pages and chunks."""
    name = "C"
    model, toks = U.engine(name, dtype), U.tokens(name, 330, 3)
    cache = model.new_cache(512, max_slots=2)
    for cuts in ([330], [100, 40, 70, 20, 9], [310]):
        slot = cache.alloc_slot()
        got, routes = U.run_cuts(model, cache, slot, toks, cuts, routes=True)
        cache.free_slot(slot)
        U.check_against_plain(name, dtype, None, toks, got, routes, f"cuts {cuts}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_over_page_and_chunk_borders(dtype):
    name, edit = "A", "sharp"
    model, toks = U.engine(name, dtype, edit), U.tokens(name, 330, 4)
    cache = model.new_cache(512, max_slots=1)
    got, routes = U.run_cuts(model, cache, cache.alloc_slot(), toks, [5], routes=True)     # 325 single tokens
    U.check_against_plain(name, dtype, edit, toks, got, routes)


def test_positions_end_where_the_table_does():
    from transformer_amd import Entry
    from transformer_amd.engine.batch import PositionPastLimit
    name = "D"
    model = U.engine(name, "float32")
    toks = U.tokens(name, 351, 8)
    cache = model.new_cache(512)
    slot = cache.alloc_slot()
    with pytest.raises(PositionPastLimit):
        model.step(cache, [Entry(slot, toks, [0])])
    got = model.step(cache, [Entry(slot, toks[:350], [349])]).cpu().numpy()
    assert U.row_error(got, U.plain_logits(name, "float32", None, tuple(toks[:350]))[349:]).max() < U.TOL["float32"]
    with pytest.raises(PositionPastLimit):
        model.step(cache, [Entry(slot, toks[350:], [0])])


def test_greedy_generation_through_the_entry_point():
    import transformer_amd as ta
    from transformer_amd.engine.generate import generate
    name, dtype = "A", "float32"
    model, plain = U.engine(name, dtype), U.plain(name, dtype)
    prompts = [U.tokens(name, n, 30 + n) for n in (5, 1, 23)]
    res = generate(model, prompts, max_new_tokens=12, sample_args=ta.SampleArgs(), stop_ids=())
    for p, out in zip(prompts, res.tokens):
        assert len(out) == 12
        seq = list(p)
        for t in out:                         # the engine's choice is the plain model's best, or ties with it
            lg = plain.forward(seq)[-1]
            assert lg.max() - lg[t] < 1e-3
            seq.append(t)
    again = generate(model, prompts, max_new_tokens=12, sample_args=ta.SampleArgs(), stop_ids=())
    assert again.tokens == res.tokens


def test_replayer_and_command_line():
    name, dtype = "D", "float32"
    folder = U.folder(name, dtype)
    toks = U.tokens(name, 40, 5)
    want = U.plain_logits(name, dtype, None, tuple(toks))
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    import tempfile
    with tempfile.TemporaryDirectory() as out:
        lines = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:30], "want": [0, 29]},
                                         {"id": "b", "tokens": toks[:1], "want": [0]}], "end": ["b"]}]
        lines += [{"step": 1 + i, "entries": [{"id": "a", "tokens": [toks[30 + i]], "want": [0]}],
                   "end": ["a"] if i == 9 else []} for i in range(10)]
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype",
                            dtype, "--out", out, "--max-tokens", "128"],
                           input="\n".join(json.dumps(l) for l in lines) + "\n", capture_output=True, text=True,
                           timeout=600)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(11)]
        first = np.fromfile(os.path.join(out, "0.f32"), dtype="<f4").reshape(3, -1)
        assert U.row_error(first, want[[0, 29, 0]]).max() < U.TOL[dtype]
        last = np.fromfile(os.path.join(out, "10.f32"), dtype="<f4").reshape(1, -1)
        assert U.row_error(last, want[39:40]).max() < U.TOL[dtype]
    r = subprocess.run([sys.executable, "-m", "transformer_amd", "generate", "--model", folder, "--dtype", dtype,
                        "--prompt", ",".join(map(str, toks[:6])), "--max-steps", "5"],
                       capture_output=True, text=True, timeout=600, cwd=root)
    assert r.returncode == 0, r.stderr[-2000:]


def test_random_weights_and_save_round_trip():
    import tempfile
    import transformer_amd as ta
    from transformer_amd import Entry
    model = ta.random_model(U.CFG_A, seed=3, dtype="float32", architecture="Linonex")
    toks = U.tokens("A", 60, 6)
    cache = model.new_cache(128)
    a = model.step(cache, [Entry(cache.alloc_slot(), toks, [59])]).cpu().numpy().copy()
    with tempfile.TemporaryDirectory() as d:
        ta.save_model(model, d)
        want = P.PlainLinonex(d).forward(toks)[-1:]
        again = ta.load_model(d, "float32")
        cache = again.new_cache(128)
        b = again.step(cache, [Entry(cache.alloc_slot(), toks, [59])]).cpu().numpy()
    assert np.abs(a - b).max() < 1e-6 * max(1.0, np.abs(a).max())
    assert U.row_error(a, want).max() < U.TOL["float32"]


def _draw_config(case):
    """A random Linonex configuration: any order of the two layer types, every option present or absent, sizes that
    are odd, equal to one another, or 1, loops anywhere."""
    r = np.random.default_rng(case)
    pick = lambda *a: a[int(r.integers(0, len(a)))]
    layers = []
    for _ in range(int(r.integers(1, 5))):
        kind = int(r.integers(0, 4))
        mlp = None
        if kind == 1:
            E, I = int(pick(1, 3, 8)), int(pick(0, 1, 4))
            mlp = U._moe(E, int(r.integers(1, min(E + I, 4) + 1)), int(pick(8, 20, 33, 64)), I, float(pick(0.5, 1.0, 2.5)))
        elif kind:
            mlp = U._dense(int(pick(8, 20, 33, 64)))
        if r.integers(0, 2):
            layers.append(U._mem(int(pick(1, 2, 3, 4)), int(pick(1, 4, 9, 16, 32, 70)), int(pick(2, 6, 16, 33, 64, 130)),
                                 float(pick(2.0, 8.0, 15.0)), mlp))
        else:
            G, g = int(pick(1, 2, 3)), int(pick(1, 2, 3))
            dk = int(pick(4, 9, 16, 32, 64))
            left = U._left(G * int(pick(1, 2, 4)), G, dk, int(pick(3, 16, 32, 64)), int(pick(1, 2, 4)), float(pick(0.5, 1.0)) * dk ** -0.5,
                           pick(None, 1, 5, 63, 64, 65, 100), pick(None, 5.0, 30.0))
            layers.append(U._par(left, U._right(g * int(pick(1, 2, 3)), g, int(pick(4, 9, 16, 32, 70)), int(pick(2, 6, 16, 33, 64)),
                                                int(pick(1, 2, 3, 4))), mlp))
    n = len(layers)
    cfg = {"architecture": "Linonex", "vocab": int(pick(5, 97, 300, 1001)), "width": int(pick(40, 64, 66, 100, 136, 33, 257)),
           "max_positions": 200, "norm": {"eps": float(pick(1e-6, 1e-5, 1e-3))}, "layers": layers}
    if r.integers(0, 3):
        a = int(r.integers(0, n))
        cfg["loop"] = {"start": a, "stop": int(r.integers(a + 1, n + 1)), "times": int(pick(1, 2, 3))}
    lens = [int(x) for x in r.integers(1, 150, size=int(r.integers(1, 5)))]
    return cfg, lens, r


@pytest.mark.parametrize("first", [7000, 7006, 7012, 7018])
def test_random_configurations_against_the_plain_model(first):
    """A batch of unequal prompts in one step into poisoned pages, then eight single tokens each, every row, in
    float32 (recorded steps) and in bfloat16."""
    import contextlib
    import tempfile
    import transformer_amd as ta
    from gpu_util import poison
    for case in range(first, first + 6):
        cfg, lens, r = _draw_config(case)
        toks = [[int(t) for t in r.integers(0, cfg["vocab"], size=n + 8)] for n in lens]
        for dtype in DTYPES:
            with tempfile.TemporaryDirectory(prefix="li_rand_") as d:
                P.make_model_folder(d, cfg, case, storage=U.STORAGE[dtype])
                ref = P.PlainLinonex(d)
                model = ta.load_model(d, dtype, "cuda:0")
            cache = model.new_cache(64 * sum(-(-(n + 8) // 64) for n in lens), max_slots=len(lens))
            poison(cache)
            slots = [cache.alloc_slot() for _ in lens]
            what = f"case {case} {dtype} {json.dumps(cfg)} prompts {lens}"
            rec = U.Routes(model) if dtype == "bfloat16" else None
            got, rows, at = [[] for _ in lens], [[] for _ in lens], 0
            with rec if rec is not None else contextlib.nullcontext():
                lg = model.step(cache, [ta.Entry(s, t[:n], list(range(n))) for s, t, n in zip(slots, toks, lens)]).cpu().numpy().copy()
                for i, n in enumerate(lens):
                    got[i].append(lg[at:at + n])
                    rows[i].append(slice(at, at + n))
                    at += n
                for j in range(8):
                    if rec is not None:
                        rec.next_step()
                    lg = model.step(cache, [ta.Entry(s, [t[n + j]], [0]) for s, t, n in zip(slots, toks, lens)]).cpu().numpy().copy()
                    for i in range(len(lens)):
                        got[i].append(lg[i:i + 1])
                        rows[i].append(slice(i, i + 1))
            errs = []
            for i, t in enumerate(toks):
                want = ref.forward(t, routes=None if rec is None else rec.of_rows(rows[i]), slack=U.SLACK)
                errs += list(U.row_error(np.concatenate(got[i]), want))
            errs = np.asarray(errs)
            assert np.isfinite(errs).all(), what
            if dtype == "float32":
                assert errs.max() < U.TOL[dtype], (what, errs.max())
            else:
                # (a row now and then is badly conditioned: a norm of numbers near zero)
                assert np.median(errs) < 0.5 * U.TOL[dtype] and np.quantile(errs, 0.9) < 1.5 * U.TOL[dtype], (what, np.quantile(errs, [0.5, 0.9]))
            for s in slots:
                cache.free_slot(s)
            cache.pool.check()
