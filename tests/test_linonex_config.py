"""Linonex without a GPU: configuration keys, the layout it spells out, where parameters are found in a
file, binding errors, pages and attention plans of chunks, and the plain implementation's own invariants."""
import copy

import numpy as np
import pytest

import linonex_util as U
import plain_linonex as P


def _cfg(d):
    from transformer_amd.config.linonex import LinonexConfig
    return LinonexConfig.from_dict(d)


def test_config_reads_every_key_and_writes_it_back():
    cfg = _cfg(U.CFG_A)
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.max_positions, cfg.loop) == (211, 72, 1e-5, 600, (1, 4, 3))
    m, p = cfg.layers[0], cfg.layers[1]
    assert (m.type, m.memory.heads, m.memory.dim, m.memory.vdim, m.memory.gate_cap, m.mlp.ff, m.mlp.experts) == \
        ("mlstm", 3, 20, 12, 8.0, 48, 0)
    a, r, e = p.left, p.right, p.mlp
    assert (p.type, a.heads, a.kv_heads, a.dim, a.vdim, a.conv, a.scale, a.chunk, a.softcap) == ("parallel", 6, 2, 20, 20, 3, 0.3, 50, 12.0)
    assert (r.heads, r.kv_heads, r.dim, r.vdim, r.conv) == (6, 3, 24, 12, 4)
    assert (e.ff, e.experts, e.identity, e.top, e.scale) == (20, 6, 3, 2, 1.7)
    assert cfg.layers[4].mlp is None
    for c in (U.CFG_A, U.CFG_B, U.CFG_C, U.CFG_D):
        assert _cfg(_cfg(c).to_dict()) == _cfg(c)
    b = _cfg(U.CFG_B)                                    # absent keys: no chunks, no cap
    assert (b.layers[0].left.chunk, b.layers[0].left.softcap) == (None, None)
    short = copy.deepcopy(U.CFG_B)
    left, router = short["layers"][0]["mixer"]["left"], short["layers"][2]["mlp"]["router"]
    del left["kv_heads"], left["vdim"], left["conv"], router["identity"], router["scale"], short["loop"]
    s = _cfg(short)
    assert (s.layers[0].left.kv_heads, s.layers[0].left.vdim, s.layers[0].left.conv, s.loop) == (1, 32, 0, None)
    assert (s.layers[2].mlp.identity, s.layers[2].mlp.scale) == (0, 1.0)
    cut = _cfg(U.CFG_A).with_layers(2)
    assert (len(cut.layers), cut.loop) == (2, (1, 2, 3)) and _cfg(U.CFG_A).with_layers(1).loop is None


def test_config_errors_name_the_key():
    from transformer_amd.config.spec import ConfigError
    par = ("layers", 1, "mixer")
    for path, value in ((("layers", 0, "type"), "mamba"), (("layers", 0, "mlp", "kind"), "glu"), (("layers", 0, "mlp", "ff"), 0),
                        (("layers", 0, "mixer", "gate_cap"), 0.0), (("layers", 0, "mixer", "gate_cap"), None),
                        (("layers", 0, "mixer", "heads"), 0), (("layers", 0, "mixer"), None), ((*par, "left"), None),
                        ((*par, "left", "kv_heads"), 4), ((*par, "left", "mask", "size"), 0), ((*par, "left", "scale"), None),
                        ((*par, "left", "softcap"), 0.0), ((*par, "left", "conv"), -1), ((*par, "right", "conv"), 0),
                        ((*par, "right", "kv_heads"), 4), ((*par, "right", "dim"), None),
                        (("layers", 1, "mlp", "router", "top"), 10), (("layers", 1, "mlp", "router", "top"), None),
                        (("layers", 1, "mlp", "router", "identity"), -1), (("layers", 1, "mlp", "expert"), None),
                        (("max_positions",), 0), (("max_positions",), None), (("loop", "stop"), 6), (("loop", "start"), 4),
                        (("loop", "times"), 0), (("norm",), None), (("width",), 0), (("layers",), [])):
        d = copy.deepcopy(U.CFG_A)
        at = d
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError):
            _cfg(d)


def test_layout_blocks_schedule_and_cache_needs():
    import torch
    from transformer_amd.cache.storage import CacheError, KVNeed, StateNeed
    from transformer_amd.parts.base import PartError, build_part
    spec = _cfg(U.CFG_A).model_spec()
    assert [(r.block, r.reenter) for r in spec.schedule] == \
        [(0, False), (1, False), (2, False), (3, False), (1, True), (2, False), (3, False), (1, True), (2, False), (3, False), (4, False)]
    assert all(r.cache_of is None and r.opening is None for r in spec.schedule)
    assert [b.mixer.kind for b in spec.blocks] == ["matrix_memory", "branch_mean", "matrix_memory", "branch_mean", "matrix_memory"]
    assert [b.ffn.kind if b.ffn is not None else None for b in spec.blocks] == ["glu", "routed_mlp", "routed_mlp", "glu", None]
    left, right = spec.blocks[1].mixer.branches
    assert (left.kind, left.chunk, left.softcap, left.conv_taps, left.window, left.rot_dims, left.sink) == \
        ("attention_sink", 50, 12.0, 3, None, 0, None)
    assert (right.kind, right.decay_rank, right.gate_rank, right.gate_activation, right.taps) == ("gated_delta", None, None, "silu", 4)
    f = spec.blocks[1].ffn
    assert (f.score, f.renormalize, f.form, f.identity, f.correction, f.factor, f.weight_on) == ("softmax", False, "glu", 3, True, 1.7, "output")
    assert (spec.after_embed.kind, spec.after_embed.positions, spec.max_position, spec.tie_embeddings) == ("learned_positions", 600, 600, False)
    needs = [build_part(b, torch.float32, "cpu").cache_need() for b in spec.blocks]
    assert needs[0] == [StateNeed((3, 20, 12)), StateNeed((3, 20)), StateNeed((3,))]
    assert needs[1] == [KVNeed(2, 20, None, 20, chunk=50), StateNeed((2, 6 * 20 + 2 * 40)),
                        StateNeed((6, 24, 12)), StateNeed((3, 2 * 3 * 24 + 6 * 12))]
    b = [build_part(x, torch.float32, "cpu").cache_need() for x in _cfg(U.CFG_B).model_spec().blocks]
    assert b[0] == [KVNeed(1, 32), StateNeed((1, 64, 8))]           # one tap: no memory
    assert KVNeed(1, 8, chunk=70).span == 70 and KVNeed(1, 8, 30).span == 30 and KVNeed(1, 8).span is None
    with pytest.raises(CacheError):
        KVNeed(1, 8, 30, chunk=70)
    import dataclasses
    for kw in (dict(chunk=0), dict(chunk=5, window=9)):
        with pytest.raises(PartError):
            build_part(dataclasses.replace(left, **kw), torch.float32, "cpu")
    for kw in (dict(identity=-1), dict(top=10), dict(weight_on="input")):
        with pytest.raises(PartError):
            build_part(dataclasses.replace(f, **kw), torch.float32, "cpu")


def test_every_parameter_has_a_file_tensor_and_back():
    from transformer_amd.config.registry import get_architecture
    from transformer_amd.engine.params import declared_params
    arch = get_architecture("Linonex")
    assert get_architecture("linonex") is arch
    for cfg_dict in (U.CFG_A, U.CFG_B, U.CFG_C, U.CFG_D):
        cfg = arch.config_from_dict(cfg_dict)
        params = declared_params(arch.model_spec(cfg))
        src = arch.weight_sources(cfg, "safetensors")
        assert set(src) == set(params)
        named = {}
        for pname, s in src.items():
            assert sum(p.shape[0] for p in s.options[0]) == params[pname].shape[0], pname
            named.update({p.name: p.shape for p in s.options[0]})
        assert named == {n: tuple(s) for n, s in P.tensor_shapes(cfg_dict).items()}


def test_loader_reports_missing_and_misshaped_tensors(tmp_path):
    from transformer_amd.api import open_model_source
    from transformer_amd.engine.params import declared_params
    from transformer_amd.weights.loader import WeightsError, plan_binding
    w = dict(P.make_model_folder(tmp_path / "ok", U.CFG_A, 1))
    arch, cfg, f = open_model_source(tmp_path / "ok")
    assert arch.name == "Linonex"
    plan_binding(declared_params(arch.model_spec(cfg)), arch.weight_sources(cfg, f.format), f)
    bad = dict(w)
    del bad["l0.mix.i.b"], bad["l1.mlp.correction"]
    bad["pos"] = bad["pos"][:-1]
    bad["l1.mlp.e6.gate"] = np.zeros((20, 72))          # identity experts have no tensors
    (tmp_path / "bad").mkdir()
    P.write_safetensors(tmp_path / "bad" / "model.safetensors", bad, "BF16")
    (tmp_path / "bad" / "config.json").write_text((tmp_path / "ok" / "config.json").read_text())
    arch, cfg, f = open_model_source(tmp_path / "bad")
    with pytest.raises(WeightsError) as e:
        plan_binding(declared_params(arch.model_spec(cfg)), arch.weight_sources(cfg, f.format), f)
    assert e.value.missing == ["l0.mix.i.b", "l1.mlp.correction"] and e.value.unexpected == ["l1.mlp.e6.gate"]
    assert [n for n, _, _ in e.value.wrong_shape] == ["pos"]


def test_pages_of_left_chunks_go_back():
    from transformer_amd.cache.pool import RELEASED
    from transformer_amd.cache.storage import KVNeed, SequenceCache
    import torch
    need = KVNeed(1, 8, chunk=150)
    assert [need.first_key(n) for n in (0, 149, 150, 299, 300)] == [0, 0, 150, 150, 300]
    cache = SequenceCache([need], 600, 1, torch.float32, "cpu")
    slot, at = cache.alloc_slot(), 0
    for n, gone in ((140, 0), (9, 0), (1, 2), (149, 2), (1, 4), (100, 4), (50, 7)):
        cache.pool.reserve({slot: n})
        cache.pool.advance(slot, n)
        cache.release_outside_windows(slot)
        at += n
        pages = cache.pool.pages(slot, 0)
        assert [p == RELEASED for p in pages] == [True] * gone + [False] * (-(-at // 64) - gone), at
        cache.pool.check()
    few = SequenceCache([need], 1 << 16, 2, torch.float32, "cpu", max_step_tokens=64)
    assert few.group_pages[0] == 2 * (150 // 64 + 3) + 1


def test_key_units_cover_a_chunk():
    from transformer_amd import kernels as K
    assert K.first_key(1, None, 100) == 0 and K.first_key(100, None, 100) == 0 and K.first_key(101, None, 100) == 100
    assert K.seen_pages(500, None, chunk=100) == [(6, 2)]           # positions 400 .. 499
    assert K.seen_pages(501, None, chunk=100) == [(7, 1)] and K.seen_pages(50, None, chunk=100) == [(0, 1)]
    lens, chunk = [1, 70, 1000, 333, 2000], 130
    for n_units in (5, 9, 40):
        units, seq = K.plan_key_units(lens, n_units, tables=np.arange(5 * 40).reshape(5, 40), chunk=chunk)
        for b, n in enumerate(lens):
            rows = units[seq[b, 0]:seq[b, 0] + seq[b, 1]]
            got = [p for r in rows for p in range(r[1], r[1] + r[2])]
            assert got == list(range((n - 1) // chunk * chunk // 64, -(-n // 64)))
            assert all(r[4] == b * 40 + r[1] for r in rows)


# ---------------------------------------------------------------- the plain functions themselves
def test_plain_memory_is_a_weighted_sum_and_carries_its_state():
    rng = np.random.default_rng(0)
    T, H, dk, dv = 30, 3, 5, 4
    q, k, v = (rng.standard_normal((T, H, n)) for n in (dk, dk, dv))
    i, f = 4.0 * rng.standard_normal((T, H)), -P.softplus(-3.0 * rng.standard_normal((T, H)))
    o, (S, n, m) = P.matrix_memory(q, k, v, i, f)
    np.testing.assert_allclose(o, P.matrix_memory_sum(q, k, v, i, f), rtol=1e-7, atol=1e-9)
    o1, st = P.matrix_memory(q[:11], k[:11], v[:11], i[:11], f[:11])
    o2, (S2, n2, m2) = P.matrix_memory(q[11:], k[11:], v[11:], i[11:], f[11:], st)
    np.testing.assert_allclose(np.concatenate([o1, o2]), o)
    np.testing.assert_allclose(S2, S); np.testing.assert_allclose(n2, n); np.testing.assert_allclose(m2, m)
    # the maximum starts at 0: a first token with a small input gate is not scaled up to weight one
    _, (S1, _, m1) = P.matrix_memory(q[:1], k[:1], v[:1], np.full((1, H), -3.0), np.full((1, H), -0.5))
    np.testing.assert_allclose(m1, -0.5)
    np.testing.assert_allclose(S1, np.exp(-2.5) * k[0][:, :, None] * v[0][:, None, :])


def test_plain_chunks_convolutions_and_branches():
    see = P.same_chunk(10, 4)
    assert [list(np.nonzero(r)[0]) for r in see[[0, 3, 4, 6, 9]]] == [[0], [0, 1, 2, 3], [4], [4, 5, 6], [8, 9]]
    assert P.same_chunk(10, None).sum() == 55 and P.same_chunk(10, 1).sum() == 10 and (P.same_chunk(10, 10) == P.same_chunk(10, None)).all()
    np.testing.assert_allclose(P.causal_conv(np.arange(1.0, 5.0)[:, None], np.array([[10.0, 1.0]]))[:, 0], [1, 12, 23, 34])
    rng = np.random.default_rng(1)
    T, H, dk, dv = 9, 2, 4, 3
    q, k, v = rng.standard_normal((T, H, dk)), P.unit_length(rng.standard_normal((T, H, dk))), rng.standard_normal((T, H, dv))
    g, b = rng.uniform(0.2, 1.0, (T, H)), rng.uniform(0, 1, (T, H))
    o, S = P.delta_rule(q, k, v, g, b)
    o1, S1 = P.delta_rule(q[:4], k[:4], v[:4], g[:4], b[:4])
    o2, S2 = P.delta_rule(q[4:], k[4:], v[4:], g[4:], b[4:], S1)
    np.testing.assert_allclose(np.concatenate([o1, o2]), o)
    np.testing.assert_allclose(S2, S)
    o3, _ = P.delta_rule(k[:1], k[:1], v[:1], g[:1], np.ones((1, H)), S)     # a full step overwrites; the read-out sees it
    np.testing.assert_allclose(o3[0], v[0], atol=1e-5)


def test_plain_routing_corrections_and_identity_experts():
    rng = np.random.default_rng(2)
    d, E, I, top = 6, 4, 2, 3
    w = {"router": rng.standard_normal((E + I, d)), "correction": np.zeros(E + I)}
    for e in range(E):
        for n, s in (("gate", (5, d)), ("up", (5, d)), ("down", (d, 5))):
            w[f"e{e}.{n}"] = rng.standard_normal(s)
    mlp = {"router": {"experts": E, "identity": I, "top": top, "scale": 1.5}}
    h = rng.standard_normal((7, d))
    w["correction"][E:] = 5.0                            # both identity experts are always chosen
    s, choice = P.route(h, w, "", mlp["router"])
    np.testing.assert_allclose(s.sum(-1), 1.0)
    best = np.argmax(s[:, :E], axis=-1)
    want = 1.5 * np.stack([s[t, E:].sum() * h[t] + s[t, best[t]] * P.glu(h[t][None], w, f"e{best[t]}.")[0] for t in range(7)])
    np.testing.assert_allclose(P.moe(h, w, "", mlp), want)
    with pytest.raises(AssertionError, match="largest scores"):
        P.moe(h, w, "", mlp, forced=np.tile([0, 1, 2], (7, 1)), slack=0.1)


def test_plain_loop_order_and_positions():
    assert P.schedule({"layers": [0] * 4}) == [(0, False), (1, False), (2, False), (3, False)]
    assert P.schedule({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, False), (1, False), (2, False), (1, True), (2, False), (3, False)]
    m, toks = U.plain("A", "float32"), U.tokens("A", 9, 0)
    layers = []
    a = m.forward(toks, layers)
    assert len(layers) == 5 + 2 * 3
    np.testing.assert_allclose(a[:5], m.forward(toks[:5]), atol=1e-9)          # causal
    w = dict(m.w)
    w["pos"] = m.w["pos"].copy()
    w["pos"][6] += 1.0
    other = []
    P.PlainLinonex(config=m.c, weights=w).forward(toks, other)
    assert np.allclose(layers[0][:6], other[0][:6]) and not np.allclose(layers[0][6], other[0][6])
    # the embedding joins before the second and the third pass: without it (a loop of one pass, written out by
    # hand) the runs differ from the second pass on
    flat = dict(m.c)
    flat["layers"], flat["loop"] = m.c["layers"][:4], {"start": 1, "stop": 4, "times": 1}
    once = []
    P.PlainLinonex(config=flat, weights=m.w).forward(toks, once)
    assert all(np.allclose(x, y) for x, y in zip(layers[:4], once))


def test_bench_shapes_of_the_design_option_are_valid_models():
    import bench
    import transformer_amd as ta
    for size, (base, kinds, near) in bench.linonex_shapes().items():
        for kind, layers in kinds.items():
            spec = ta.LinonexConfig.from_dict({**base, "layers": layers}).model_spec()
            assert len(spec.blocks) == len(layers) and spec.hidden == base["width"], (size, kind)
        for arch, cfg_dict in near.values():
            assert ta.get_architecture("LlamaForCausalLM" if arch == "llama" else arch).config_from_dict(cfg_dict) \
                .model_spec().hidden == base["width"]
