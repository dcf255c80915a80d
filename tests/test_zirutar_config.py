"""Zirutar without a GPU: configuration keys, the layout it spells out, where parameters are
found in a file, binding errors, pages that stay for a sequence's first tokens, the single-token
attention's plan over what a window shows, and the plain implementation's own invariants."""
import copy
import json

import numpy as np
import pytest

import plain_zirutar as P
import zirutar_util as U


def _cfg(d):
    from transformer_amd.config.zirutar import ZirutarConfig
    return ZirutarConfig.from_dict(d)


def _named(d):
    """A configuration whose low-rank widths are given by hand, as ``decay_rank`` / ``gate_rank``."""
    d = copy.deepcopy(d)
    for l in d["layers"]:
        r = l["mixer"].pop("ranks", None)
        if r is not None:
            l["mixer"]["decay_rank"], l["mixer"]["gate_rank"] = r
    return d


def test_config_reads_every_key_and_writes_it_back():
    cfg = _cfg(_named(U.CFG_A))
    assert (cfg.vocab, cfg.width, cfg.eps, cfg.embed_scale, cfg.logit_scale, cfg.side_dim, cfg.loop) == \
        (211, 72, 1e-5, 3.0, 0.7, 10, (1, 4, 3))
    a, d, _, l, last = cfg.layers
    assert (a.type, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.keep_first, a.ff, a.limit) == \
        ("attention", 6, 2, 20, 20, 0.6, 50, 7, 48, 1.2)
    assert (d.type, d.heads, d.kv_heads, d.dim, d.vdim, d.conv, d.decay_rank, d.gate_rank, d.ff) == \
        ("channel_delta", 6, 3, 24, 12, 4, 8, 5, 40)
    assert (l.type, l.heads, l.dim, l.rot_dim, l.vdim, l.kv_rank, l.scale, l.rot_dims, l.rot_base) == \
        ("latent_attention", 5, 12, 6, 9, 20, 0.3, 6, 500.0)
    assert last.ff is None
    for c in (U.CFG_A, U.CFG_B, U.CFG_C, U.CFG_D):
        assert _cfg(_cfg(_named(c)).to_dict()) == _cfg(_named(c))
    b = _cfg(_named(U.CFG_B))            # absent keys: no window, nothing kept, no token input, scales of 1
    assert (b.layers[0].window, b.layers[0].keep_first, b.side_dim, b.embed_scale, b.logit_scale) == (None, 0, None, 1.0, 1.0)
    short = copy.deepcopy(_named(U.CFG_B))
    del short["layers"][0]["mixer"]["kv_heads"], short["layers"][0]["mixer"]["vdim"], short["loop"]
    assert (_cfg(short).layers[0].kv_heads, _cfg(short).layers[0].vdim, _cfg(short).loop) == (1, 32, None)
    cut = _cfg(_named(U.CFG_A)).with_layers(2)
    assert (len(cut.layers), cut.loop) == (2, (1, 2, 3)) and _cfg(_named(U.CFG_A)).with_layers(1).loop is None


def test_config_errors_name_the_key():
    from transformer_amd.config.spec import ConfigError
    for path, value in ((("layers", 0, "type"), "mamba"), (("layers", 0, "mlp", "kind"), "moe"), (("layers", 0, "mlp", "ff"), 0),
                        (("layers", 0, "mlp", "limit"), 0.0), (("layers", 0, "mlp", "limit"), None),
                        (("layers", 0, "mixer", "kv_heads"), 4), (("layers", 0, "mixer", "vdim"), 16),
                        (("layers", 0, "mixer", "mask", "size"), 0), (("layers", 0, "mixer", "mask", "keep_first"), -1),
                        (("layers", 0, "mixer", "scale"), None), (("layers", 0, "mixer"), None),
                        (("layers", 1, "mixer", "conv"), 0), (("layers", 1, "mixer", "kv_heads"), 4),
                        (("layers", 1, "mixer", "conv"), None), (("layers", 3, "mixer", "rot", "dims"), 5),
                        (("layers", 3, "mixer", "rot", "dims"), 8), (("layers", 3, "mixer", "kv_rank"), 0),
                        (("layers", 3, "mixer", "rot", "base"), None), (("token_side", "dim"), 0), (("loop", "stop"), 6),
                        (("loop", "start"), 4), (("loop", "times"), 0), (("loop", "times"), None), (("norm",), None),
                        (("width",), 0), (("layers",), [])):
        d = _named(U.CFG_A)
        at = d
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError):
            _cfg(d)
    with pytest.raises(ConfigError, match="ranks"):          # a hand-made configuration has to name them
        d = copy.deepcopy(U.CFG_A)
        _cfg(d).model_spec()


def test_layout_blocks_schedule_and_cache_needs():
    import torch
    from transformer_amd.cache.storage import KVNeed, StateNeed
    from transformer_amd.parts.base import build_part
    spec = _cfg(_named(U.CFG_A)).model_spec()
    assert [(r.block, r.opening) for r in spec.schedule] == \
        [(0, None), (1, 0), (2, None), (3, None), (1, 1), (2, None), (3, None), (1, 2), (2, None), (3, None), (4, None)]
    assert all(r.cache_of is None for r in spec.schedule) and spec.stream_rows == 3
    assert [b.mixer.kind for b in spec.blocks] == ["attention_sink", "gated_delta", "attention_sink", "latent_attention", "gated_delta"]
    assert [b.ffn.kind if b.ffn is not None else None for b in spec.blocks] == ["glu"] * 4 + [None]
    assert all(b.kind == "prenorm" and b.side.kind == "token_side" and b.norm1.kind == "rmsnorm_offset" for b in spec.blocks)
    assert [b.side.offset for b in spec.blocks] == [0, 10, 20, 30, 40]
    a, d, l = spec.blocks[0].mixer, spec.blocks[1].mixer, spec.blocks[3].mixer
    assert (a.window, a.keep_first, a.unit_norm, a.values_from_keys, a.head_gate, a.sink, a.rot_dims) == (50, 7, True, True, True, None, 0)
    assert (d.num_heads, d.num_kv_heads, d.taps, d.decay_rank, d.gate_rank) == (6, 3, 4, 8, 5)
    assert (l.q_rank, l.sink, l.gated, l.window, l.rot_dims) == (None, True, False, None, 6)
    f = spec.blocks[0].ffn
    assert (f.activation, f.limit, f.gate_slope, f.up_shift) == ("limited", 1.2, 1.702, 1.0)
    needs = [build_part(b, torch.float32, "cpu").cache_need() for b in spec.blocks]
    assert needs[0] == KVNeed(2, 20, 50, 20, 7) and needs[2] == KVNeed(1, 32, 90, 32, 70)
    assert needs[1] == [StateNeed((6, 24, 12)), StateNeed((3, 2 * 3 * 24 + 6 * 12))]
    assert needs[3] == KVNeed(1, 26, None, 0)
    assert spec.after_embed.kind == "chain" and spec.on_logits.scale == 0.7 and spec.tie_embeddings is True
    b = _cfg(_named(U.CFG_B)).model_spec()
    assert b.after_embed is None and b.on_logits is None and b.schedule[0].opening == 0 and b.blocks[0].side is None
    assert build_part(b.blocks[2], torch.float32, "cpu").cache_need() == [StateNeed((1, 64, 8))]       # one tap: no memory
    assert KVNeed(1, 8, None, 8, 5) == KVNeed(1, 8)          # without a window everything stays anyway


def test_every_parameter_has_a_file_tensor_and_back():
    from transformer_amd.config.registry import get_architecture
    from transformer_amd.engine.params import declared_params
    arch = get_architecture("Zirutar")
    assert get_architecture("zirutar") is arch
    for cfg_dict in (U.CFG_A, U.CFG_B, U.CFG_C, U.CFG_D):
        cfg = arch.config_from_dict(_named(cfg_dict))
        params = declared_params(arch.model_spec(cfg))
        src = arch.weight_sources(cfg, "safetensors")
        assert set(src) == set(params)
        named = {}
        for pname, s in src.items():
            if not s.options:
                continue
            assert sum(p.shape[0] for p in s.options[0]) == params[pname].shape[0], pname
            named.update({p.name: p.shape for p in s.options[0]})
        assert named == {n: tuple(s) for n, s in P.tensor_shapes(cfg_dict).items()}


def test_loader_reads_ranks_and_reports_missing_and_misshaped_tensors(tmp_path):
    from transformer_amd.api import open_model_source
    from transformer_amd.engine.params import declared_params
    from transformer_amd.weights.loader import WeightsError, plan_binding
    w = dict(P.make_model_folder(tmp_path / "ok", U.CFG_A, 1))
    arch, cfg, f = open_model_source(tmp_path / "ok")
    assert arch.name == "Zirutar" and (cfg.layers[1].decay_rank, cfg.layers[1].gate_rank) == (8, 5)
    plan_binding(declared_params(arch.model_spec(cfg)), arch.weight_sources(cfg, f.format), f)
    bad = dict(w)
    del bad["l1.mix.A_log"]
    bad["l3.mix.sink"] = bad["l3.mix.sink"][:-1]
    bad["loop.step"] = bad["loop.step"][:2]
    bad["l0.mix.v"] = np.zeros((40, 72))            # the values are the keys
    (tmp_path / "bad").mkdir()
    P.write_safetensors(tmp_path / "bad" / "model.safetensors", bad, "BF16")
    (tmp_path / "bad" / "config.json").write_text((tmp_path / "ok" / "config.json").read_text())
    arch, cfg, f = open_model_source(tmp_path / "bad")
    with pytest.raises(WeightsError) as e:
        plan_binding(declared_params(arch.model_spec(cfg)), arch.weight_sources(cfg, f.format), f)
    assert e.value.missing == ["l1.mix.A_log"] and e.value.unexpected == ["l0.mix.v"]
    assert sorted(n for n, _, _ in e.value.wrong_shape) == ["l3.mix.sink", "loop.step"]


def test_pages_of_kept_first_tokens_stay_with_the_slot():
    from transformer_amd.cache.pool import RELEASED, CacheError, SlotPool
    s = SlotPool(2, 64, {0: 12})
    a, b = s.alloc(), s.alloc()
    s.reserve({a: 500, b: 10}); s.advance(a, 500); s.advance(b, 10)
    window, keep = 100, 2                                      # pages of the first tokens that stay
    assert s.release_before(a, 0, 500 + 1 - window, keep) == 4  # positions < 401: pages 0 .. 5, of which two stay
    assert s.release_before(a, 0, 500 + 1 - window, keep) == 0
    assert s.release_before(b, 0, 10 + 1 - window, keep) == 0   # shorter than what is kept
    pages = s.pages(a, 0)
    assert [p == RELEASED for p in pages] == [False] * 2 + [True] * 4 + [False] * 2
    s.check()
    with pytest.raises(CacheError):
        s.release_before(a, 0, 450, 1)                          # another number of kept pages than before
    s.reserve({a: 60}); s.advance(a, 60)
    assert s.release_before(a, 0, 560 + 1 - window, keep) == 1
    s.check()
    s.reset(a)
    s.check()
    s.reserve({a: 64}); s.advance(a, 64)
    assert s.release_before(a, 0, 10 ** 6, 0) == 1              # forgotten with the pages
    s.free(a); s.free(b)
    s.check()
    assert s.pools[0].free_count == 12


def test_key_units_cover_what_a_window_shows():
    from transformer_amd import kernels as K
    assert K.seen_pages(1, None) == [(0, 1)] and K.seen_pages(500, None) == [(0, 8)]
    assert K.seen_pages(500, 100) == [(6, 2)]                   # positions 400 .. 499
    assert K.seen_pages(500, 100, 1) == [(0, 1), (6, 2)] and K.seen_pages(500, 100, 65) == [(0, 2), (6, 2)]
    assert K.seen_pages(500, 100, 400) == [(0, 8)]              # the kept ones meet the window
    assert K.seen_pages(50, 100, 7) == [(0, 1)]
    lens, window, keep = [1, 70, 1000, 333, 2000], 130, 70
    for n_units in (5, 9, 10, 11, 40):
        units, seq = K.plan_key_units(lens, n_units, tables=np.arange(5 * 40).reshape(5, 40), window=window, keep_first=keep)
        for b, n in enumerate(lens):
            rows = units[seq[b, 0]:seq[b, 0] + seq[b, 1]]
            assert (rows[:, 0] == b).all() and (rows[:, 2] > 0).all() and (rows[:, 6] == seq[b, 1]).all() and (rows[:, 3] == n).all()
            got = [p for r in rows for p in range(r[1], r[1] + r[2])]
            assert got == sorted(set(got))
            want = [p for f, c in K.seen_pages(n, window if n_units >= 9 else None, keep) for p in range(f, f + c)]
            if n_units >= 9:                                    # eight ranges in all: enough units for each
                assert got == want
            assert set(p for f, c in K.seen_pages(n, window, keep) for p in range(f, f + c)) <= set(got)
            assert all(r[4] == b * 40 + r[1] for r in rows)


# ---------------------------------------------------------------- the plain functions themselves
def test_plain_window_and_kept_tokens():
    see = P.visible(10, 3, 2)
    assert list(np.nonzero(see[7])[0]) == [0, 1, 5, 6, 7] and list(np.nonzero(see[1])[0]) == [0, 1]
    assert list(np.nonzero(P.visible(10, 1, 0)[6])[0]) == [6] and P.visible(10, None, 0).sum() == 55
    assert (P.visible(10, 4, 10) == P.visible(10, None, 0)).all()
    rng = np.random.default_rng(0)
    s = rng.standard_normal((10, 10))
    p = P.softmax_rows(s, see)
    np.testing.assert_allclose(p.sum(-1), 1.0)
    assert (p[~see] == 0).all()
    sunk = P.softmax_rows(s, see, 1.3)
    np.testing.assert_allclose(sunk * (1 + np.exp(1.3) / np.where(see, np.exp(s), 0).sum(-1, keepdims=True)), p)


def test_plain_values_are_keys_before_their_norm():
    rng = np.random.default_rng(1)
    d, w = 6, {}
    w["q"], w["k"], w["g"], w["o"] = rng.standard_normal((8, d)), rng.standard_normal((4, d)), np.zeros((2, d)), np.eye(8)
    h = rng.standard_normal((5, d))
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "scale": 1.0, "mask": {"size": 1}}
    got = P.shared_kv_attention(h, w, "", m, 1e-6)               # one key: its value, half of it through the gate
    np.testing.assert_allclose(got, 0.5 * np.tile(h @ w["k"].T, (1, 2)))
    w["k"] = w["k"] * 7.0                                        # the scores do not see the keys' length, the values do
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "scale": 1.0}
    w2 = {**w, "k": w["k"] / 7.0}
    np.testing.assert_allclose(P.shared_kv_attention(h, w, "", m, 0.0), 7.0 * P.shared_kv_attention(h, w2, "", m, 0.0))


def test_plain_delta_rule_overwrites_and_carries_its_state():
    rng = np.random.default_rng(2)
    T, H, dk, dv = 9, 2, 4, 3
    q, k, v = rng.standard_normal((T, H, dk)), P.unit_length(rng.standard_normal((T, H, dk))), rng.standard_normal((T, H, dv))
    g, b = rng.uniform(0.2, 1.0, (T, H, dk)), rng.uniform(0, 1, (T, H))
    o, S = P.delta_rule(q, k, v, g, b)
    o1, S1 = P.delta_rule(q[:4], k[:4], v[:4], g[:4], b[:4])
    o2, S2 = P.delta_rule(q[4:], k[4:], v[4:], g[4:], b[4:], S1)
    np.testing.assert_allclose(np.concatenate([o1, o2]), o)
    np.testing.assert_allclose(S2, S)
    # a full step and no decay: what the state answers to a token's key is that token's value, whatever was there
    one = np.ones((1, H))
    _, S3 = P.delta_rule(q[:1], k[:1], v[:1], np.ones((1, H, dk)), one, S)
    np.testing.assert_allclose(np.einsum("hkv,hk->hv", S3, k[0]), v[0], atol=1e-5)
    # the read-out sees the current token's write and the decay acts on it before
    o4, _ = P.delta_rule(k[:1], k[:1], v[:1], g[:1], one)
    np.testing.assert_allclose(o4[0], v[0], atol=1e-5)
    np.testing.assert_allclose(P.causal_conv(np.arange(1.0, 5.0)[:, None], np.array([[10.0, 1.0]]))[:, 0], [1, 12, 23, 34])


def test_plain_loop_order_and_token_input():
    assert P.schedule({"layers": [0] * 4}) == [(0, None), (1, None), (2, None), (3, None)]
    assert P.schedule({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == \
        [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    m, toks = U.plain("A", "float32"), U.tokens("A", 9, 0)
    layers = []
    a = m.forward(toks, layers)
    assert len(layers) == 5 + 2 * 3
    np.testing.assert_allclose(a[:5], m.forward(toks[:5]), atol=1e-9)          # causal
    w = dict(m.w)
    w["loop.step"] = m.w["loop.step"] * np.array([[1.0], [1.0], [0.0]])        # the third pass opens with nothing
    other = []
    P.PlainZirutar(config=m.c, weights=w).forward(toks, other)
    same = [np.allclose(x, y) for x, y in zip(layers, other)]
    assert same == [True] * 7 + [False] * 4
    g = P.limited_glu(np.array([[9.0, -9.0]]), {"gate": np.eye(2), "up": np.eye(2), "down": np.eye(2)}, "", 1.5)
    np.testing.assert_allclose(g[0], [1.5 * P.sigmoid(1.702 * 1.5) * 2.5, -9.0 * P.sigmoid(-1.702 * 9.0) * -0.5])


def test_bench_shapes_of_the_design_option_are_valid_models():
    import bench
    import transformer_amd as ta
    for size, (base, kinds, near) in bench.zirutar_shapes().items():
        for kind, layers in kinds.items():
            spec = ta.ZirutarConfig.from_dict({**base, "layers": layers}).model_spec()
            assert len(spec.blocks) == len(layers) and spec.hidden == base["width"], (size, kind)
        for arch, cfg_dict in near.values():
            assert ta.get_architecture("LlamaForCausalLM" if arch == "llama" else arch).config_from_dict(cfg_dict) \
                .model_spec().hidden == base["width"]
