"""Decode and prefill throughput of the Llama-3.1-8B shape with random weights.

    python bench.py [--gpus 1] [--steps K] [--warmup W]

One JSON line on stdout. ``value`` is decoded tokens per second at batch 8: a
step is one decode step of the generation loop itself (``run_batches`` over the
engine's stepper: step function, argmax on the GPU, every step's tokens back on
the host while the next step runs). Prompts have unequal, seeded lengths of
128-2048 tokens; the context length is 4096. ``points`` holds the same at batch 1
and 64, at a long context, for other prompt lengths and for the Llama-2-7B shape,
each with its time, context and fraction of the roofline.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)

# published peaks of MI355X
HBM_GBS = 8000.0
PEAK_TFLOPS = {"bf16": 2500.0, "fp16": 2500.0, "fp8": 5000.0, "fp32": 157.3}

from transformer_amd.config.shapes import LLAMA2_7B, LLAMA3_70B, LLAMA31_8B, SHAPES  # noqa: E402,F401

# prompt lengths of the decode batch that each configuration is quoted with
PROMPTS = {"8b": (128, 2048), "7b": (64, 1024), "70b": (2048, 2048)}
CONTEXT = 4096
PROMPT_MIN, PROMPT_MAX = 128, 2048
PREFILL_TOKENS = 2048


def prefill_flops(cfg, T):
    """Matrix products of T prompt tokens, causal attention, one row of the output matrix."""
    d, nh, nkv, dh, di = cfg.hidden, cfg.num_heads, cfg.num_kv_heads, cfg.head_dim, cfg.intermediate
    per_layer = 2 * T * d * (nh + 2 * nkv) * dh + 2 * T * nh * dh * d + 2 * T * d * 2 * di + 2 * T * di * d
    attn = 2 * 2 * nh * dh * (T * (T + 1) // 2)
    return cfg.num_layers * (per_layer + attn) + 2 * d * cfg.vocab


def decode_bytes(model, cfg, contexts):
    """What a decode step has to read: every weight it uses, once, and the cache of
    the live sequences."""
    import torch
    w = model.weight_bytes()
    if model.w["embed"].data_ptr() != model.w["head"].data_ptr():
        w -= model.w["embed"].numel() * model.w["embed"].element_size()   # only rows are read
    item = torch.empty((), dtype=model.dtype).element_size()
    return w + sum(contexts) * cfg.kv_bytes_per_token(item)


def time_decode(model, cfg, batch, steps, warmup, seed, prompt_min=PROMPT_MIN, prompt_max=PROMPT_MAX):
    """Times ``steps`` decode steps of the generation loop itself: ``run_batches`` over a
    ``ModelStepper`` (all prompts in one step, then one token per sequence and step, the next
    step started before the last one's tokens have reached the host), greedy, no stop token.
    The stepper is the engine's own with a clock added: before the first timed step is started
    and before the step after the last timed one, it waits for the GPU and reads the time, so
    exactly ``steps`` steps lie between the two readings, after ``warmup`` untimed ones.
    Returns (seconds, each sequence's context half-way, the loop's own Timing)."""
    import numpy as np
    import torch
    from transformer_amd.engine.generate import ModelStepper, run_batches
    from transformer_amd.sampling.sampler import Sampler
    rng = np.random.default_rng(seed)
    lens = [int(x) for x in rng.integers(prompt_min, prompt_max + 1, batch)]
    new_tokens = warmup + steps + 2
    cache = model.new_cache(sum(-(-(n + new_tokens) // 64) * 64 for n in lens), max_slots=batch)
    prompts = [[int(t) for t in rng.integers(0, cfg.vocab, n)] for n in lens]

    class Clocked(ModelStepper):
        def __init__(self, *args):
            super().__init__(*args)
            self.calls, self.marks, self.lengths = 0, [], None

        def step_async(self, items, previous=None, take=None):
            if self.calls in (1 + warmup, 1 + warmup + steps):      # call 0 runs the prompts
                torch.cuda.synchronize()
                self.marks.append(time.perf_counter())
                if self.lengths is None:
                    self.lengths = [self.cache.length(slot) for slot, *_ in items]
            self.calls += 1
            return super().step_async(items, previous, take)

    stepper = Clocked(model, cache, Sampler(device=model.device))
    result = run_batches(stepper, prompts, new_tokens, (), cache.num_pages * 64, batch,
                         max_position=model.spec.max_position)
    torch.cuda.synchronize()
    if len(stepper.marks) != 2 or len(result.batches) != 1 or \
            any(len(t) != new_tokens for t in result.tokens):
        raise RuntimeError("the generation loop did not run the steps that were to be timed")
    dt = stepper.marks[1] - stepper.marks[0]
    ctx_mid = [n + steps // 2 for n in stepper.lengths]
    del cache, stepper
    torch.cuda.empty_cache()
    return dt, ctx_mid, result.timing


def decode_point(model, cfg, batch, steps, warmup, seed, prompt_min, prompt_max):
    """One decode measurement with everything its roofline needs."""
    dt, ctx, timing = time_decode(model, cfg, batch, steps, warmup, seed, prompt_min, prompt_max)
    nbytes = decode_bytes(model, cfg, ctx)
    gbs = nbytes / (dt / steps) / 1e9
    return {"tok_s": round(batch * steps / dt, 2), "ms_per_step": round(dt / steps * 1e3, 4),
            "mean_context": round(sum(ctx) / len(ctx), 1), "gbs": round(gbs, 1),
            "frac": round(gbs / HBM_GBS, 4),
            # the loop's own table: every single-token step it ran, the recording of the first among them
            "loop_tok_s": round(timing.decode_tokens / max(timing.decode_seconds, 1e-9), 2)}


def time_prefill(model, cfg, reps, seed, tokens=PREFILL_TOKENS, lengths=None):
    """Median seconds of one step that runs a prompt of ``tokens`` tokens (or prompts of
    ``lengths``, together in one step) and returns the logits of each prompt's last place."""
    import numpy as np
    import torch
    from transformer_amd import Entry
    rng = np.random.default_rng(seed)
    lengths = list(lengths) if lengths is not None else [tokens]
    toks = [[int(t) for t in rng.integers(0, cfg.vocab, n)] for n in lengths]
    cache = model.new_cache(sum(-(-n // 64) * 64 for n in lengths), max_slots=len(lengths))
    times = []
    for r in range(reps + 1):
        slots = [cache.alloc_slot() for _ in lengths]
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        model.step(cache, [Entry(s, t, (len(t) - 1,)) for s, t in zip(slots, toks)])
        torch.cuda.synchronize()
        dt = time.perf_counter() - t0
        for s_ in slots:
            cache.free_slot(s_)
        if r > 0:                       # the first run warms the library's kernel choice
            times.append(dt)
    del cache
    torch.cuda.empty_cache()
    return sorted(times)[len(times) // 2]          # the median


def prefill_point(model, cfg, dkey, reps, seed, tokens=None, lengths=None):
    lengths = list(lengths) if lengths is not None else [tokens]
    pt = time_prefill(model, cfg, reps, seed, lengths=lengths)
    fl = sum(prefill_flops(cfg, n) for n in lengths)
    total = sum(lengths)
    return {"value": round(total / pt, 1), "tokens": total, "ms": round(pt * 1e3, 3),
            "frac": round(fl / pt / (PEAK_TFLOPS[dkey] * 1e12), 4)}


# ---------------------------------------------------------------------------------------------
# --design vametar: the Vametar decoder beside the Llama decoder at equal layer sizes

def vametar_shapes():
    """Layer sizes that resemble real models' (random weights). Each gives the Vametar mixers'
    sizes and the Llama layer of the same width, heads and feed-forward."""
    def shape(width, heads, kv, ff, rec_width, rec_blocks, gla_heads, gla_dim, gla_vdim, vocab):
        att = {"type": "attention", "mlp": {"kind": "dense", "ff": ff},
               "mixer": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 64, "scale": 128 ** -0.5,
                         "rot": {"base": 500000.0, "dims": 128}, "v_mix": True}}
        rec = {"type": "rglru", "mlp": {"kind": "dense", "ff": ff},
               "mixer": {"width": rec_width, "blocks": rec_blocks, "conv": 4}}
        gla = {"type": "gla", "mlp": {"kind": "dense", "ff": ff},
               "mixer": {"heads": gla_heads, "dim": gla_dim, "vdim": gla_vdim, "tau": 16.0, "rank": 16}}
        base = {"architecture": "Vametar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                "residual_mult": 0.7, "logit_scale": 2.0,
                "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}}}
        llama = {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "hidden_size": width,
                 "num_attention_heads": heads, "num_key_value_heads": kv, "head_dim": 128,
                 "intermediate_size": ff, "vocab_size": vocab, "rope_theta": 500000.0, "rms_norm_eps": 1e-5,
                 "tie_word_embeddings": False, "max_position_embeddings": 1 << 20, "rope_scaling": None}
        return base, {"attention": att, "rglru": rec, "gla": gla}, llama
    return {"w2048": shape(2048, 16, 4, 8192, 2560, 10, 16, 64, 128, 32000),
            "w4096": shape(4096, 32, 8, 14336, 4096, 16, 32, 128, 128, 32000)}


def kunitar_shapes():
    """Layer sizes that resemble real models' (random weights): Kunitar models whose layers are
    all of one kind, the mixed order with a layer that reads its neighbour's cached rows, and the
    Llama layer of the same width, heads and dense feed-forward. The Vametar layer with gated
    linear attention of the same heads stands beside the recurrence (``vametar_like``)."""
    def shape(width, heads, q_rank, kv_rank, window, ff, wkv_heads, experts, top, eff, sff, vocab):
        dense = {"kind": "dense", "ff": ff}
        moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": eff}, "shared": {"ff": sff}}

        def lat(mlp, kv_from=None):
            m = {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "q_rank": q_rank, "kv_rank": kv_rank,
                 "scale": 192 ** -0.5, "rot": {"base": 500000.0, "dims": 64}, "mask": {"size": window}}
            if kv_from is not None:
                m["kv_from"] = kv_from
            return {"type": "latent_attention", "mixer": m, "mlp": mlp}

        def wkv(mlp):
            return {"type": "wkv", "mixer": {"heads": wkv_heads, "dim": 64, "decay_rank": 64}, "mlp": mlp}

        base = {"architecture": "Kunitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                "embedding": {"scale": 2.0}, "token_side": {"dim": 64}}
        kinds = {"latent": lambda n: [lat(dense)] * n, "wkv": lambda n: [wkv(dense)] * n,
                 "latent_moe": lambda n: [lat(moe)] * n,
                 "mixed": lambda n: [[wkv(dense), wkv(moe), lat(moe), lat(moe, kv_from=4 * (i // 4) + 2)][i % 4]
                                     for i in range(n)]}
        llama = {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "hidden_size": width,
                 "num_attention_heads": heads, "num_key_value_heads": max(1, heads // 4), "head_dim": 128,
                 "intermediate_size": ff, "vocab_size": vocab, "rope_theta": 500000.0, "rms_norm_eps": 1e-5,
                 "tie_word_embeddings": False, "max_position_embeddings": 1 << 20, "rope_scaling": None}
        vametar_like = {"architecture": "Vametar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                        "residual_mult": 0.7, "logit_scale": 2.0,
                        "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}},
                        "layers": [{"type": "gla", "mlp": {"kind": "dense", "ff": ff},
                                    "mixer": {"heads": wkv_heads, "dim": 64, "vdim": 64, "tau": 16.0, "rank": 64}}]}
        llama["vametar_like"] = vametar_like
        return base, {k: f(4) for k, f in kinds.items()}, llama
    return {"w2048": shape(2048, 16, 768, 256, 1024, 8192, 32, 32, 4, 1024, 2048, 32000),
            "w4096": shape(4096, 32, 1536, 512, 4096, 14336, 64, 64, 6, 1408, 2816, 32000)}


def luduvik_shapes():
    """Layer sizes that resemble real models' (random weights): Luduvik models whose layers are
    all lightning or all parallel (each with the routed feed-forward), the mixed order, and the
    closest layers of the other decoders at the same width and heads: the Vametar decoder's gated
    linear attention and its attention, the Kunitar decoder's recurrence with the routed
    feed-forward of the same experts, and the Llama layer."""
    def shape(width, heads, kv, lin_heads, experts, top, eff, sff, ff, vocab):
        moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": eff, "limit": 7.0},
               "shared": {"ff": sff, "limit": 7.0}}
        decay = [1.0 - 2.0 ** -(5.0 + 4.0 * i / lin_heads) for i in range(lin_heads)]
        light = {"type": "lightning", "mixer": {"heads": lin_heads, "dim": 128, "vdim": 128, "decay": decay}, "mlp": moe}
        par = {"type": "parallel", "mlp": moe, "mixer": {
            "left": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                     "rot": {"base": 500000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}},
            "right": {"heads": lin_heads, "dim": 128, "vdim": 128, "decay": decay, "rot": {"base": 10000.0, "dims": 128}}}}
        base = {"architecture": "Luduvik", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}}
        kinds = {"lightning": [light] * 4, "parallel": [par] * 4, "mixed": [light, par, light, light]}
        vam = {"architecture": "Vametar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "residual_mult": 0.7,
               "logit_scale": 2.0, "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}}}
        dense = {"kind": "dense", "ff": ff}
        near = {
            "vametar_gla": ("Vametar", {**vam, "layers": [{"type": "gla", "mlp": dense, "mixer": {
                "heads": lin_heads, "dim": 128, "vdim": 128, "tau": 16.0, "rank": 16}}] * 4}),
            "vametar_attention": ("Vametar", {**vam, "layers": [{"type": "attention", "mlp": dense, "mixer": {
                "heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                "rot": {"base": 500000.0, "dims": 64}}}] * 4}),
            "kunitar_wkv_moe": ("Kunitar", {"architecture": "Kunitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                                            "embedding": {"scale": 2.0}, "layers": [{
                                                "type": "wkv", "mixer": {"heads": 2 * lin_heads, "dim": 64, "decay_rank": 64},
                                                "mlp": {"kind": "moe", "router": {"experts": experts, "top": top},
                                                        "expert": {"ff": eff}, "shared": {"ff": sff}}}] * 4}),
            "llama": ("llama", {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "hidden_size": width,
                                "num_attention_heads": heads, "num_key_value_heads": kv, "head_dim": 128,
                                "intermediate_size": ff, "vocab_size": vocab, "rope_theta": 500000.0, "rms_norm_eps": 1e-5,
                                "tie_word_embeddings": False, "max_position_embeddings": 1 << 20, "rope_scaling": None,
                                "num_hidden_layers": 4}),
        }
        return base, kinds, near
    return {"w2048": shape(2048, 16, 4, 16, 32, 4, 1024, 2048, 8192, 32000),
            "w4096": shape(4096, 32, 8, 32, 64, 6, 1408, 2816, 14336, 32000)}


def saredra_shapes():
    """Layer sizes that resemble real models' (random weights): Saredra models whose layers are
    all attention or all parallel (each with the routed feed-forward), the mixed order with a
    layer that reads another's keys and values, and the closest layers of the other decoders at
    the same width and heads: the Luduvik decoder's parallel layer (softmax attention beside a
    matrix-state recurrence, with routed experts of the same sizes), the Vametar decoder's
    attention and its gated linear attention, and the Llama layer."""
    def shape(width, heads, kv, ssm_heads, experts, top, eff, ff, vocab):
        moe = {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": 4, "keep": 2}},
               "expert": {"ff": eff}}
        soft = {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5, "softcap": 50.0,
                "mask": {"size": 1024}}
        att = {"type": "attention", "mixer": {**soft, "rot": {"base": 500000.0, "dims": 64}}, "mlp": moe}
        reader = {"type": "attention", "mixer": {**att["mixer"], "kv_from": 0}, "mlp": moe}
        par = {"type": "parallel", "mlp": moe, "mixer": {
            "left": {**soft, "conv": 4, "rot": {"base": 500000.0, "dims": 64,
                                                 "scaling": {"factor": 8.0, "original": 8192, "fast": 32.0, "slow": 1.0}}},
            "left_scale": 1.0, "right_scale": 1.0,
            "right": {"heads": ssm_heads, "vdim": 64, "state": 128, "groups": 8, "conv": 4, "norm_groups": 8}}}
        base = {"architecture": "Saredra", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}}
        kinds = {"attention": [att] * 4, "parallel": [par] * 4, "mixed": [att, par, reader, att]}
        vam = {"architecture": "Vametar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "residual_mult": 0.7,
               "logit_scale": 2.0, "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}}}
        dense = {"kind": "dense", "ff": ff}
        lmoe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": eff, "limit": 7.0}}
        lin = ssm_heads // 2
        near = {
            "luduvik_parallel": ("Luduvik", {"architecture": "Luduvik", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                                             "layers": [{"type": "parallel", "mlp": lmoe, "mixer": {
                                                 "left": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                                          "rot": {"base": 500000.0, "dims": 64}},
                                                 "right": {"heads": lin, "dim": 128, "vdim": 128,
                                                           "decay": [1.0 - 2.0 ** -(5.0 + 4.0 * i / lin) for i in range(lin)]}}}] * 4}),
            "vametar_attention": ("Vametar", {**vam, "layers": [{"type": "attention", "mlp": dense, "mixer": {
                "heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                "rot": {"base": 500000.0, "dims": 64}}}] * 4}),
            "vametar_gla": ("Vametar", {**vam, "layers": [{"type": "gla", "mlp": dense, "mixer": {
                "heads": lin, "dim": 128, "vdim": 128, "tau": 16.0, "rank": 16}}] * 4}),
            "llama": ("llama", {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "hidden_size": width,
                                "num_attention_heads": heads, "num_key_value_heads": kv, "head_dim": 128,
                                "intermediate_size": ff, "vocab_size": vocab, "rope_theta": 500000.0, "rms_norm_eps": 1e-5,
                                "tie_word_embeddings": False, "max_position_embeddings": 1 << 20, "rope_scaling": None,
                                "num_hidden_layers": 4}),
        }
        return base, kinds, near
    return {"w2048": shape(2048, 16, 4, 64, 32, 4, 1024, 8192, 32000),
            "w4096": shape(4096, 32, 8, 128, 64, 6, 1408, 14336, 32000)}


def zirutar_shapes():
    """Layer sizes that resemble real models' (random weights): Zirutar models whose layers are all
    attention, all latent attention or all delta rule (each with the limited feed-forward and the
    token input), the mixed order, and the closest layers of the other decoders at the same width and
    heads: the Saredra decoder's windowed attention, the Kunitar decoder's latent attention, the Vametar
    decoder's gated linear attention, and the Llama layer."""
    def shape(width, heads, kv, q_rank, rank, window, keep, low, ff, vocab):
        mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
        dense = {"kind": "dense", "ff": ff}
        att = {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 2.0,
                                                          "mask": {"size": window, "keep_first": keep}}}
        latent = {"heads": heads, "dim": 128, "rot_dim": 64, "vdim": 128, "kv_rank": rank, "scale": 192 ** -0.5,
                  "rot": {"base": 500000.0, "dims": 64}}
        lat = {"type": "latent_attention", "mixer": latent, "mlp": mlp}
        delta = {"type": "channel_delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4,
                                                               "decay_rank": low, "gate_rank": low}}
        base = {"architecture": "Zirutar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "embedding": {"scale": 2.0},
                "logit_scale": 0.5, "token_side": {"dim": 64}}
        kinds = {"attention": [att] * 4, "latent": [lat] * 4, "delta": [delta] * 4, "mixed": [att, delta, lat, att]}
        near = {
            "saredra_attention": ("Saredra", {"architecture": "Saredra", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                                              "layers": [{"type": "attention", "mlp": dense, "mixer": {
                                                  "heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "scale": 128 ** -0.5,
                                                  "mask": {"size": window}, "rot": {"base": 500000.0, "dims": 64}}}] * 4}),
            "kunitar_latent": ("Kunitar", {"architecture": "Kunitar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                                           "embedding": {"scale": 2.0}, "token_side": {"dim": 64},
                                           "layers": [{"type": "latent_attention", "mixer": {**latent, "q_rank": q_rank},
                                                       "mlp": dense}] * 4}),
            "vametar_gla": ("Vametar", {"architecture": "Vametar", "vocab": vocab, "width": width, "norm": {"eps": 1e-5},
                                        "residual_mult": 0.7, "logit_scale": 2.0,
                                        "embedding": {"bigram": {"buckets": 65521, "mul_prev": 31, "mul_cur": 7}},
                                        "layers": [{"type": "gla", "mlp": dense, "mixer": {
                                            "heads": heads, "dim": 128, "vdim": 128, "tau": 16.0, "rank": low}}] * 4}),
            "llama": ("llama", {"architectures": ["LlamaForCausalLM"], "model_type": "llama", "hidden_size": width,
                                "num_attention_heads": heads, "num_key_value_heads": kv, "head_dim": 128,
                                "intermediate_size": ff, "vocab_size": vocab, "rope_theta": 500000.0, "rms_norm_eps": 1e-5,
                                "tie_word_embeddings": False, "max_position_embeddings": 1 << 20, "rope_scaling": None,
                                "num_hidden_layers": 4}),
        }
        return base, kinds, near
    return {"w2048": shape(2048, 16, 4, 768, 256, 1024, 64, 64, 8192, 32000),
            "w4096": shape(4096, 32, 8, 1536, 512, 1024, 128, 128, 14336, 32000)}


def linonex_shapes():
    """Layer sizes that resemble real models' (random weights): Linonex models whose layers are all
    matrix memory or all parallel (chunked attention beside a delta rule), each with the dense and with the
    routed feed-forward, the mixed order, and the closest layers of the other decoders at the same width and
    heads: the Vametar decoder's gated linear attention (the matrix memory's heads), the Zirutar decoder's
    delta rule, the Saredra decoder's parallel layer with routed experts of the same sizes, and the Llama
    layer."""
    def shape(width, heads, kv, mem, mem_dim, chunk, experts, top, eff, ff, vocab):
        dense = {"kind": "dense", "ff": ff}
        moe = {"kind": "moe", "expert": {"ff": eff}, "router": {"experts": experts, "identity": experts // 8, "scale": 2.0, "top": top}}
        memory = {"heads": mem, "dim": mem_dim, "vdim": 2 * mem_dim, "gate_cap": 15.0}
        sides = {"left": {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128, "conv": 4, "scale": 128 ** -0.5,
                          "softcap": 30.0, "mask": {"size": chunk}},
                 "right": {"heads": heads, "kv_heads": heads, "dim": 128, "vdim": 128, "conv": 4}}
        lay = lambda kind, mlp: {"type": kind, "mlp": mlp, "mixer": memory if kind == "mlstm" else sides}
        base = {"architecture": "Linonex", "vocab": vocab, "width": width, "norm": {"eps": 1e-5}, "max_positions": 1 << 16}
        kinds = {"mlstm": [lay("mlstm", dense)] * 4, "parallel": [lay("parallel", dense)] * 4,
                 "mlstm_moe": [lay("mlstm", moe)] * 4, "parallel_moe": [lay("parallel", moe)] * 4,
                 "mixed": [lay("mlstm", dense), lay("parallel", moe), lay("parallel", dense), lay("mlstm", moe)]}
        sar = saredra_shapes()[f"w{width}"]
        smoe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": eff}}
        spar = {**sar[1]["parallel"][0], "mlp": smoe}
        zi = zirutar_shapes()[f"w{width}"]
        zdelta = {**zi[1]["delta"][0], "mlp": {**dense, "limit": 7.0}}
        vam = zi[2]["vametar_gla"][1]
        near = {
            "vametar_gla": ("Vametar", {**vam, "layers": [{"type": "gla", "mlp": dense, "mixer": {
                "heads": mem, "dim": mem_dim, "vdim": 2 * mem_dim, "tau": 16.0, "rank": 16}}] * 4}),
            "zirutar_delta": ("Zirutar", {**zi[0], "layers": [zdelta] * 4}),
            "saredra_parallel": ("Saredra", {**sar[0], "layers": [spar] * 4}),
            "llama": zi[2]["llama"],
        }
        return base, kinds, near
    return {"w2048": shape(2048, 16, 4, 8, 128, 1024, 32, 4, 1024, 8192, 32000),
            "w4096": shape(4096, 32, 8, 8, 256, 1024, 64, 6, 1408, 14336, 32000)}


def _routed_parts(model):
    return [b.ffn for b in model.blocks if getattr(getattr(b, "ffn", None), "spec", None) is not None
            and getattr(b.ffn.spec, "kind", "") == "routed_mlp"]


def _expert_entries(sp):
    """Matrix entries of one routed expert: up and down, and a gate matrix where it has one."""
    return (3 if getattr(sp, "form", "mlp") in ("limited_glu", "glu") else 2) * sp.hidden * sp.intermediate


def _leaf_mixers(m):
    """The mixers of a block: itself, or the branches of mixers that run side by side."""
    subs = getattr(m, "branches", None)
    return [m] if subs is None else [x for b in subs for x in _leaf_mixers(b)]


def generic_step_bytes(model, contexts):
    """What a single-token step reads and writes: every matrix once (of the embedding tables
    only rows), each sequence's keys and values, and its fixed-size state twice."""
    import torch
    from transformer_amd.cache.storage import KVNeed, StateNeed
    w = model.weight_bytes()
    skip = {model.w["embed"].data_ptr()}
    if model.w["embed"].data_ptr() != model.w["head"].data_ptr():
        w -= model.w["embed"].numel() * model.w["embed"].element_size()
    table = getattr(getattr(model, "after_embed", None), "w", {}).get("table")
    if table is not None and table.data_ptr() not in skip:
        w -= table.numel() * table.element_size()
    item = torch.empty((), dtype=model.dtype).element_size()
    per_token = per_seq = 0
    for need in model.cache_needs:
        if isinstance(need, KVNeed):
            per_token += need.num_kv_heads * (need.head_dim + need.value_dim) * item
        elif isinstance(need, StateNeed):
            n = 1
            for d in need.shape:
                n *= d
            per_seq += 2 * n * torch.empty((), dtype=need.dtype).element_size()
    for f in _routed_parts(model):       # of the experts only those that the step's tokens can reach
        sp = f.spec
        w -= max(0, sp.experts - len(contexts) * sp.top) * _expert_entries(sp) * item
    windowed = 0
    for need in model.cache_needs:       # a window (or chunk) bounds what a layer reads of a sequence
        if isinstance(need, KVNeed) and need.span is not None:
            windowed += sum(max(0, need.first_key(c) - need.keep_first) for c in contexts) * need.num_kv_heads * \
                (need.head_dim + need.value_dim) * item
    return w + sum(contexts) * per_token - windowed + len(contexts) * per_seq


def generic_prefill_flops(model, T):
    """2 * T * (entries of every matrix but the embedding tables) plus, for each attention
    layer, the causal score and value products."""
    from transformer_amd.cache.storage import KVNeed
    params = model.all_params()
    mats = sum(t.numel() for n, t in model.tensors.items()
               if params[n].role == "matrix" and n not in ("embed.weight", "head.weight", "after_embed.table"))
    mats -= sum(t.numel() for n, t in model.tensors.items() if n.endswith(".table"))
    for f in _routed_parts(model):       # a token goes through ``top`` of the experts
        sp = f.spec
        mats -= (sp.experts - sp.top) * _expert_entries(sp)
    fl = 2 * T * mats + 2 * model.spec.hidden * model.spec.vocab
    for m in (x for blk in model.blocks for x in _leaf_mixers(blk.mixer)):
        need = m.cache_need()
        need = need[0] if isinstance(need, (list, tuple)) and need else need
        if isinstance(need, KVNeed):
            window = getattr(m.spec, "window", None)
            pairs = T * (T + 1) // 2 if window is None or window >= T else window * (window + 1) // 2 + (T - window) * window
            chunk = getattr(m.spec, "chunk", None)
            if chunk is not None:
                pairs = T // chunk * (chunk * (chunk + 1) // 2) + (T % chunk) * (T % chunk + 1) // 2
            if hasattr(m, "nq"):
                fl += 2 * m.nq * (need.head_dim + need.value_dim) * pairs
            else:                        # one latent row per token: scores over its whole width, sums over the latent
                fl += 2 * m.H * (need.head_dim + m.spec.kv_rank) * pairs
    return fl


class _Vocab:
    def __init__(self, vocab):
        self.vocab = vocab


def _design_row(model, a, dkey):
    import torch
    cfg = _Vocab(model.spec.vocab)
    dt, ctx, _ = time_decode(model, cfg, a.batch, a.steps, a.warmup, 1, 512, 1024)
    nbytes = generic_step_bytes(model, ctx)
    pt = time_prefill(model, cfg, 3, 2, tokens=a.prefill_tokens)
    fl = generic_prefill_flops(model, a.prefill_tokens)
    return {"decode_tok_s": round(a.batch * a.steps / dt, 1),
            "decode_ms_per_step": round(dt / a.steps * 1e3, 4),
            "decode_gbs": round(nbytes / (dt / a.steps) / 1e9, 1),
            "decode_frac_hbm": round(nbytes / (dt / a.steps) / 1e9 / HBM_GBS, 4),
            "prefill_tok_s": round(a.prefill_tokens / pt, 1), "prefill_ms": round(pt * 1e3, 3),
            "prefill_frac_matrix_peak": round(fl / pt / (PEAK_TFLOPS[dkey] * 1e12), 4)}


def bench_kunitar(a):
    """Prefill and decode throughput of Kunitar models whose layers are all of one kind, and of
    the mixed order, beside the Llama decoder with layers of the same width, heads and dense
    feed-forward and the Vametar decoder's gated linear attention of the recurrence's heads.
    One JSON line of its own; the default workload is untouched."""
    import torch
    import transformer_amd as ta
    dkey = "bf16" if a.dtype == "bfloat16" else "fp32"
    layers = a.layers or 4
    out = {"design": "kunitar", "dtype": dkey, "layers": layers, "batch": a.batch,
           "prefill_tokens": a.prefill_tokens, "data": "synthetic", "sizes": {}}
    for size, (base, kinds, llama) in kunitar_shapes().items():
        if a.design_size and size not in a.design_size.split(","):
            continue
        llama = dict(llama)
        vametar_like = llama.pop("vametar_like")
        rows = {}
        cases = [("llama", None), ("vametar_gla", None)] + list(kinds.items())
        if a.design_case:
            cases = [c for c in cases if c[0] in a.design_case.split(",")]
        for name, lay in cases:
            if name == "llama":
                model = ta.random_model(ta.LlamaConfig.from_dict({**llama, "num_hidden_layers": layers}),
                                        seed=0, dtype=a.dtype)
            elif name == "vametar_gla":
                model = ta.random_model({**vametar_like, "layers": vametar_like["layers"] * layers}, seed=0,
                                        dtype=a.dtype, architecture="Vametar")
            else:
                lay = (lay * (-(-layers // len(lay))))[:layers]
                model = ta.random_model({**base, "layers": lay}, seed=0, dtype=a.dtype, architecture="Kunitar")
            rows[name] = _design_row(model, a, dkey)
            del model
            torch.cuda.empty_cache()
            print(f"[bench] {size} {name}: {rows[name]}", file=sys.stderr, flush=True)
        out["sizes"][size] = rows
    print(json.dumps(out))
    return 0


def bench_beside(a, design, architecture, shapes):
    """Prefill and decode throughput of a design's models, each of layers of one kind and of the mixed
    order (``shapes``: {size: (base configuration, {kind: layers}, {name: (architecture,
    configuration)} of the closest layers of the other decoders at the same width)}). One JSON line
    of its own; the default workload is untouched."""
    import torch
    import transformer_amd as ta
    dkey = "bf16" if a.dtype == "bfloat16" else "fp32"
    layers = a.layers or 4
    out = {"design": design, "dtype": dkey, "layers": layers, "batch": a.batch,
           "prefill_tokens": a.prefill_tokens, "data": "synthetic", "sizes": {}}

    def fit(lay):
        return (list(lay) * (-(-layers // len(lay))))[:layers]

    for size, (base, kinds, near) in shapes.items():
        if a.design_size and size not in a.design_size.split(","):
            continue
        cases = [(n, arch, c) for n, (arch, c) in near.items()] + \
                [(n, architecture, {**base, "layers": lay}) for n, lay in kinds.items()]
        if a.design_case:
            cases = [c for c in cases if c[0] in a.design_case.split(",")]
        rows = {}
        for name, arch, cfg in cases:
            if arch == "llama":
                model = ta.random_model(ta.LlamaConfig.from_dict({**cfg, "num_hidden_layers": layers}), seed=0, dtype=a.dtype)
            else:
                model = ta.random_model({**cfg, "layers": fit(cfg["layers"])}, seed=0, dtype=a.dtype, architecture=arch)
            rows[name] = _design_row(model, a, dkey)
            del model
            torch.cuda.empty_cache()
            print(f"[bench] {size} {name}: {rows[name]}", file=sys.stderr, flush=True)
        out["sizes"][size] = rows
    print(json.dumps(out))
    return 0


def bench_design(a):
    """Prefill and decode throughput of Vametar models whose layers are all of one kind, and
    of the mixed order, beside the Llama decoder with layers of the same width, heads and
    feed-forward. One JSON line of its own; the default workload is untouched."""
    import torch
    import transformer_amd as ta
    dkey = "bf16" if a.dtype == "bfloat16" else "fp32"
    layers = a.layers or 8
    out = {"design": "vametar", "dtype": dkey, "layers": layers, "batch": a.batch,
           "prefill_tokens": a.prefill_tokens, "data": "synthetic", "sizes": {}}
    for size, (base, kinds, llama) in vametar_shapes().items():
        if a.design_size and size not in a.design_size.split(","):
            continue
        rows = {}
        order = ["gla", "attention", "rglru", "attention", "gla"]
        cases = [("llama", None)] + [(k, [kinds[k]] * layers) for k in ("attention", "rglru", "gla")] + \
                [("mixed", [kinds[order[i % len(order)]] for i in range(layers)])]
        for name, lay in cases:
            if name == "llama":
                model = ta.random_model(ta.LlamaConfig.from_dict({**llama, "num_hidden_layers": layers}),
                                        seed=0, dtype=a.dtype)
            else:
                model = ta.random_model({**base, "layers": lay}, seed=0, dtype=a.dtype, architecture="Vametar")
            cfg = _Vocab(model.spec.vocab)
            dt, ctx, _ = time_decode(model, cfg, a.batch, a.steps, a.warmup, 1, 512, 1024)
            nbytes = generic_step_bytes(model, ctx)
            pt = time_prefill(model, cfg, 3, 2, tokens=a.prefill_tokens)
            fl = generic_prefill_flops(model, a.prefill_tokens)
            rows[name] = {"decode_tok_s": round(a.batch * a.steps / dt, 1),
                          "decode_ms_per_step": round(dt / a.steps * 1e3, 4),
                          "decode_gbs": round(nbytes / (dt / a.steps) / 1e9, 1),
                          "decode_frac_hbm": round(nbytes / (dt / a.steps) / 1e9 / HBM_GBS, 4),
                          "prefill_tok_s": round(a.prefill_tokens / pt, 1), "prefill_ms": round(pt * 1e3, 3),
                          "prefill_frac_matrix_peak": round(fl / pt / (PEAK_TFLOPS[dkey] * 1e12), 4)}
            del model
            torch.cuda.empty_cache()
            print(f"[bench] {size} {name}: {rows[name]}", file=sys.stderr, flush=True)
        out["sizes"][size] = rows
    print(json.dumps(out))
    return 0


def read_probe_gbs(device, nbytes=1 << 30, workgroups=2048, reps=5):
    """GB/s of a kernel that only reads: the machine's own ceiling for the weight streams of a
    decode step (the roofline of the line is the published 8 TB/s; this says how much of the
    distance to it is the memory system's)."""
    import torch
    from transformer_amd import kernels
    buf = torch.zeros(nbytes // 4, dtype=torch.int32, device=device)
    sink = torch.zeros(256, dtype=torch.int32, device=device)
    best = float("inf")
    for _ in range(reps + 1):
        e0, e1 = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        e0.record()
        kernels.read_probe(buf, workgroups, sink)
        e1.record()
        torch.cuda.synchronize()
        best = min(best, e0.elapsed_time(e1) * 1e-3)
    return nbytes / best / 1e9


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=128)
    ap.add_argument("--warmup", type=int, default=16)
    ap.add_argument("--batch", type=int, default=8)
    ap.add_argument("--layers", type=int, default=None, help="build fewer layers than the model has")
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float32"])
    ap.add_argument("--shape", default="8b", choices=sorted(SHAPES),
                    help="layer sizes: the headline model (8b), Llama-2-7B (7b) or Llama-3-70B (70b)")
    ap.add_argument("--prompt-min", type=int, default=None, help="shortest prompt of the decode batch")
    ap.add_argument("--prompt-max", type=int, default=None, help="longest prompt of the decode batch")
    ap.add_argument("--no-points", action="store_true", help="skip batch 1 and 64 and the prefill")
    ap.add_argument("--no-extra", action="store_true",
                    help="skip the further points (long context, other prompt lengths, the 7B shape)")
    ap.add_argument("--probe", action="store_true",
                    help="also measure what a kernel that only reads gets from this machine's memory "
                         "and add it to the line (\"probe\")")
    ap.add_argument("--prefill-tokens", type=int, default=PREFILL_TOKENS,
                    help="tokens of the prompt whose step is timed (the line's \"prefill\")")
    ap.add_argument("--prefill-only", action="store_true",
                    help="run only the 2,048-token prefill (for profiling); prints its own line")
    ap.add_argument("--design", default=None, choices=["vametar", "kunitar", "luduvik", "saredra", "zirutar", "linonex"],
                    help="instead of the default workload: prefill and decode of this design at a few "
                         "layer sizes, beside the Llama decoder at the same sizes (a line of its own)")
    ap.add_argument("--design-size", default=None, help="with --design: only these sizes (w2048,w4096)")
    ap.add_argument("--design-case", default=None, help="with --design kunitar, luduvik, saredra, zirutar or linonex: only these rows (llama,latent,...)")
    a = ap.parse_args()
    if a.design == "kunitar" and a.gpus == 1:
        return bench_kunitar(a)
    if a.design == "luduvik" and a.gpus == 1:
        return bench_beside(a, "luduvik", "Luduvik", luduvik_shapes())
    if a.design == "saredra" and a.gpus == 1:
        return bench_beside(a, "saredra", "Saredra", saredra_shapes())
    if a.design == "zirutar" and a.gpus == 1:
        return bench_beside(a, "zirutar", "Zirutar", zirutar_shapes())
    if a.design == "linonex" and a.gpus == 1:
        return bench_beside(a, "linonex", "Linonex", linonex_shapes())
    if a.design and a.gpus == 1:
        return bench_design(a)
    if a.gpus != 1:
        print(f"bench.py measures one GPU; --gpus {a.gpus} is not supported by this engine")
        return 2
    import torch
    import transformer_amd as ta
    shape_name, shape = SHAPES[a.shape]
    if a.prompt_min is None:
        a.prompt_min = PROMPTS[a.shape][0]
    if a.prompt_max is None:
        a.prompt_max = max(PROMPTS[a.shape][1], a.prompt_min)
    # longer prompts than the shape's context are a measurement of their own: let positions reach them
    room = max(a.prompt_max + 2 * (a.steps + a.warmup) + 8, a.prefill_tokens)
    if a.shape == "8b" and not (a.no_points or a.no_extra or a.prefill_only):
        room = max(room, 8192 + 64)          # the further points reach 8 k tokens
    shape = {**shape, "max_position_embeddings": max(shape["max_position_embeddings"], room)}
    cfg = ta.LlamaConfig.from_dict(shape)
    layers = a.layers or cfg.num_layers
    model = ta.random_model(cfg, seed=0, dtype=a.dtype, num_layers=layers)
    mcfg = model.config
    torch.cuda.synchronize()
    dkey = "bf16" if a.dtype == "bfloat16" else "fp32"

    if a.prefill_only:
        pt = time_prefill(model, mcfg, reps=max(1, a.steps), seed=2, tokens=a.prefill_tokens)
        fl = prefill_flops(mcfg, a.prefill_tokens)
        print(json.dumps({"prefill_ms": round(pt * 1e3, 3), "tokens": a.prefill_tokens,
                          "tok_per_s": round(a.prefill_tokens / pt, 1),
                          "frac": round(fl / pt / (PEAK_TFLOPS[dkey] * 1e12), 4)}))
        return 0
    main_point = decode_point(model, mcfg, a.batch, a.steps, a.warmup, 1, a.prompt_min, a.prompt_max)
    line = {
        "metric": f"decode tok/s @ batch {a.batch}; {shape_name} shape", "value": main_point["tok_s"],
        "unit": "tok/s", "n_gpus": 1, "steps": a.steps, "warmup": a.warmup,
        "ms_per_step": main_point["ms_per_step"], "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": dkey, "data": "synthetic",
        "config": {"model": f"{shape_name} shape, random weights N(0,0.02)",
                   "layers": layers, "layers_of_model": cfg.num_layers, "hidden": cfg.hidden,
                   "heads": cfg.num_heads, "kv_heads": cfg.num_kv_heads, "head_dim": cfg.head_dim,
                   "intermediate": cfg.intermediate, "vocab": cfg.vocab,
                   "rope_theta": cfg.rope_theta, "rms_eps": cfg.rms_eps,
                   "global_batch": a.batch, "seq_len": max(CONTEXT, a.prompt_max + a.steps + a.warmup),
                   "prompt_min": a.prompt_min, "prompt_max": a.prompt_max,
                   "mean_context": main_point["mean_context"],
                   "prefill_tokens": a.prefill_tokens, "parallelism": "single GPU",
                   "sampling": "greedy", "loop": "engine.generate.run_batches"},
        "roofline": {"bound": "hbm", "achieved": main_point["gbs"], "peak": HBM_GBS,
                     "unit": "GB/s", "frac": main_point["frac"]},
        "loop_tok_s": main_point["loop_tok_s"],
    }
    if a.probe:
        gbs = read_probe_gbs(model.device)
        line["probe"] = {"read_gbs": round(gbs, 1), "achieved_of_read": round(main_point["gbs"] / gbs, 4),
                         "what": "1 GiB read by 2048 workgroups with non-temporal loads, best of 5"}
    if not a.no_points:
        line["prefill"] = prefill_point(model, mcfg, dkey, 5, 2, tokens=a.prefill_tokens)
        # every point with what its roofline needs, flat: tokens a second under the point's
        # name, then <name>_ms (a step), _ctx (mean context), _gbs and _frac (of the HBM peak;
        # prefill points: of the matrix cores' peak)
        points = {}

        def add_decode(name, pt):
            points[name] = pt["tok_s"]
            points[name + "_ms"], points[name + "_ctx"] = pt["ms_per_step"], pt["mean_context"]
            points[name + "_gbs"], points[name + "_frac"] = pt["gbs"], pt["frac"]

        def add_prefill(name, pt):
            points[name] = pt["value"]
            points[name + "_ms"], points[name + "_tokens"], points[name + "_frac"] = pt["ms"], pt["tokens"], pt["frac"]

        few, short = max(16, a.steps // 2), max(4, a.warmup // 2)
        for b in (1, 64):
            add_decode(f"decode_b{b}", decode_point(model, mcfg, b, few, short, 3 + b, a.prompt_min, a.prompt_max))
        if not a.no_extra and a.shape == "8b":
            import numpy as np
            # a long context, short and long prompts, many short prompts in one step
            add_decode("decode_b8_ctx8k", decode_point(model, mcfg, 8, 16, 4, 11, 7000, 8000))
            add_prefill("prefill_512", prefill_point(model, mcfg, dkey, 5, 12, tokens=512))
            add_prefill("prefill_8192", prefill_point(model, mcfg, dkey, 3, 13, tokens=8192))
            mixed = [int(x) for x in np.random.default_rng(14).integers(32, 257, 16)]
            add_prefill("prefill_16_prompts_32_to_256", prefill_point(model, mcfg, dkey, 5, 14, lengths=mixed))
            # the Llama-2-7B shape (every head has keys of its own: four times the cache per token)
            del model
            torch.cuda.empty_cache()
            name7, shape7 = SHAPES["7b"]
            cfg7 = ta.LlamaConfig.from_dict(shape7)
            model = ta.random_model(cfg7, seed=0, dtype=a.dtype,
                                    num_layers=min(layers, cfg7.num_layers) if a.layers else None)
            add_decode("llama2_7b_decode_b16", decode_point(model, model.config, 16, 16, 4, 15, *PROMPTS["7b"]))
        line["points"] = points
    print(json.dumps(line))
    return 0


if __name__ == "__main__":
    sys.exit(main())
