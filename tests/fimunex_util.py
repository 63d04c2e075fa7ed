"""Fixtures of the Fimunex tests: small configurations, checkpoints on
disk and engines over them."""

import json
import os
import tempfile

import torch

import fimunex_plain as plain
from nesizen_util import F32
from resilient_llm_amd.engine import LLMEngine, PagedKVCache
from resilient_llm_amd.models import build_model, get_config


def att(heads, kv_heads, dim, vdim, chunk, rot=None, base=1000.0, factor=2.0,
        original=64, fast=4.0, slow=0.5, scale=None, softcap=12.0, diff=0.4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "diff": diff, "mask": {"size": chunk}, "softcap": softcap,
            "scale": dim ** -0.5 if scale is None else scale,
            "rot": {"dims": dim if rot is None else rot, "base": base,
                    "scaling": {"factor": factor, "original": original,
                                "fast": fast, "slow": slow}}}


def moe(experts, identity, top, ff, count=1, keep=1):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "identity": identity, "top": top,
                       "groups": {"count": count, "keep": keep}}}


def layer(mixer, mlp):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


# sizes that are nobody's favourite multiples
ODD = plain.make_config([
    layer(att(3, 1, 10, 14, 21, rot=6), moe(5, 1, 3, 23, 3, 2)),
    layer(att(2, 2, 9, 33, 64, rot=4, softcap=3.0), None),
    layer(att(5, 1, 18, 18, 7, rot=18, factor=1.0, diff=0.0),
          moe(3, 0, 1, 41)),
], width=42, vocab=101, eps=1e-4, taps=2, softcap=5.0, loop=(0, 2, 3))

# sizes that the tiled kernels take
EVEN = plain.make_config([
    layer(att(8, 2, 32, 64, 50), moe(6, 2, 2, 64, 2, 1)),
    layer(att(4, 4, 64, 48, 33, rot=32, factor=6.0), moe(4, 4, 3, 96, 8, 5)),
    layer(att(6, 1, 16, 136, 16, rot=16, diff=0.7), None),
    layer(att(10, 1, 48, 32, 100, rot=32), moe(7, 1, 4, 40, 4, 3)),
], width=128, vocab=200, eps=1e-6, taps=5, loop=(1, 3, 2))

# no convolution over time, every expert, a chunk of one
PLAIN = plain.make_config([
    layer(att(2, 1, 16, 8, 1), moe(2, 1, 3, 24)),
    layer(att(1, 1, 24, 40, 1000, rot=8), moe(1, 0, 1, 30)),
], width=40, vocab=64, taps=1, loop=(1, 2, 1))

CONFIGS = {"odd": ODD, "even": EVEN, "plain": PLAIN}

_ckpts: dict = {}
_models: dict = {}
_plain: dict = {}


def checkpoint(config, seed=0, decisive=False, edit=None):
    """(directory, weights) of a random checkpoint of ``config``."""
    key = (json.dumps(config, sort_keys=True), seed, decisive)
    if edit is None and key in _ckpts:
        return _ckpts[key]
    import safetensors.torch as st
    w = plain.random_weights(config, seed, decisive)
    if edit is not None:
        edit(w)
    d = tempfile.mkdtemp(prefix="fimunex-")
    st.save_file(w, os.path.join(d, "model.safetensors"))
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(config, f)
    if edit is None:
        _ckpts[key] = (d, w)
    return d, w


def make_engine(config, device, dtype, seed=0, blocks=64, slots=4, edit=None,
                kv_dtype=None, **kw):
    """At 16 bits a router's close call may fall either way after rounding:
    those checkpoints decide theirs by far."""
    d, w = checkpoint(config, seed, dtype != F32, edit)
    key = (d, device, dtype)
    if key not in _models:
        cfg = get_config(d)
        cfg.fit_positions(2048)
        _models[key] = build_model(cfg, weights=d, device=device, dtype=dtype)
    model = _models[key]
    kv = PagedKVCache.for_model(model.config, blocks, device=device,
                                kv_dtype=kv_dtype or dtype, state_slots=slots)
    # whatever was never written must never be read
    for n, (_, which) in enumerate(model.config.sublayers):
        held = list(kv.layer(n)) if which == "mix" and kv_dtype is None \
            else []
        if kv.states is not None:
            held.append(kv.states.tail(n))
        for t in held:
            t.fill_(float("nan"))
    return LLMEngine(model, kv, **kw), w


def expected(config, w, tokens):
    key = (id(w), tuple(tokens))
    if key not in _plain:
        _plain[key] = (plain.run(config, w, tokens)[0], w)
    return _plain[key][0]
