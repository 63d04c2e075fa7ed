"""Fixtures of the Riruzen tests: small configurations, checkpoints on
disk and engines over them."""

import json
import os
import tempfile

import torch

import riruzen_plain as plain
from resilient_llm_amd.engine import LLMEngine, PagedKVCache
from resilient_llm_amd.models import build_model, get_config


def lat(heads, dim, vdim, q_rank, kv_rank, scale=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank,
            "kv_rank": kv_rank,
            "scale": dim ** -0.5 if scale is None else scale}


def rec(heads, dim, vdim):
    return {"heads": heads, "dim": dim, "vdim": vdim}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


# sizes that are nobody's favourite multiples, a layer without feed-forward
ODD = plain.make_config([
    layer("hgrn2", rec(3, 20, 18), dense(41)),
    layer("latent_attention", lat(5, 12, 22, 19, 27), dense(70)),
    layer("latent_attention", lat(3, 9, 7, 14, 36, scale=0.21), None),
    layer("hgrn2", rec(1, 33, 50), None),
], width=78, vocab=101, groups=3, taps=3, eps=1e-4, logit_scale=1.7)

# sizes that the tiled kernels take; many heads on few latents
EVEN = plain.make_config([
    layer("latent_attention", lat(4, 64, 96, 56, 128), dense(160)),
    layer("hgrn2", rec(2, 128, 160), dense(64)),
    layer("hgrn2", rec(5, 64, 40), None),
    layer("latent_attention", lat(36, 16, 24, 72, 40), dense(96)),
], width=160, vocab=200, groups=5, taps=4, eps=1e-6, logit_scale=0.25)

# one norm group, one tap (no state at all), attention only
ATTN_ONLY = plain.make_config([
    layer("latent_attention", lat(2, 16, 32, 24, 64), dense(48)),
    layer("latent_attention", lat(20, 24, 16, 40, 24), dense(56)),
], width=40, vocab=64, groups=1, taps=1, logit_scale=1.0)

# recurrent only, a long convolution
REC_ONLY = plain.make_config([
    layer("hgrn2", rec(2, 16, 24), None),
    layer("hgrn2", rec(2, 48, 16), dense(40)),
], width=48, vocab=80, groups=4, taps=6)

CONFIGS = {"odd": ODD, "even": EVEN, "attn": ATTN_ONLY, "rec": REC_ONLY}

_ckpts: dict = {}
_models: dict = {}
_plain: dict = {}


def checkpoint(config, seed=0, edit=None):
    """(directory, weights) of a random checkpoint of ``config``."""
    key = (json.dumps(config, sort_keys=True), seed)
    if edit is None and key in _ckpts:
        return _ckpts[key]
    import safetensors.torch as st
    w = plain.random_weights(config, seed)
    if edit is not None:
        edit(w)
    d = tempfile.mkdtemp(prefix="riruzen-")
    st.save_file(w, os.path.join(d, "model.safetensors"))
    with open(os.path.join(d, "config.json"), "w") as f:
        json.dump(config, f)
    if edit is None:
        _ckpts[key] = (d, w)
    return d, w


def make_engine(config, device, dtype, seed=0, blocks=64, slots=4, edit=None,
                kv_dtype=None, **kw):
    d, w = checkpoint(config, seed, edit)
    key = (d, device, dtype)
    if key not in _models:
        _models[key] = build_model(get_config(d), weights=d, device=device,
                                   dtype=dtype)
    model = _models[key]
    kv = PagedKVCache.for_model(model.config, blocks, device=device,
                                kv_dtype=kv_dtype or dtype, state_slots=slots)
    # whatever was never written must never be read
    for i, x in enumerate(config["layers"]):
        held = []
        if x["type"] == "latent_attention":
            held += kv.layer(i) if kv_dtype is None else ()
        else:
            held.append(kv.states.layer(i))
        if config["canon"]["taps"] > 1:
            held.append(kv.states.tail(i))
        for t in held:
            t.fill_(float("nan"))
    return LLMEngine(model, kv, **kw), w


def expected(config, w, tokens):
    key = (id(w), tuple(tokens))
    if key not in _plain:
        _plain[key] = (plain.run(config, w, tokens)[0], w)
    return _plain[key][0]
