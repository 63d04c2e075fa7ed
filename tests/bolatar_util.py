"""Fixtures of the Bolatar tests: small configurations, checkpoints on
disk and engines over them."""

import json
import os
import tempfile

import torch

import bolatar_plain as plain
from resilient_llm_amd.engine import LLMEngine, PagedKVCache
from resilient_llm_amd.models import build_model, get_config


def delta(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "conv": conv}


def mlstm(heads, dim, vdim, cap):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def parallel(heads, kv_heads, dim, vdim, rec_heads, rec_dim, coef=0.3,
             every=16, scale=None):
    return {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": vdim,
                     "scale": dim ** -0.5 if scale is None else scale,
                     "q_temp": {"coef": coef, "every": every}},
            "right": {"heads": rec_heads, "dim": rec_dim}}


def dense(ff, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


# sizes that are nobody's favourite multiples
ODD = plain.make_config([
    layer("parallel", parallel(3, 1, 20, 28, 2, 18, every=7), dense(41)),
    layer("delta", delta(3, 1, 20, 18, 4), dense(70, 0.6)),
    layer("mlstm", mlstm(3, 22, 17, 4.0), None),
    layer("delta", delta(2, 2, 33, 50, 1), None),
    layer("parallel", parallel(5, 5, 9, 7, 3, 5, coef=1.0, every=1,
                               scale=0.21), None),
], width=78, vocab=101, eps=1e-4, scale=1.6, softcap=5.0)

# sizes that the tiled kernels take
EVEN = plain.make_config([
    layer("mlstm", mlstm(2, 64, 96, 15.0), dense(64, 7.0)),
    layer("parallel", parallel(8, 2, 64, 96, 2, 64, every=50), dense(96)),
    layer("delta", delta(4, 2, 128, 64, 2), None),
    layer("parallel", parallel(4, 4, 32, 128, 1, 128, every=1000),
          dense(160)),
    layer("mlstm", mlstm(1, 128, 144, 3.0), dense(48)),
    layer("delta", delta(6, 1, 64, 80, 5), dense(56)),
], width=128, vocab=200, eps=1e-6)

# no layer with keys and values
REC_ONLY = plain.make_config([
    layer("delta", delta(2, 1, 16, 24, 6), None),
    layer("mlstm", mlstm(2, 48, 16, 8.0), dense(40)),
], width=48, vocab=80)

CONFIGS = {"odd": ODD, "even": EVEN, "rec": REC_ONLY}

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
    d = tempfile.mkdtemp(prefix="bolatar-")
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
        held = [kv.states.layer(i)]
        if x["type"] == "parallel":
            held += kv.layer(i) if kv_dtype is None else ()
        if x["type"] == "mlstm":
            held.append(kv.states.scalar(i))
        if kv.states.tail(i) is not None:
            held.append(kv.states.tail(i))
        for t in held:
            t.fill_(float("nan"))
    return LLMEngine(model, kv, **kw), w


def expected(config, w, tokens):
    key = (id(w), tuple(tokens))
    if key not in _plain:
        _plain[key] = (plain.run(config, w, tokens)[0], w)
    return _plain[key][0]
