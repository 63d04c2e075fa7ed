"""Fimunex through the engine against the plain implementation: whole
prompts, token by token, portions, mixed batches, reused pages and slots,
loops, generation, graphs, migration, tensor parallelism, replay."""

import copy
import json
import os
import subprocess
import sys

import pytest
import torch

import fimunex_plain as plain
from fimunex_util import (
    CONFIGS, EVEN, ODD, PLAIN, att, checkpoint, expected, layer, make_engine,
    moe,
)
from nesizen_util import (
    BF16, F32, GPU, TARGETS, check, cut, feed_portions, row_errors, tokens_of,
)
from resilient_llm_amd.engine import LLMEngine, PagedKVCache, SamplingParams
from resilient_llm_amd.models import build_model, get_config

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt(name, device, dtype):
    config = CONFIGS[name]
    e, w = make_engine(config, device, dtype)
    for n, seed in ((1, 1), (2, 2), (97, 3), (150, 4)):
        t = tokens_of(config, n, seed)
        check(feed_portions(e, t, [n]), expected(config, w, t), dtype,
              f"{n} tokens")
    assert e.kv.free_blocks == e.kv.num_blocks


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_token_by_token(name, device, dtype):
    """Decoding from the first token on, over every chunk's edge."""
    config = CONFIGS[name]
    e, w = make_engine(config, device, dtype)
    t = tokens_of(config, 150, 4)
    check(feed_portions(e, t, [1] * len(t)), expected(config, w, t), dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("sizes", [[2], [3, 5], [16], [17, 2, 1, 31],
                                   [64, 1, 65]],
                         ids=lambda s: "-".join(map(str, s)))
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions(name, sizes, device, dtype):
    config = CONFIGS[name]
    e, w = make_engine(config, device, dtype)
    t = tokens_of(config, 150, 4)
    check(feed_portions(e, t, cut(len(t), sizes)), expected(config, w, t),
          dtype)


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_reuse_pages_and_slots(name, device, dtype):
    """Unequal requests, portions beside single tokens, requests that sit
    out steps, more requests than slots over time, a pool that only fits
    the live ones."""
    config = CONFIGS[name]
    lens = [97, 150, 1, 33, 2, 64, 49, 17]
    e, w = make_engine(config, device, dtype, blocks=24, slots=3)
    reqs = {f"r{i}": tokens_of(config, n, 20 + i) for i, n in enumerate(lens)}
    waiting, pos, got = list(reqs), {}, {r: [] for r in reqs}
    sizes = [1, 40, 2, 1, 17, 1, 1, 64, 3]
    step = 0
    while waiting or pos:
        while waiting and len(pos) < 3:
            pos[waiting.pop(0)] = 0
        entries, end = [], []
        for k, rid in enumerate(list(pos)):
            if len(pos) > 1 and (step + k) % 5 == 4:
                continue                           # sits this step out
            n = min(sizes[(step * 2 + k) % len(sizes)],
                    len(reqs[rid]) - pos[rid])
            entries.append((rid, reqs[rid][pos[rid]:pos[rid] + n], range(n)))
            pos[rid] += n
            if pos[rid] == len(reqs[rid]):
                end.append(rid)
                del pos[rid]
        logits = e.feed(entries, end)
        row = 0
        for rid, toks, _ in entries:
            got[rid].append(logits[row:row + len(toks)])
            row += len(toks)
        step += 1
    for rid, t in reqs.items():
        check(torch.cat(got[rid]), expected(config, w, t), dtype, rid)
    assert e.kv.free_blocks == e.kv.num_blocks
    if e.states is not None:
        assert e.states.free_slots == 3


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("config", [ODD, EVEN], ids=["odd", "even"])
def test_residual_after_every_layer(config, device, dtype):
    """Where a difference comes from: models cut off after each layer that
    runs, the loop written out."""
    t = tokens_of(config, 40, 6)
    _, w = checkpoint(config, decisive=dtype != F32)
    _, after = plain.run(config, w, t)
    order = plain.layer_order(config)
    for n in range(len(order)):
        part = dict(config, layers=[config["layers"][i]
                                    for i in order[:n + 1]],
                    loop={"start": 0, "stop": 0, "times": 1})

        def same(weights):
            for k in weights:
                head, _, rest = k.partition(".")
                if head[1:].isdigit():
                    k_from = f"l{order[int(head[1:])]}.{rest}"
                else:
                    k_from = k
                weights[k] = w[k_from].clone()
        e, _ = make_engine(part, device, dtype, edit=same)
        h = plain.rms(after[n], config["norm"]["eps"]) \
            * (1 + w["final.norm"].double())
        want = plain.soft_cap(h @ w["head"].double().T,
                              config["logit_softcap"])
        check(feed_portions(e, t, [30, 1, 9]), want, dtype, f"run {n}")


@pytest.mark.parametrize("loop", [(0, 0, 1), (0, 3, 1), (0, 1, 4), (1, 3, 2),
                                  (2, 3, 2), (0, 3, 2)])
def test_every_pass_of_a_loop_has_its_own_cache(loop):
    config = plain.make_config(
        [layer(att(2, 1, 8, 8, 40), moe(3, 1, 2, 16)),
         layer(att(2, 1, 8, 8, 40), None),
         layer(att(1, 1, 12, 6, 40), moe(2, 0, 1, 16))],
        width=24, vocab=50, loop=loop)
    e, w = make_engine(config, "cpu", F32)
    t = tokens_of(config, 60, 2)
    check(feed_portions(e, t, [30, 1, 1, 2, 26]), expected(config, w, t), F32)
    cfg = e.model.config
    assert cfg.order == plain.layer_order(config)
    assert len(cfg.cache_layers()) == len(cfg.sublayers)


def _finder(chunk, dim=32, heads=2):
    """A model whose attention asks for token 7: its keys answer every
    query, in map 1 only, over all other tokens of the chunk."""
    config = plain.make_config(
        [layer(att(heads, 1, dim, 32, chunk, rot=8, scale=1.0, softcap=20.0,
                   diff=0.2), None)], width=64, vocab=60)

    def sharp(w):
        w["embed"][:, :2] = 0
        w["embed"][7, 0] = 40.0
        w["embed"][:, 1] = 4.0
        w["l0.norm1"].zero_()
        w["l0.canon1"].zero_()
        for x in "qk":
            w[f"l0.mix.{x}"] *= 0.05
            w[f"l0.mix.{x}.b"] *= 0.05
            w[f"l0.mix.{x}.norm"].fill_(1.0)
        # beyond the rotated dimensions, so that distance does not matter
        w["l0.mix.q"].view(heads, 2, dim, 64)[:, 0, 12, 1] = 2.0
        w["l0.mix.k"].view(1, 2, dim, 64)[:, 0, 12, 0] = 2.0
    return config, sharp


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_a_far_token_shows(device, dtype):
    """Changing a token hundreds back in the chunk changes the answer, and
    every cut finds it."""
    config, sharp = _finder(1024)
    e, w = make_engine(config, device, dtype, edit=sharp)
    t = [x if x != 7 else 8 for x in tokens_of(config, 700, 5)]
    quiet = expected(config, w, t)
    t[17] = 7
    want = expected(config, w, t)
    assert float(row_errors(want[400:], quiet[400:]).median()) > 0.2
    for sizes in ([700], [640] + [1] * 60, [300, 2, 100, 5]):
        check(feed_portions(e, t, cut(700, sizes)), want, dtype, str(sizes))


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("chunk", [48, 64, 70])
def test_the_chunks_first_token_is_seen_and_the_last_ones_is_not(
        chunk, device, dtype):
    """A loud token just inside and one just outside of a chunk's edge."""
    config, sharp = _finder(chunk)
    e, w = make_engine(config, device, dtype, edit=sharp)
    base = [x if x != 7 else 8 for x in tokens_of(config, 3 * chunk + 5, 5)]
    for at in (chunk - 1, chunk, 2 * chunk - 1, 2 * chunk):
        t = list(base)
        t[at] = 7
        want, quiet = expected(config, w, t), expected(config, w, base)
        far = row_errors(want, quiet)
        after = slice(at + 1, (at // chunk + 1) * chunk)
        if after.stop > after.start:
            assert float(far[after].median()) > 0.1
        assert float(far[after.stop:].max()) < 1e-9
        n = len(t)
        for sizes in ([n], [chunk - 1, 2], [chunk + 1, 1, 1],
                      [chunk - 3] + [1] * (n - chunk + 3)):
            check(feed_portions(e, t, cut(n, sizes)), want, dtype,
                  f"{at} {sizes[:3]}")


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_wanted_places_and_their_order(device, dtype):
    e, w = make_engine(ODD, device, dtype)
    a, b = tokens_of(ODD, 20, 1), tokens_of(ODD, 9, 2)
    assert e.feed([("a", a[:8], []), ("b", b[:4], [])]).shape[0] == 0
    got = e.feed([("b", b[4:5], [0]), ("a", a[8:], [11, 0, 3])])
    wa, wb = expected(ODD, w, a), expected(ODD, w, b)
    check(got, torch.stack([wb[4], wa[19], wa[8], wa[11]]), dtype)


def _greedy_plain(config, w, prompt, n):
    t = list(prompt)
    for _ in range(n):
        t.append(int(plain.run(config, w, t)[0][-1].argmax()))
    return t[len(prompt):]


def _drain(e, max_steps=500):
    outs = {}
    for _ in range(max_steps):
        if not e.has_work():
            return outs
        for o in e.step():
            outs.setdefault(o.req_id, []).append(o.token_id)
    raise AssertionError("engine did not finish")


GREEDY = plain.make_config([
    layer(att(2, 1, 16, 24, 20), moe(4, 2, 2, 40, 2, 1)),
    layer(att(3, 3, 8, 16, 33, rot=4), moe(3, 0, 2, 24)),
], width=48, vocab=61, loop=(0, 1, 2))

DEVICE = pytest.mark.parametrize(
    "device", ["cpu", pytest.param("cuda:0", marks=GPU)])


@DEVICE
def test_greedy_generation(device):
    """add_request/step: admission, chunked prompts, mixed steps, state
    slots fewer than requests."""
    e, w = make_engine(GREEDY, device, F32, slots=2, chunk_size=7)
    prompts = {f"g{i}": tokens_of(GREEDY, n, 50 + i)
               for i, n in enumerate([23, 5, 40, 1])}
    for rid, p in prompts.items():
        e.add_request(rid, p, SamplingParams(max_tokens=12,
                                             stop_on_eos=False))
    outs = _drain(e)
    for rid, p in prompts.items():
        assert outs[rid] == _greedy_plain(GREEDY, w, p, 12), rid
    assert e.kv.free_blocks == e.kv.num_blocks
    assert e.states.free_slots == 2


@DEVICE
def test_long_generation(device):
    """Far past the prompt, over many pages and chunks."""
    e, w = make_engine(GREEDY, device, F32)
    p = tokens_of(GREEDY, 9, 3)
    e.add_request("l", p, SamplingParams(max_tokens=300, stop_on_eos=False))
    out = _drain(e)["l"]
    full = plain.run(GREEDY, w, p + out)[0]
    assert out == full[len(p) - 1:-1].argmax(-1).tolist()


@DEVICE
def test_sampled_generation_is_reproducible(device):
    runs = []
    for _ in range(2):
        e, _ = make_engine(GREEDY, device, F32)
        e.add_request("s", tokens_of(GREEDY, 9, 1), SamplingParams(
            max_tokens=15, temperature=0.8, seed=5))
        e.add_request("p", tokens_of(GREEDY, 4, 2), SamplingParams(
            max_tokens=15, temperature=0.9, top_p=0.7, seed=6))
        runs.append(_drain(e))
    assert runs[0] == runs[1]
    assert all(0 <= t < 61 for t in runs[0]["s"] + runs[0]["p"])


@GPU
@pytest.mark.parametrize("dtype", [F32, BF16], ids=["f32", "bf16"])
@pytest.mark.parametrize("config", [GREEDY, EVEN, PLAIN],
                         ids=["small", "even", "plain"])
def test_decode_graph_matches_eager(config, dtype):
    """Whole-step graphs (padded lanes, reloads, many replays) give what
    the same kernels give eagerly."""
    from resilient_llm_amd.engine.graph import install_graph_runner
    got = []
    for graphs in (False, True):
        e, _ = make_engine(config, "cuda:0", dtype, slots=9, blocks=128,
                           max_batch_size=8, enable_prefix_caching=False)
        if graphs:
            install_graph_runner(e, max_blocks_per_seq=16)
        for i, n in enumerate([30, 3, 61, 12, 7]):
            e.add_request(f"q{i}", tokens_of(config, n, i), SamplingParams(
                max_tokens=20 + 11 * i, stop_on_eos=False))
        outs = {}
        while e.has_work():
            for o in e.step():
                outs.setdefault(o.req_id, []).append(o.token_id)
            torch.cuda.synchronize()
        got.append(outs)
    if dtype == F32:
        assert got[0] == got[1]
        return
    # the split over keys follows the width of the block table, so at 16
    # bits a near tie may fall either way: nearly all tokens agree
    for rid, want in got[0].items():
        assert len(got[1][rid]) == len(want)
    same = sum(a == b for r in got[0] for a, b in zip(got[0][r], got[1][r]))
    assert same > 0.6 * sum(map(len, got[0].values()))


@GPU
def test_capture_after_another_runner_was_dropped():
    """An engine and its graph runner refer to each other, so a dropped pair
    waits for the garbage collector, which must not find it while the next
    runner captures."""
    import gc
    from resilient_llm_amd.engine.graph import install_graph_runner
    was = gc.get_threshold()
    got = []
    try:
        for _ in range(3):
            gc.set_threshold(20)
            e, _ = make_engine(GREEDY, "cuda:0", F32, max_batch_size=2)
            install_graph_runner(e, max_blocks_per_seq=8)
            e.add_request("r", tokens_of(GREEDY, 9, 1), SamplingParams(
                max_tokens=8, stop_on_eos=False))
            got.append(_drain(e))
            gc.set_threshold(100000)     # the pair stays until the next one
            del e
    finally:
        gc.set_threshold(*was)
    assert got[0] == got[1] == got[2]


def test_abort_and_capacity_return_state():
    e, _ = make_engine(GREEDY, "cpu", F32, slots=2, blocks=8)
    for rid in "ab":
        e.add_request(rid, tokens_of(GREEDY, 20, 1),
                      SamplingParams(max_tokens=40, stop_on_eos=False))
    e.step()
    e.step()
    assert e.states.free_slots == 0
    e.abort("a")
    _drain(e)
    assert e.states.free_slots == 2
    assert e.kv.free_blocks == 8


@DEVICE
def test_live_migration_carries_the_whole_state(device):
    prompt = tokens_of(GREEDY, 19, 7)
    sp = SamplingParams(max_tokens=16, stop_on_eos=False)
    ref, _ = make_engine(GREEDY, device, F32)
    ref.add_request("m", prompt, sp)
    want = _drain(ref)["m"]
    src, _ = make_engine(GREEDY, device, F32)
    dst, _ = make_engine(GREEDY, device, F32)
    dst.feed([("other", tokens_of(GREEDY, 30, 8), [])])     # occupy slot 0
    src.add_request("m", prompt, sp)
    got = []
    for _ in range(6):
        got += [o.token_id for o in src.step()]
    src.request_extract("m")
    got += [o.token_id for o in src.step()]
    state = src.take_extracted("m")
    # three passes, each with a tail ahead of either sublayer
    assert set(state["recurrent"]["tails"]) == set(range(6))
    assert src.kv.free_blocks == src.kv.num_blocks
    dst.queue_adopt(state)
    got += _drain(dst)["m"]
    assert dst.take_adopt_result("m") == "ok"
    assert got == want


def test_state_rules_out_prefix_cache_and_speculation():
    e, _ = make_engine(GREEDY, "cpu", F32)
    assert not e.enable_prefix_caching
    with pytest.raises(ValueError, match="spec_lookup"):
        make_engine(GREEDY, "cpu", F32, spec_lookup=3)


def test_a_model_without_taps_keeps_both():
    e, w = make_engine(PLAIN, "cpu", F32, spec_lookup=3)
    assert e.enable_prefix_caching and e.states is None
    p = tokens_of(PLAIN, 20, 3) * 2
    for rid in "ab":                     # the second finds cached blocks
        e.add_request(rid, p, SamplingParams(max_tokens=8,
                                             stop_on_eos=False))
        assert _drain(e)[rid] == _greedy_plain(PLAIN, w, p, 8)
    assert e.kv.prefix_hits > 0


@GPU
def test_fp8_cache_runs_and_stays_near():
    e, w = make_engine(EVEN, "cuda:0", BF16, kv_dtype=torch.float8_e4m3fn)
    t = tokens_of(EVEN, 120, 5)
    got = feed_portions(e, t, [70, 1, 1, 1, 30] + [1] * 17)
    assert float(row_errors(got, expected(EVEN, w, t)).median()) < 0.15


# ------------------------------------------------------------ integration
def test_registry_picks_the_class_by_config():
    from resilient_llm_amd.models import (
        FimunexForCausalLM, get_model_class, model_names,
    )
    d, _ = checkpoint(GREEDY)
    assert get_model_class(d) is FimunexForCausalLM
    assert get_model_class("tiny", d) is FimunexForCausalLM
    assert get_model_class("fimunex-tiny") is FimunexForCausalLM
    assert {"fimunex-tiny", "fimunex-2b"} <= set(model_names())


@pytest.mark.parametrize("model", ["fimunex-tiny", "checkpoint"])
def test_worker_serves_it(model):
    import asyncio

    from resilient_llm_amd.workers.base import GenerationRequest
    from resilient_llm_amd.workers.engine_worker import EngineWorker
    name = model if model != "checkpoint" else checkpoint(
        dict(GREEDY, vocab=300))[0]
    w = EngineWorker(device="cpu", model_name=name, num_blocks=64,
                     max_batch_size=3)
    try:
        async def go():
            reqs = [GenerationRequest(
                request_id=f"r{i}", model=name, max_tokens=5,
                messages=[{"role": "user", "content": "hi " * (i + 1)}])
                for i in range(4)]
            return await asyncio.gather(*[w.generate(r) for r in reqs])
        for r in asyncio.run(go()):
            assert 1 <= r.completion_tokens <= 5
        assert w.engine.states.n_slots == 4
    finally:
        asyncio.run(w.close())


def test_cache_size_per_token():
    from resilient_llm_amd.workers.engine_worker import default_num_blocks
    cfg = get_config("fimunex-2b")
    assert len(cfg.order) == 12
    assert cfg.kv_elems_per_token() == 12 * 4 * 256
    assert default_num_blocks(cfg, kv_gb=1.0) == \
        (1 << 30) // (12 * 1024 * 16 * 2)


def test_loader_refuses_what_does_not_fit():
    import safetensors.torch as st

    from resilient_llm_amd.models import FimunexConfig
    d, w = checkpoint(GREEDY, edit=lambda w: w.pop("l1.mix.lq2"))
    with pytest.raises(KeyError, match="l1.mix.lq2"):
        build_model(get_config(d), weights=d, dtype=F32)
    w["l1.mix.lq2"] = torch.zeros(7, dtype=BF16)
    st.save_file(w, os.path.join(d, "model.safetensors"))
    with pytest.raises(ValueError, match="l1.mix.lq2"):
        build_model(get_config(d), weights=d, dtype=F32)
    good = layer(att(2, 1, 8, 8, 16), moe(3, 1, 2, 8, 2, 1))
    FimunexConfig.from_dict(dict(GREEDY, layers=[good]))

    def change(*path, value):
        bad = copy.deepcopy(good)
        at = bad
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        return bad
    for bad in (change("type", value="gla"),
                change("mixer", "kv_heads", value=4),
                change("mixer", "rot", "dims", value=7),
                change("mixer", "rot", "dims", value=10),
                change("mixer", "vdim", value=600),
                change("mixer", "mask", "size", value=0),
                change("mixer", "softcap", value=0.0),
                change("mlp", "kind", value="dense"),
                change("mlp", "router", "top", value=3),
                change("mlp", "router", "groups", value={"count": 3,
                                                         "keep": 1}),
                change("mlp", "router", "groups", value={"count": 2,
                                                         "keep": 3}),
                change("mlp", "router", "experts", value=256)):
        with pytest.raises(ValueError):
            FimunexConfig.from_dict(dict(GREEDY, layers=[bad]))
    for loop in ((0, 3, 1), (2, 1, 1), (0, 1, 0)):
        with pytest.raises(ValueError, match="loop"):
            FimunexConfig.from_dict(dict(GREEDY, loop=dict(
                zip(("start", "stop", "times"), loop))))


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_replay_program(device, dtype, tmp_path):
    import numpy as np
    d, w = checkpoint(GREEDY, decisive=dtype != F32)
    t = tokens_of(GREEDY, 70, 3)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": t[:50],
                                      "want": []}], "end": []},
             {"step": 1, "entries": [
                 {"id": "x", "tokens": t[50:], "want": [19, 2]},
                 {"id": "y", "tokens": t[:5], "want": [4]}], "end": ["x"]},
             {"step": 2, "entries": [{"id": "y", "tokens": t[5:6],
                                      "want": [0]}], "end": ["y"]}]
    cmd = [sys.executable, os.path.join(REPO, "bin", "trace_run"), "--model",
           d, "--dtype", str(dtype).split(".")[1], "--out", str(tmp_path),
           "--max-tokens", "192"]
    if device == "cpu":
        cmd += ["--device", "cpu"]
    r = subprocess.run(cmd, input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    done = [x for x in r.stdout.splitlines() if x.startswith("done")]
    assert done == ["done 0", "done 1", "done 2"]
    assert not (tmp_path / "0.f32").exists()
    want = expected(GREEDY, w, t)
    for step, rows in ((1, [69, 52, 4]), (2, [5])):
        got = np.fromfile(tmp_path / f"{step}.f32", dtype="<f4")
        check(torch.from_numpy(got).view(len(rows), -1), want[rows], dtype)


def _tp_rank(rank, world, port, d, tokens, out):
    import torch.distributed as dist
    torch.set_num_threads(1)
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(port))
    dist.init_process_group("gloo", rank=rank, world_size=world)
    cfg = get_config(d)
    m = build_model(cfg, weights=d, device="cpu", dtype=F32, tp_rank=rank,
                    tp_world=world)
    kv = PagedKVCache.for_model(cfg, 16, tp_world=world, kv_dtype=F32,
                                state_slots=2)
    e = LLMEngine(m, kv)
    got = feed_portions(e, tokens, [20, 1, 1, 8])
    if rank == 0:
        torch.save(got, out)
    dist.destroy_process_group()


def test_tensor_parallel_matches_single(tmp_path):
    import socket

    import torch.multiprocessing as mp
    config = plain.make_config([
        layer(att(4, 2, 16, 24, 13), moe(4, 2, 3, 40, 3, 2)),
        layer(att(2, 2, 8, 10, 50, rot=4), None),
        layer(att(6, 2, 12, 8, 21), moe(2, 1, 1, 30)),
    ], width=48, vocab=61, loop=(1, 3, 2))
    d, w = checkpoint(config)
    t = tokens_of(config, 30, 3)
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
    out = str(tmp_path / "tp.pt")
    mp.spawn(_tp_rank, args=(2, port, d, t, out), nprocs=2)
    check(torch.load(out, weights_only=True), expected(config, w, t), F32)
