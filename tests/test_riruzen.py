"""Riruzen through the engine against the plain implementation: whole
prompts, token by token, portions, mixed batches, reused pages and slots,
generation, graphs, migration, tensor parallelism, replay."""

import json
import os
import subprocess
import sys

import pytest
import torch

import riruzen_plain as plain
from nesizen_util import (
    BF16, F32, GPU, TARGETS, check, cut, feed_portions, row_errors, tokens_of,
)
from resilient_llm_amd.engine import LLMEngine, PagedKVCache, SamplingParams
from resilient_llm_amd.models import build_model, get_config
from riruzen_util import (
    ATTN_ONLY, CONFIGS, EVEN, ODD, checkpoint, dense, expected, lat, layer,
    make_engine, rec,
)

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
    """Decoding from the first token on."""
    config = CONFIGS[name]
    e, w = make_engine(config, device, dtype)
    t = tokens_of(config, 97, 3)
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
def test_residual_after_every_layer(device, dtype):
    """Where a difference comes from: models cut off after each layer."""
    t = tokens_of(ODD, 40, 6)
    _, w = checkpoint(ODD)
    _, after = plain.run(ODD, w, t)
    for i in range(len(ODD["layers"])):
        config = dict(ODD, layers=ODD["layers"][:i + 1])

        def same(part):
            part.update({k: w[k] for k in part})
        e, _ = make_engine(config, device, dtype, edit=same)
        h = plain.group_norm(after[i], w["final.norm"].double(),
                             ODD["norm"]["groups"], ODD["norm"]["eps"])
        want = h @ w["embed"].double().T * ODD["logit_scale"]
        check(feed_portions(e, t, [30, 1, 9]), want, dtype, f"layer {i}")


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_a_far_token_shows(device, dtype):
    """Latent attention that asks for one token hundreds back: changing
    that token changes the answer, and every cut finds it."""
    config = plain.make_config(
        [layer("latent_attention", lat(2, 16, 32, 24, 64, scale=1.0), None)],
        width=64, vocab=60, taps=3, max_positions=800)

    def sharp(w):
        # channel 0 is only set for token 7, queries ask for it
        w["embed"][:, 0] = 0
        w["embed"][7, 0] = 60.0
        w["pos"][:, 0] = 0
        w["l0.canon1"][0] = 0
        w["l0.norm1"].fill_(1)
        w["l0.mix.dkv"][0].zero_()
        w["l0.mix.dkv"][0, 0] = 8.0
        w["l0.mix.dkv.norm"].fill_(1)
        w["l0.mix.dq.norm"].fill_(1)
        w["l0.mix.uk"].zero_()
        w["l0.mix.uk"].view(2, 16, 64)[:, 0, 0] = 1
        w["l0.mix.uq"].zero_()
        # a query latent channel that is the same for every token
        w["embed"][:, 1] = 6.0
        w["pos"][:, 1] = 0
        w["l0.canon1"][1] = 0
        w["l0.mix.dq"][0].zero_()
        w["l0.mix.dq"][0, 1] = 4.0
        w["l0.mix.uq"].view(2, 16, 24)[:, 0, 0] = 1
    e, w = make_engine(config, device, dtype, edit=sharp)
    t = tokens_of(config, 700, 5)
    t = [x if x != 7 else 8 for x in t]
    quiet = expected(config, w, t)
    t[17] = 7
    want = expected(config, w, t)
    assert float(row_errors(want[400:], quiet[400:]).min()) > 0.1
    for sizes in ([700], [640] + [1] * 60, [300, 2, 100, 5]):
        check(feed_portions(e, t, cut(700, sizes)), want, dtype, str(sizes))


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
    layer("latent_attention", lat(2, 16, 24, 20, 40), dense(40)),
    layer("hgrn2", rec(2, 16, 12), None),
    layer("latent_attention", lat(3, 8, 16, 12, 32), dense(24)),
], width=48, vocab=61, groups=4, taps=4)

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
    """Far past the prompt, over many pages."""
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
@pytest.mark.parametrize("config", [GREEDY, EVEN, ATTN_ONLY],
                         ids=["small", "even", "attn"])
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
def test_live_migration_carries_tails_and_states(device):
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
    assert set(state["recurrent"]["tails"]) == {0, 1, 2}
    assert set(state["recurrent"]["states"]) == {1}
    assert src.kv.free_blocks == src.kv.num_blocks
    dst.queue_adopt(state)
    got += _drain(dst)["m"]
    assert dst.take_adopt_result("m") == "ok"
    assert got == want


def test_prefix_cache_only_without_state():
    e, _ = make_engine(GREEDY, "cpu", F32)
    assert not e.enable_prefix_caching
    with pytest.raises(ValueError, match="spec_lookup"):
        make_engine(GREEDY, "cpu", F32, spec_lookup=3)
    a, w = make_engine(ATTN_ONLY, "cpu", F32)     # a single tap: no tail
    assert a.states is None and a.enable_prefix_caching
    head = tokens_of(ATTN_ONLY, 40, 1)
    for rid, tail in (("x", [3, 4]), ("y", [9, 8, 7])):
        a.add_request(rid, head + tail, SamplingParams(max_tokens=6,
                                                       stop_on_eos=False))
        assert _drain(a)[rid] == _greedy_plain(ATTN_ONLY, w, head + tail, 6)
    assert a.kv.prefix_hits >= 2


@DEVICE
def test_lookup_speculation_without_state(device):
    e, w = make_engine(ATTN_ONLY, device, F32, spec_lookup=3)
    p = tokens_of(ATTN_ONLY, 6, 4) * 4
    e.add_request("l", p, SamplingParams(max_tokens=14, stop_on_eos=False))
    assert _drain(e)["l"] == _greedy_plain(ATTN_ONLY, w, p, 14)


@GPU
def test_fp8_cache_runs_and_stays_near():
    e, w = make_engine(EVEN, "cuda:0", BF16, kv_dtype=torch.float8_e4m3fn)
    t = tokens_of(EVEN, 120, 5)
    got = feed_portions(e, t, [70, 1, 1, 1, 30] + [1] * 17)
    assert float(row_errors(got, expected(EVEN, w, t)).median()) < 0.15


# ------------------------------------------------------------ integration
def test_positions_end_with_the_table():
    config = plain.make_config([layer("hgrn2", rec(1, 8, 8), None)],
                               width=16, vocab=30, max_positions=24)
    e, w = make_engine(config, "cpu", F32)
    t = tokens_of(config, 24, 1)
    check(feed_portions(e, t, [20, 1, 3]), expected(config, w, t), F32)
    from resilient_llm_amd.engine.engine import CapacityExceeded
    with pytest.raises(CapacityExceeded):
        e.feed([("x", tokens_of(config, 25, 1), [])])
    with pytest.raises(CapacityExceeded):
        e.add_request("y", t[:20], SamplingParams(max_tokens=5))
    cfg = get_config(checkpoint(config)[0])
    cfg.fit_positions(4096)
    assert cfg.max_position == 24


def test_registry_picks_the_class_by_config():
    from resilient_llm_amd.models import (
        NesizenForCausalLM, RiruzenForCausalLM, get_model_class, model_names,
    )
    d, _ = checkpoint(GREEDY)
    assert get_model_class(d) is RiruzenForCausalLM
    assert get_model_class("tiny", d) is RiruzenForCausalLM
    assert get_model_class("riruzen-tiny") is RiruzenForCausalLM
    assert get_model_class("nesizen-tiny") is NesizenForCausalLM
    assert {"riruzen-tiny", "riruzen-1b"} <= set(model_names())


@pytest.mark.parametrize("model", ["riruzen-tiny", "checkpoint"])
def test_worker_serves_it(model):
    import asyncio

    from resilient_llm_amd.workers.base import GenerationRequest
    from resilient_llm_amd.workers.engine_worker import EngineWorker
    name = model if model != "checkpoint" else checkpoint(
        plain.make_config(GREEDY["layers"], width=48, vocab=300))[0]
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
    cfg = get_config("riruzen-1b")
    assert cfg.kv_elems_per_token() == 4 * 512
    assert default_num_blocks(cfg, kv_gb=1.0) == (1 << 30) // (2048 * 16 * 2)


def test_loader_refuses_what_does_not_fit():
    import safetensors.torch as st

    from resilient_llm_amd.models import RiruzenConfig
    d, w = checkpoint(GREEDY, edit=lambda w: w.pop("l1.mix.lower"))
    with pytest.raises(KeyError, match="l1.mix.lower"):
        build_model(get_config(d), weights=d, dtype=F32)
    w["l1.mix.lower"] = torch.zeros(7, dtype=BF16)
    st.save_file(w, os.path.join(d, "model.safetensors"))
    with pytest.raises(ValueError, match="l1.mix.lower"):
        build_model(get_config(d), weights=d, dtype=F32)
    for change in ({"width": 50}, {"canon": {"taps": 0}},
                   {"layers": [layer("attention", {}, None)]},
                   {"layers": [layer("hgrn2", rec(1, 300, 8), None)]}):
        with pytest.raises(ValueError):
            RiruzenConfig.from_dict(dict(GREEDY, **change))


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_replay_program(device, dtype, tmp_path):
    import numpy as np
    d, w = checkpoint(GREEDY)
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
           "--max-tokens", "640"]                 # more than the table holds
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
        layer("latent_attention", lat(4, 16, 24, 20, 40), dense(40)),
        layer("hgrn2", rec(2, 16, 12), None),
        layer("hgrn2", rec(4, 8, 10), dense(30)),
    ], width=48, vocab=61, groups=3)
    d, w = checkpoint(config)
    t = tokens_of(config, 30, 3)
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        port = s.getsockname()[1]
    out = str(tmp_path / "tp.pt")
    mp.spawn(_tp_rank, args=(2, port, d, t, out), nprocs=2)
    check(torch.load(out, weights_only=True), expected(config, w, t), F32)
