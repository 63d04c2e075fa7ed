#!/usr/bin/env python3
"""Flagship serving benchmark — the driver contract.

Measures BASELINE.json's metric: sustained reqs/sec + success-rate + p50
latency @ 64 concurrent, Llama-3-8B bf16, synthetic prompts, random-init
weights, on N GPUs of one node (weak scaling: 64 concurrent clients per
GPU).

Full-stack path: every rank hosts one EngineWorker on its GPU behind the
unix-socket RPC; rank 0 additionally runs the OpenAI-compatible gateway
(router + ledger) and the closed-loop load generator over HTTP.  One
"step" = every concurrency slot completes exactly one request
(prompt 128 tokens -> 64 new tokens, greedy).  W untimed warmup steps,
then K timed steps bracketed by gloo barrier + torch.cuda.synchronize on
both sides; elapsed is the MAX over ranks; rank 0 prints ONE JSON line.

Launch (driver):
  python bench.py --gpus 1 --steps K --warmup W
  python -m torch.distributed.run --nnodes=1 --nproc-per-node N \
      --master-addr 127.0.0.1 bench.py --gpus N --steps K --warmup W

`--design nesizen` (or riruzen, bolatar) measures something else:
engine-level prefill and decode throughput of that design at layer sizes of
real models, beside existing models of equal width, depth and active
parameters (one JSON line per model and size; see run_design).
"""

from __future__ import annotations

import argparse
import asyncio
import json
import os
import socket
import sys
import tempfile
import threading
import time

REPO_ROOT = os.path.dirname(os.path.abspath(__file__))
if REPO_ROOT not in sys.path:
    sys.path.insert(0, REPO_ROOT)

PROMPT_TOKENS = 128
OUTPUT_TOKENS = 64
CONCURRENCY_PER_GPU = 64

# distributed hardening (the first 8-GPU run happens
# blind — a dead rank must produce a diagnosis, not a silent hang):
# rendezvous + collective timeout, and a faulthandler watchdog that dumps
# all thread stacks and exits non-zero if a barrier never completes.
RENDEZVOUS_TIMEOUT_S = float(os.environ.get("RLLI_BENCH_RDZV_TIMEOUT_S", "300"))
WATCHDOG_S = float(os.environ.get("RLLI_BENCH_WATCHDOG_S", "1200"))

_RANK = os.environ.get("RANK", "0")


def log(msg):
    print(f"[bench r{_RANK}] {msg}", file=sys.stderr, flush=True)


def arm_watchdog(tag: str, seconds: float = WATCHDOG_S):
    """If this rank is still stuck here after ``seconds``, dump every
    thread's stack to stderr and hard-exit so torchrun tears the job
    down with a readable cause instead of hanging the driver."""
    import faulthandler
    log(f"watchdog armed: {tag} ({seconds:.0f}s)")
    faulthandler.dump_traceback_later(seconds, exit=True)


def disarm_watchdog():
    import faulthandler
    faulthandler.cancel_dump_traceback_later()


def free_port() -> int:
    with socket.socket() as s:
        s.bind(("127.0.0.1", 0))
        return s.getsockname()[1]


class LoopThread:
    """An asyncio loop on a daemon thread; run() schedules coroutines."""

    def __init__(self) -> None:
        self.loop = asyncio.new_event_loop()
        self._thread = threading.Thread(
            target=self.loop.run_forever, daemon=True)
        self._thread.start()

    def run(self, coro, timeout=None):
        return asyncio.run_coroutine_threadsafe(coro, self.loop).result(timeout)


def start_worker(loopth: LoopThread, device: str, label: str, sock: str,
                 model: str, max_batch: int, num_blocks: int,
                 use_graphs: bool, kv_dtype: str = "bf16",
                 quant=None):
    from resilient_llm_amd.workers.engine_worker import EngineWorker
    from resilient_llm_amd.workers.rpc import WorkerRpcServer

    async def _start():
        worker = EngineWorker(device=device, model_name=model,
                              device_label=label,
                              max_batch_size=max_batch,
                              max_queue=max_batch * 4,
                              num_blocks=num_blocks,
                              kv_dtype=kv_dtype,
                              quant=quant,
                              use_graphs=use_graphs)
        server = WorkerRpcServer(worker, sock)
        await server.start()
        return worker

    return loopth.run(_start(), timeout=600)


def spawn_gateways(n_gpus: int, model: str, port: int, run_dir: str,
                   n_procs: int) -> list:
    """Gateway PROCESSES sharing the port via SO_REUSEPORT (the same
    scale-out LiteLLM's --num_workers provides); the bench config has no
    rate limits, so per-process windows are irrelevant here."""
    import subprocess
    sockets = ",".join(os.path.join(run_dir, f"w{r}.sock")
                       for r in range(n_gpus))
    procs = []
    ready_files = []
    for g in range(n_procs):
        rf = os.path.join(run_dir, f"gw{g}.ready")
        ready_files.append(rf)
        env = dict(os.environ)
        env["PYTHONPATH"] = REPO_ROOT + os.pathsep + env.get("PYTHONPATH", "")
        procs.append(subprocess.Popen(
            [sys.executable, "-m", "resilient_llm_amd.gateway.bench_gateway",
             "--port", str(port), "--model", model, "--sockets", sockets,
             "--ready-file", rf], env=env))
    deadline = time.time() + 900
    while time.time() < deadline:
        if all(os.path.exists(rf) for rf in ready_files):
            return procs
        for p in procs:
            assert p.poll() is None, "gateway process died during startup"
        time.sleep(0.25)
    raise RuntimeError("gateways failed to come up")


class LoadGen:
    """Driver for the loadgen subprocess (scripts/loadgen.py) — the
    client side runs in its own process so rank 0's gateway loop does
    not share a GIL with it at 8-GPU request rates."""

    def __init__(self, port: int, concurrency: int, prompt_tokens: int,
                 output_tokens: int) -> None:
        import subprocess
        self.proc = subprocess.Popen(
            [sys.executable, os.path.join(REPO_ROOT, "scripts", "loadgen.py"),
             "--port", str(port), "--concurrency", str(concurrency),
             "--prompt-tokens", str(prompt_tokens),
             "--output-tokens", str(output_tokens)],
            stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
        ready = self.proc.stdout.readline().strip()
        assert ready == "READY", ready

    def round(self) -> dict:
        self.proc.stdin.write("ROUND\n")
        self.proc.stdin.flush()
        line = self.proc.stdout.readline()
        return json.loads(line)

    def close(self) -> None:
        try:
            self.proc.stdin.write("QUIT\n")
            self.proc.stdin.flush()
            self.proc.wait(timeout=10)
        except Exception:
            self.proc.kill()


def design_models(design: str) -> dict:
    """size -> {name: configuration}: the design, then existing models of
    equal width, depth, heads and (active) feed-forward size."""
    from resilient_llm_amd.models import (
        BolatarConfig, FimunexConfig, LlamaConfig, NesizenConfig,
        RiruzenConfig,
    )
    from resilient_llm_amd.models import bolatar, fimunex, nesizen, riruzen

    def llama(width, layers, heads, kv, ff):
        return LlamaConfig(name=f"llama-w{width}", hidden_size=width,
                           n_layers=layers, n_heads=heads, n_kv_heads=kv,
                           head_dim=128, intermediate_size=ff,
                           vocab_size=65536, max_position=32768)

    def nesi(width, layers, heads, kv, gla_heads, mlp, first=None,
             attn_every=3, window=1024):
        return NesizenConfig.from_dict(
            {"width": width, "vocab": 65536, "streams": 2,
             "norm": {"eps": 1e-5},
             "layers": nesizen.hybrid_layers(
                 layers, attn_every,
                 {"heads": heads, "kv_heads": kv, "dim": 128, "vdim": 128,
                  "scale": 128 ** -0.5, "rot": {"dims": 64, "base": 1e6},
                  "mask": {"size": window, "keep_first": 4}},
                 {"heads": gla_heads, "dim": 128, "vdim": 256, "tau": 16.0},
                 mlp, first)},
            name=f"nesizen-w{width}")

    def moe(experts, top, ff):
        return {"kind": "moe", "expert": {"ff": ff, "limit": 7.0},
                "router": {"experts": experts, "top": top}}

    def riru(width, layers, heads, q_rank, ff):
        return RiruzenConfig.from_dict(
            {"width": width, "vocab": 65536, "logit_scale": 1.0,
             "max_positions": 32768, "canon": {"taps": 4},
             "norm": {"eps": 1e-5, "groups": 4},
             "layers": riruzen.hybrid_layers(
                 layers, 3,
                 {"heads": heads, "dim": 128, "vdim": 128, "q_rank": q_rank,
                  "kv_rank": 512, "scale": 128 ** -0.5},
                 {"heads": heads, "dim": 128, "vdim": 128},
                 {"kind": "dense", "ff": ff})}, name=f"riruzen-w{width}")

    def bola(width, layers, heads, kv, ff):
        return BolatarConfig.from_dict(
            {"width": width, "vocab": 65536, "logit_softcap": 30.0,
             "max_positions": 32768, "embedding": {"scale": 1.0},
             "norm": {"eps": 1e-5},
             "layers": bolatar.hybrid_layers(
                 layers, 3,
                 {"left": {"heads": heads, "kv_heads": kv, "dim": 128,
                           "vdim": 128, "scale": 128 ** -0.5,
                           "q_temp": {"coef": 0.1, "every": 4096}},
                  "right": {"heads": heads, "dim": 64}},
                 {"heads": heads, "kv_heads": heads // 2, "dim": 128,
                  "vdim": 128, "conv": 4},
                 {"heads": heads // 2, "dim": 128, "vdim": 256,
                  "gate_cap": 15.0},
                 {"kind": "dense", "ff": ff, "limit": 7.0})},
            name=f"bolatar-w{width}", decay_rank=64)

    def fimu(width, layers, heads, kv, mlp):
        return FimunexConfig.from_dict(
            {"width": width, "vocab": 65536, "logit_softcap": 30.0,
             "canon": {"taps": 4}, "norm": {"eps": 1e-5},
             "loop": {"start": 0, "stop": layers, "times": 1},
             "layers": fimunex.uniform_layers(
                 layers, fimunex.diff_attention(heads, kv, 64, 128, 4096),
                 mlp)}, name=f"fimunex-w{width}")

    def dense(ff):
        return {"kind": "dense", "ff": ff}
    if design == "fimunex":
        # attention in every layer, as far as either sees; two matrices of
        # 3/2 the width are as large as the gated three
        relu2 = fimunex.relu2_moe
        return {"w2048": {"fimunex": fimu(2048, 12, 16, 4,
                                          relu2(32, 8, 4, 1536, 8, 4)),
                          "nesizen": nesi(2048, 12, 16, 4, 8,
                                          moe(32, 4, 1024), attn_every=1,
                                          window=4096),
                          "llama": llama(2048, 12, 16, 4, 4096)},
                "w4096": {"fimunex": fimu(4096, 6, 32, 8,
                                          relu2(16, 4, 2, 5376, 4, 2)),
                          "nesizen": nesi(4096, 6, 32, 8, 16,
                                          moe(16, 2, 3584), attn_every=1,
                                          window=4096),
                          "llama": llama(4096, 6, 32, 8, 7168)}}
    if design == "bolatar":
        # two matrices of 3/2 the width are as large as the gated three
        return {"w2048": {"bolatar": bola(2048, 12, 16, 4, 4096),
                          "nesizen": nesi(2048, 12, 16, 4, 8, dense(6144)),
                          "llama": llama(2048, 12, 16, 4, 4096)},
                "w4096": {"bolatar": bola(4096, 6, 32, 8, 7168),
                          "nesizen": nesi(4096, 6, 32, 8, 16, dense(10752)),
                          "llama": llama(4096, 6, 32, 8, 7168)}}
    if design == "nesizen":
        return {"w2048": {"nesizen": nesi(2048, 12, 16, 4, 8,
                                          moe(32, 4, 1024), dense(6144)),
                          "llama": llama(2048, 12, 16, 4, 4096)},
                "w4096": {"nesizen": nesi(4096, 6, 32, 8, 16,
                                          moe(16, 2, 3584), dense(10752)),
                          "llama": llama(4096, 6, 32, 8, 7168)}}
    # two matrices of 3/2 the width are as large as the gated three
    return {"w2048": {"riruzen": riru(2048, 12, 16, 768, 4096),
                      "nesizen": nesi(2048, 12, 16, 4, 8, dense(6144)),
                      "llama": llama(2048, 12, 16, 4, 4096)},
            "w4096": {"riruzen": riru(4096, 6, 32, 1536, 7168),
                      "nesizen": nesi(4096, 6, 32, 8, 16, dense(10752)),
                      "llama": llama(4096, 6, 32, 8, 7168)}}


def run_design(design: str, sizes: list, which: list, steps: int,
               phases: list) -> None:
    """Engine-level throughput, no gateway: prefill = prompt tokens/s of
    one full prefill step, decode = output tokens/s of graph-replayed
    steps.  Random weights, synthetic tokens."""
    import torch

    from resilient_llm_amd.engine import (
        LLMEngine, PagedKVCache, SamplingParams,
    )
    from resilient_llm_amd.engine.graph import install_graph_runner
    from resilient_llm_amd.models import build_model

    def sync():
        torch.cuda.synchronize()
        return time.monotonic()

    rng = torch.Generator().manual_seed(0)

    def prompt(n):
        return torch.randint(5, 60000, (n,), generator=rng).tolist()

    for size in sizes:
        for kind, cfg in design_models(design)[size].items():
            if which and kind not in which:
                continue
            model = build_model(cfg, device="cuda:0", dtype=torch.bfloat16)
            for phase in phases:
                name, batch, ctx = phase.split(":")
                batch, ctx = int(batch), int(ctx)
                per_seq = -(-(ctx + 512) // 16)
                kv = PagedKVCache.for_model(
                    cfg, batch * per_seq + 8, device="cuda:0",
                    state_slots=batch + 1)
                e = LLMEngine(model, kv, max_batch_size=batch,
                              max_prefill_tokens=max(batch * ctx, 8192)
                              if name == "prefill" else 8192,
                              chunk_size=8192, enable_prefix_caching=False)
                n_out = 1 if name == "prefill" else 500
                times = []
                if name == "prefill":
                    for rep in range(steps + 2):
                        for b in range(batch):
                            e.add_request(f"{rep}-{b}", prompt(ctx),
                                          SamplingParams(max_tokens=n_out))
                        t0 = sync()
                        e.step()
                        times.append(sync() - t0)
                        assert not e.has_work()
                    ms = sorted(times[2:])[steps // 2] * 1e3
                    tok = batch * ctx
                else:
                    install_graph_runner(e, max_blocks_per_seq=per_seq)
                    for b in range(batch):
                        e.add_request(f"d{b}", prompt(ctx), SamplingParams(
                            max_tokens=n_out, stop_on_eos=False))
                    while len(e.running) < batch:
                        e.step()
                    for _ in range(5):
                        e.step()
                    n = 64
                    for _ in range(steps):
                        t0 = sync()
                        for _ in range(n):
                            e.step()
                        times.append((sync() - t0) / n)
                    ms = sorted(times)[len(times) // 2] * 1e3
                    tok = batch
                print(json.dumps({
                    "design": kind, "size": size, "phase": name,
                    "batch": batch, "context": ctx,
                    "ms_per_step": round(ms, 3),
                    "tokens_per_s": round(tok / ms * 1e3, 1),
                    "params_gib": round(model.param_bytes() / 2**30, 2),
                    "dtype": "bf16", "data": "synthetic"}), flush=True)
                del e, kv
                torch.cuda.empty_cache()
            del model
            torch.cuda.empty_cache()


def main() -> None:
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=4)
    ap.add_argument("--warmup", type=int, default=1)
    ap.add_argument("--model", default="llama-3-8b")
    ap.add_argument("--concurrency", type=int, default=CONCURRENCY_PER_GPU,
                    help="concurrent clients per GPU (weak scaling)")
    ap.add_argument("--prompt-tokens", type=int, default=PROMPT_TOKENS)
    ap.add_argument("--output-tokens", type=int, default=OUTPUT_TOKENS)
    ap.add_argument("--no-graphs", action="store_true")
    ap.add_argument("--kv-dtype", default="bf16", choices=("bf16", "fp8"),
                    help="paged-KV element type (fp8 = opt-in e4m3 cache; "
                         "the headline metric stays bf16)")
    ap.add_argument("--quant", default=None, choices=("fp8",),
                    help="W8A8-fp8 weight quantization (opt-in mode; the "
                         "headline metric stays bf16)")
    ap.add_argument("--device", default=None,
                    help="override torch device (tests: cpu)")
    ap.add_argument("--design", default=None,
                    choices=("nesizen", "riruzen", "bolatar", "fimunex"),
                    help="measure this design's engine throughput beside "
                         "existing models of equal size instead of serving")
    ap.add_argument("--design-sizes", default="w2048,w4096")
    ap.add_argument("--design-models", default="",
                    help="comma list of models to measure (default: all)")
    ap.add_argument("--design-phases", default="prefill:4:2048,"
                    "prefill:1:8192,decode:1:2048,decode:16:2048,"
                    "decode:64:2048",
                    help="comma list of phase:sequences:tokens")
    args = ap.parse_args()
    if args.design:
        run_design(args.design, args.design_sizes.split(","),
                   [m for m in args.design_models.split(",") if m],
                   max(1, args.steps), args.design_phases.split(","))
        return
    globals()["OUTPUT_TOKENS"] = args.output_tokens

    import torch
    import torch.distributed as dist

    rank = int(os.environ.get("RANK", "0"))
    world = int(os.environ.get("WORLD_SIZE", "1"))
    local_rank = int(os.environ.get("LOCAL_RANK", str(rank)))
    n_gpus = args.gpus
    assert world == n_gpus or world == 1, \
        f"WORLD_SIZE {world} must equal --gpus {n_gpus}"
    distributed = world > 1
    if distributed:
        import datetime
        os.environ.setdefault("MASTER_ADDR", "127.0.0.1")
        arm_watchdog("rendezvous", RENDEZVOUS_TIMEOUT_S + 60)
        dist.init_process_group(
            backend="gloo", rank=rank, world_size=world,
            timeout=datetime.timedelta(seconds=RENDEZVOUS_TIMEOUT_S))
        disarm_watchdog()
        log(f"rendezvous complete: rank {rank}/{world}")

    on_gpu = args.device is None and torch.cuda.is_available()
    # co-located ranks (rehearsal: 2 ranks on a 1-GPU box) wrap onto the
    # devices that exist; on a full node this is the identity mapping
    dev_index = local_rank % max(1, torch.cuda.device_count()) if on_gpu else 0
    device = args.device or (f"cuda:{dev_index}" if on_gpu else "cpu")
    if on_gpu:
        torch.cuda.set_device(dev_index)
        if dev_index != local_rank:
            log(f"co-located: local_rank {local_rank} -> cuda:{dev_index}")

    def sync(tag="sync"):
        arm_watchdog(tag)
        if on_gpu:
            torch.cuda.synchronize()
        if distributed:
            dist.barrier()
        disarm_watchdog()

    # shared run dir for worker sockets (rank 0 creates, broadcasts)
    if distributed:
        holder = [tempfile.mkdtemp(prefix="rlli-bench-")] if rank == 0 else [None]
        dist.broadcast_object_list(holder, src=0)
        run_dir = holder[0]
    else:
        run_dir = tempfile.mkdtemp(prefix="rlli-bench-")

    conc_total = args.concurrency * n_gpus
    max_seq_blocks = -(-(args.prompt_tokens + args.output_tokens + 8) // 16)
    num_blocks = args.concurrency * (max_seq_blocks + 1) + 64

    loopth = LoopThread()
    t_init = time.time()
    worker = start_worker(loopth, device, f"gpu:{rank}",
                          os.path.join(run_dir, f"w{rank}.sock"),
                          args.model, max_batch=args.concurrency,
                          num_blocks=num_blocks,
                          use_graphs=on_gpu and not args.no_graphs,
                          kv_dtype=args.kv_dtype, quant=args.quant)
    log(f"rank {rank}: worker up on {device} in {time.time() - t_init:.1f}s "
        f"({num_blocks} KV blocks)")
    sync("post-worker-startup barrier")

    port = None
    loadgen = None
    gateways: list = []
    rounds_timed: list = []
    if rank == 0:
        port = free_port()
        n_gw = max(1, min(4, (n_gpus + 1) // 2))
        gateways = spawn_gateways(n_gpus if distributed else 1, args.model,
                                  port, run_dir, n_gw)
        loadgen = LoadGen(port, conc_total, args.prompt_tokens,
                          args.output_tokens)
        log(f"{n_gw} gateway process(es) on :{port}, driving {conc_total} "
            f"concurrent clients (loadgen subprocess)")

    # ---- warmup ----
    for w in range(args.warmup):
        if rank == 0:
            res = loadgen.round()
            log(f"warmup {w}: {res['ok']}/{res['total']} ok")
        sync(f"warmup {w} barrier")

    # ---- timed ----
    sync("pre-timed barrier")
    t0 = time.monotonic()
    arm_watchdog("timed rounds", WATCHDOG_S)
    for k in range(args.steps):
        if rank == 0:
            rounds_timed.append(loadgen.round())
    disarm_watchdog()
    sync("post-timed barrier")
    elapsed = time.monotonic() - t0
    try:
        h = loopth.run(worker.health(), timeout=30)
        stats = h.get("engine_stats", {})
        log(f"rank {rank} engine stats: {stats}")
        admits = worker.engine.stats.get("admit_events", [])
        log(f"rank {rank} admits (t, n, still_waiting): {admits[:40]}")
        if worker.engine._trace:
            tr = worker.engine._trace[-220:]
            lines = []
            prev = None
            for t0, kind, ms in tr:
                gap = 0.0 if prev is None else (t0 - prev) * 1e3
                lines.append(f"{t0:.4f} +{gap:6.2f}ms {kind} host={ms}ms")
                prev = t0
            log("step trace (last 220):\n" + "\n".join(lines))
    except Exception:
        pass
    if distributed:
        t = torch.tensor([elapsed], dtype=torch.float64)
        dist.all_reduce(t, op=dist.ReduceOp.MAX)
        elapsed = float(t.item())

    if rank == 0:
        loadgen.close()
        for g in gateways:
            g.terminate()
        n_req = sum(r["total"] for r in rounds_timed)
        n_ok = sum(r["ok"] for r in rounds_timed)
        lats = sorted(l for r in rounds_timed for l in r["latencies"])
        p50 = lats[len(lats) // 2] if lats else None
        p99 = lats[min(len(lats) - 1, int(0.99 * len(lats)))] if lats else None
        out_toks = sum(r["completion_tokens"] for r in rounds_timed)
        total_toks = out_toks + sum(r["prompt_tokens"] for r in rounds_timed)
        reqs_per_s = n_ok / elapsed
        result = {
            "metric": "sustained reqs/sec + success-rate + p50 latency "
                      "@ 64 concurrent, Llama-3-8B",
            "value": round(reqs_per_s, 3),
            "unit": "reqs/s",
            "n_gpus": n_gpus,
            "steps": args.steps,
            "warmup": args.warmup,
            "ms_per_step": round(elapsed / args.steps * 1000.0, 1),
            "higher_is_better": True,
            "scaling": "weak",
            "vs_baseline": None,
            "dtype": "fp8-w8a8(gate_up/down/lm_head)+bf16"
                     if args.quant == "fp8" else "bf16",
            "data": "synthetic",
            "config": {
                "model": args.model,
                "global_batch": conc_total,
                "seq_len": args.prompt_tokens + args.output_tokens,
                "parallelism": f"dp{n_gpus}",
                "concurrency_per_gpu": args.concurrency,
                "prompt_tokens": args.prompt_tokens,
                "output_tokens": args.output_tokens,
                "success_rate": round(n_ok / n_req, 4) if n_req else None,
                "p50_latency_s": round(p50, 3) if p50 else None,
                "p99_latency_s": round(p99, 3) if p99 else None,
                "output_tokens_per_s": round(out_toks / elapsed, 1),
                "total_tokens_per_s": round(total_toks / elapsed, 1),
                "temperature": 0.0,
            },
        }
        print(json.dumps(result), flush=True)
    if distributed:
        dist.barrier()
        dist.destroy_process_group()
    os._exit(0)   # daemon loops/threads: exit hard once results are printed


if __name__ == "__main__":
    main()
