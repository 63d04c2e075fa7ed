"""Op dispatch: hand-written gfx950 HIP kernels on GPU, fp32 torch
references on CPU.

On a CUDA/ROCm device the HIP extension is REQUIRED — a missing .so
raises immediately rather than silently falling back to eager PyTorch
(the round-end check records which native libraries the GPU tests
actually loaded).  On CPU the ops/ref.py implementations run, which is
what the no-GPU plumbing tests and the gloo multi-process tests use.
"""

from __future__ import annotations

import os
import torch

from . import ref  # noqa: F401

_HERE = os.path.dirname(os.path.abspath(__file__))
_SO_PATH = os.path.join(_HERE, "_rlli_hip.so")
_loaded = False
_loaded_libs: set = set()


class ExtensionMissing(RuntimeError):
    pass


def load_extension(required: bool = False) -> bool:
    """Load the in-tree .so (idempotent).  ``required=True`` (or any GPU
    call) raises if it is absent — no silent eager fallback on GPU."""
    global _loaded
    if _loaded:
        return True
    if os.path.exists(_SO_PATH):
        torch.ops.load_library(_SO_PATH)
        _loaded = True
        return True
    if required:
        raise ExtensionMissing(
            f"HIP extension not built: {_SO_PATH} missing. "
            f"Run `python -m resilient_llm_amd.ops.build`.")
    return False


def extension_loaded() -> bool:
    return _loaded


def _gpu() -> None:
    load_extension(required=True)


def load_libraries(libs) -> None:
    """Load kernel libraries by name (idempotent); raises if one is not
    built."""
    for lib in libs:
        if lib in _loaded_libs:
            continue
        if lib == "rlli_hip":
            _gpu()
            continue
        path = os.path.join(_HERE, f"_{lib}.so")
        if not os.path.exists(path):
            raise ExtensionMissing(
                f"HIP extension not built: {path} missing. "
                f"Run `python -m resilient_llm_amd.ops.build`.")
        torch.ops.load_library(path)
        _loaded_libs.add(lib)


# ------------------------------------------------------------------ ops
def rmsnorm(x: torch.Tensor, w: torch.Tensor, eps: float = 1e-5) -> torch.Tensor:
    if x.is_cuda:
        _gpu()
        return torch.ops.rlli.rmsnorm(x, w, eps)
    return ref.rmsnorm(x, w, eps)


def rmsnorm_residual_(x: torch.Tensor, residual: torch.Tensor, w: torch.Tensor,
                      eps: float = 1e-5) -> torch.Tensor:
    if x.is_cuda:
        _gpu()
        return torch.ops.rlli.rmsnorm_residual_(x, residual, w, eps)
    return ref.rmsnorm_residual_(x, residual, w, eps)


def rmsnorm_fp8(x, w, eps: float = 1e-5):
    """Fused rmsnorm + per-row fp8-e4m3 quantization -> (q, scales)."""
    if x.is_cuda:
        _gpu()
        return torch.ops.rlli.rmsnorm_fp8(x, w, eps)
    return ref.rmsnorm_fp8(x, w, eps)


def rmsnorm_residual_fp8(x, residual, w, eps: float = 1e-5):
    if x.is_cuda:
        _gpu()
        return torch.ops.rlli.rmsnorm_residual_fp8(x, residual, w, eps)
    return ref.rmsnorm_residual_fp8(x, residual, w, eps)


def silu_mul_fp8(gate_up):
    if gate_up.is_cuda:
        _gpu()
        return torch.ops.rlli.silu_mul_fp8(gate_up)
    return ref.silu_mul_fp8(gate_up)


def silu_mul(gate_up: torch.Tensor) -> torch.Tensor:
    if gate_up.is_cuda:
        _gpu()
        return torch.ops.rlli.silu_mul(gate_up)
    return ref.silu_mul(gate_up)


def rope_kv_append_(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                    positions: torch.Tensor, cos_sin: torch.Tensor,
                    k_cache: torch.Tensor, v_cache: torch.Tensor,
                    slot_mapping: torch.Tensor) -> None:
    if q.is_cuda:
        _gpu()
        torch.ops.rlli.rope_kv_append_(q, k, v, positions, cos_sin,
                                       k_cache, v_cache, slot_mapping)
    else:
        ref.rope_kv_append_(q, k, v, positions, cos_sin, k_cache, v_cache,
                            slot_mapping)


def rope_kv_append_qkv_(qkv: torch.Tensor, positions: torch.Tensor,
                        cos_sin: torch.Tensor, k_cache: torch.Tensor,
                        v_cache: torch.Tensor, slot_mapping: torch.Tensor,
                        n_q: int) -> None:
    """Fused-QKV form: rope + cache append on strided views of the raw
    qkv GEMM output (no .contiguous() copies)."""
    if qkv.is_cuda:
        _gpu()
        torch.ops.rlli.rope_kv_append_qkv_(qkv, positions, cos_sin, k_cache,
                                           v_cache, slot_mapping, n_q)
        return
    T = qkv.shape[0]
    n_kv, _, D = k_cache.shape[1], k_cache.shape[2], k_cache.shape[3]
    q = qkv[:, :n_q * D].view(T, n_q, D)
    k = qkv[:, n_q * D:(n_q + n_kv) * D].view(T, n_kv, D)
    v = qkv[:, (n_q + n_kv) * D:].view(T, n_kv, D)
    ref.rope_kv_append_(q, k, v, positions, cos_sin, k_cache, v_cache,
                        slot_mapping)


def decode_attn_qkv(qkv: torch.Tensor, k_cache: torch.Tensor,
                    v_cache: torch.Tensor, block_table: torch.Tensor,
                    seq_lens: torch.Tensor, scale: float,
                    n_q: int) -> torch.Tensor:
    if qkv.is_cuda:
        _gpu()
        return torch.ops.rlli.decode_attn_qkv(qkv, k_cache, v_cache,
                                              block_table, seq_lens, scale, n_q)
    B = qkv.shape[0]
    D = k_cache.shape[3]
    q = qkv[:, :n_q * D].reshape(B, n_q, D)
    out = ref.decode_attn(q, k_cache, v_cache, block_table, seq_lens, scale)
    return out.reshape(B, n_q * D)


def decode_attn_rope_qkv(qkv, positions, cos_sin, k_cache, v_cache,
                         slot_mapping, block_table, seq_lens, scale: float,
                         n_q: int) -> torch.Tensor:
    """Fused decode step: rope(q,k) + cache append + paged attention in
    one kernel on GPU; composed from the unfused reference ops on CPU."""
    if qkv.is_cuda:
        _gpu()
        return torch.ops.rlli.decode_attn_rope_qkv(
            qkv, positions, cos_sin, k_cache, v_cache, slot_mapping,
            block_table, seq_lens, scale, n_q)
    rope_kv_append_qkv_(qkv, positions, cos_sin, k_cache, v_cache,
                        slot_mapping, n_q)
    return decode_attn_qkv(qkv, k_cache, v_cache, block_table, seq_lens,
                           scale, n_q)


def prefill_attn_qkv(qkv: torch.Tensor, cu_seqlens: torch.Tensor,
                     scale: float, n_q: int, n_kv: int,
                     head_dim: int) -> torch.Tensor:
    if qkv.is_cuda:
        _gpu()
        return torch.ops.rlli.prefill_attn_qkv(qkv, cu_seqlens, scale, n_q,
                                               n_kv, head_dim)
    T = qkv.shape[0]
    D = head_dim
    q = qkv[:, :n_q * D].reshape(T, n_q, D)
    k = qkv[:, n_q * D:(n_q + n_kv) * D].reshape(T, n_kv, D)
    v = qkv[:, (n_q + n_kv) * D:].reshape(T, n_kv, D)
    return ref.prefill_attn(q, k, v, cu_seqlens, scale).reshape(T, n_q * D)


def decode_attn(q: torch.Tensor, k_cache: torch.Tensor, v_cache: torch.Tensor,
                block_table: torch.Tensor, seq_lens: torch.Tensor,
                scale: float) -> torch.Tensor:
    if q.is_cuda:
        _gpu()
        return torch.ops.rlli.decode_attn(q, k_cache, v_cache, block_table,
                                          seq_lens, scale)
    return ref.decode_attn(q, k_cache, v_cache, block_table, seq_lens, scale)


def prefill_attn(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor,
                 cu_seqlens: torch.Tensor, scale: float) -> torch.Tensor:
    if q.is_cuda:
        _gpu()
        return torch.ops.rlli.prefill_attn(q, k, v, cu_seqlens, scale)
    return ref.prefill_attn(q, k, v, cu_seqlens, scale)


def sample(logits: torch.Tensor, temperatures: torch.Tensor,
           seeds: torch.Tensor, step: int = 0) -> torch.Tensor:
    """Greedy argmax / Gumbel-max temperature sampling; ``seeds`` is a
    per-row int64 tensor (per-request reproducibility), ``step`` a
    uniform step offset mixed in-kernel."""
    if logits.is_cuda:
        _gpu()
        return torch.ops.rlli.sample(logits, temperatures, seeds, step)
    return ref.sample(logits, temperatures, seeds, step)


def prefill_paged_attn(qkv, k_cache, v_cache, chunk_row0, chunk_pos0,
                       chunk_nrows, chunk_btrow, block_tables,
                       scale: float, n_q: int) -> torch.Tensor:
    if qkv.is_cuda:
        _gpu()
        return torch.ops.rlli.prefill_paged_attn(
            qkv, k_cache, v_cache, chunk_row0, chunk_pos0, chunk_nrows,
            chunk_btrow, block_tables, scale, n_q)
    return ref.prefill_paged_attn(qkv, k_cache, v_cache, chunk_row0,
                                  chunk_pos0, chunk_nrows, chunk_btrow,
                                  block_tables, scale, n_q)


def skinny_linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """Decode-projection GEMM (M<=64): custom MFMA weight-streaming
    kernel on GPU, F.linear on CPU."""
    if x.is_cuda:
        _gpu()
        return torch.ops.rlli.skinny_linear(x, w)
    return torch.nn.functional.linear(x, w)


def linear_auto(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """Pick the skinny-M kernel when the shape qualifies, else
    hipBLASLt via F.linear."""
    if (x.is_cuda and x.dim() == 2 and 1 <= x.shape[0] <= 64
            and x.shape[1] % 256 == 0 and w.shape[0] % 64 == 0):
        _gpu()
        return torch.ops.rlli.skinny_linear(x, w)
    return torch.nn.functional.linear(x, w)


def skinny2_linear(x: torch.Tensor, w: torch.Tensor,
                   splitk: int = 0) -> torch.Tensor:
    """v2 zero-LDS skinny GEMM (M <= 64); splitk <= 0 = auto."""
    if x.is_cuda:
        _gpu()
        return torch.ops.rlli.skinny2_linear(x, w, splitk)
    return torch.nn.functional.linear(x, w)


def skinny2_silu_linear(gu: torch.Tensor, w: torch.Tensor,
                        splitk: int = 0) -> torch.Tensor:
    """Fused SwiGLU + down-proj: (silu(gu[:, :K]) * gu[:, K:]) @ w^T with
    the activation computed inside the GEMM's A-fragment loads — deletes
    the silu_mul launch and its intermediate tensor."""
    if gu.is_cuda:
        _gpu()
        return torch.ops.rlli.skinny2_silu_linear(gu, w, splitk)
    return torch.nn.functional.linear(ref.silu_mul(gu), w)


build_cos_sin = ref.build_cos_sin
yarn_cos_sin = ref.yarn_cos_sin


# ----------------------------------------------- mixed-layer model ops
# f32 or bf16 activations.  On the GPU one namespace per kernel library
# (build.py), on the CPU one ref_*.py each.
from . import ref_attn, ref_blk, ref_lat, ref_mix, ref_rec  # noqa: E402
from .ref_rec import REC_CHUNK  # noqa: E402

_CPU_FORMS = {"rlli_attn": ref_attn, "rlli_mix": ref_mix,
              "rlli_blk": ref_blk, "rlli_rec": ref_rec, "rlli_lat": ref_lat}


def _ns(lib: str, t: torch.Tensor):
    """The op namespace of ``lib`` for ``t``'s device."""
    if t.is_cuda:
        load_libraries((lib,))
        return getattr(torch.ops, lib)
    return _CPU_FORMS[lib]


def _mix(t: torch.Tensor):
    return _ns("rlli_mix", t)


def hyper_embed(ids, table, w_embed, x, in_w, gain, eps: float):
    """Fill the streams with the normed embedding; returns the normed
    input of the first sublayer.  Gains multiply (1 + w is folded in)."""
    return _mix(table).hyper_embed(ids, table, w_embed, x, in_w, gain, eps)


def hyper_step(x, y, mix, out_w, in_w, gain, eps: float, rows=None,
               keep: bool = True):
    """Write one sublayer's output into the streams and return the normed
    input of the next (``in_w`` None: the plain stream sum).  ``y`` may be
    [T, parts, W]; ``rows`` restricts the result (then keep=False)."""
    return _mix(y).hyper_step(x, y, mix, out_w, in_w, gain, eps, rows, keep)


def relu2(x):
    return _mix(x).relu2(x)


def window_tile_rows(group: int, device) -> int:
    """Prompt-tile height that the tiled attention kernel wants."""
    if torch.device(device).type == "cuda":
        load_libraries(("rlli_mix",))
        return torch.ops.rlli_mix.window_tile_rows(group)
    return 32


def window_prefill(qkv, k_cache, v_cache, positions, cos_sin, slots,
                   block_tables, prompt, sink, scale: float, n_q: int,
                   window: int, keep_first: int, has_kv: bool):
    """Prompt rows: rotate, append to the cache (``has_kv``), attend."""
    if not qkv.is_cuda:
        return ref_attn.window_prefill(
            qkv, k_cache, v_cache, positions, cos_sin, slots, block_tables,
            prompt, sink, scale, n_q, window, keep_first, has_kv, None, None,
            0.0, 0, None)
    attn = _ns("rlli_attn", qkv)
    attn.window_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                       has_kv, None)
    mask = (sink, scale, n_q, window, keep_first, has_kv)
    if attn.window_fast(k_cache, v_cache, qkv.dtype == torch.float32):
        h = window_tile_rows(n_q // k_cache.shape[1], qkv.device)
        return _mix(qkv).window_tiled(qkv, k_cache, v_cache, block_tables,
                                      prompt.tiles(h), h, *mask)
    return attn.window_rows(qkv, k_cache, v_cache, block_tables,
                            prompt.tiles(32), 32, *mask, None, None, 0.0, 0)


def window_decode(qkv, k_cache, v_cache, positions, cos_sin, slots,
                  block_tables, sink, scale: float, n_q: int, window: int,
                  keep_first: int, has_kv: bool):
    """One new token per sequence: rotation, append and attention fused."""
    return _ns("rlli_attn", qkv).window_decode(
        qkv, k_cache, v_cache, positions, cos_sin, slots, block_tables, sink,
        scale, n_q, window, keep_first, has_kv, None, None, 0.0, 0, None)


FULL = 1 << 30        # a window that never ends


def biased_decode(qkv, k_cache, v_cache, positions, slots, block_tables,
                  scale: float, n_q: int, r1, r2, temp_coef: float,
                  temp_every: int, v_eps=None):
    """Causal attention without rotation: a score loses r1 ln(1 + r2
    distance), queries are multiplied by 1 + temp_coef ln((p + 1) //
    temp_every + 1), values cached over their root mean square (``v_eps``).
    One new token per sequence, append included."""
    return _ns("rlli_attn", qkv).window_decode(
        qkv, k_cache, v_cache, positions, None, slots, block_tables, None,
        scale, n_q, FULL, 0, True, r1, r2, temp_coef, temp_every, v_eps)


def biased_prefill(qkv, k_cache, v_cache, positions, slots, block_tables,
                   prompt, scale: float, n_q: int, r1, r2, temp_coef: float,
                   temp_every: int, v_eps=None):
    """The same for prompt rows: append, then attend over the sequence's
    gathered keys and values (sizes that the tiled kernel does not take:
    over the pages, row by row)."""
    score = (r1, r2, temp_coef, temp_every)
    if not qkv.is_cuda:
        return ref_attn.window_prefill(
            qkv, k_cache, v_cache, positions, None, slots, block_tables,
            prompt, None, scale, n_q, FULL, 0, True, *score, v_eps)
    attn = _ns("rlli_attn", qkv)
    attn.window_append(qkv, k_cache, v_cache, positions, None, slots, n_q,
                       True, v_eps)
    _, n_kv, _, dim = k_cache.shape
    vdim = v_cache.shape[3]
    if qkv.dtype == torch.float32 or not attn.expanded_ok(dim, vdim):
        return attn.window_rows(qkv, k_cache, v_cache, block_tables,
                                prompt.tiles(32), 32, None, scale, n_q, FULL,
                                0, True, *score)
    blocks, kv_off, tokens = prompt.gathered(64)
    k, vt = attn.kv_gather(k_cache, v_cache, block_tables, blocks, tokens)
    out = torch.empty((qkv.shape[0], n_q * vdim), dtype=qkv.dtype,
                      device=qkv.device)
    attn.expanded_attn(qkv[:, :n_q * dim], k, vt, None, prompt.tiles(128),
                       kv_off, n_q, n_kv, scale, out, *score)
    return out


def diff_decode(qkv, gate, k_cache, v_cache, positions, cos_sin, slots,
                block_tables, n_q: int, bias, q_norm, k_norm, scale: float,
                chunk: int, cap: float, lam: float, out_scale: float,
                eps: float):
    """Differential attention, one new token per sequence, append included.
    ``qkv``: q | k | v | .., ``bias`` added to the three; a head's query and
    key are two maps side by side, each normed and rotated (pairs i, i + rot
    / 2); scores capped; a query sees its chunk of positions; the maps'
    outputs a1 - lam a2 over their root mean square, times out_scale and the
    sigmoid of ``gate`` [rows, n_q]."""
    return _ns("rlli_attn", qkv).diff_decode(
        qkv, k_cache, v_cache, positions, cos_sin, slots, block_tables, gate,
        scale, n_q, bias, q_norm, k_norm, chunk, cap, lam, out_scale, eps)


def diff_prefill(qkv, gate, k_cache, v_cache, positions, cos_sin, slots,
                 block_tables, prompt, n_q: int, bias, q_norm, k_norm,
                 scale: float, chunk: int, cap: float, lam: float,
                 out_scale: float, eps: float):
    """The same for prompt rows: append, then attend over what the rows'
    chunks hold, gathered (sizes that the tiled kernel does not take: over
    the pages, row by row)."""
    if not qkv.is_cuda:
        return ref_attn.diff_prefill(
            qkv, gate, k_cache, v_cache, positions, cos_sin, slots,
            block_tables, prompt, n_q, bias, q_norm, k_norm, scale, chunk,
            cap, lam, out_scale, eps)
    attn = _ns("rlli_attn", qkv)
    attn.diff_append(qkv, k_cache, v_cache, positions, cos_sin, slots, n_q,
                     bias, q_norm, k_norm, eps)
    tail = (chunk, cap, lam, out_scale, eps)
    _, n_kv, _, width = k_cache.shape
    vdim = v_cache.shape[3]
    if (qkv.dtype == torch.float32 or qkv.shape[1] % 8
            or not attn.expanded_ok(width // 2, vdim, 2)):
        return attn.diff_rows(qkv, k_cache, v_cache, block_tables,
                              prompt.tiles(32), 32, gate, scale, n_q, *tail)
    blocks, kv_off, tokens = prompt.gathered(64, chunk)
    k, vt = attn.kv_gather(k_cache, v_cache, block_tables, blocks, tokens)
    out = torch.empty((qkv.shape[0], n_q * vdim), dtype=qkv.dtype,
                      device=qkv.device)
    attn.diff_expanded(qkv[:, :n_q * width], k, vt, gate, prompt.tiles(128),
                       kv_off, n_q, n_kv, scale, out, *tail)
    return out


def _out(proj, state, vdim, out):
    if out is not None:
        return out
    return torch.empty((proj.shape[0], state.shape[1] * vdim),
                       dtype=proj.dtype, device=proj.device)


def gla_decode(proj, a2, a2_bias, norm, state, slots, positions, vdim: int,
               tau: float, eps: float, out=None):
    """Gated linear attention, one new token per sequence.  ``out`` may be
    a column range of a wider matrix."""
    out = _out(proj, state, vdim, out)
    _ns("rlli_rec", proj).gla_decode(proj, a2, a2_bias, norm, state, slots,
                                     positions, vdim, tau, eps, out)
    return out


def gla_prefill(proj, a2, a2_bias, norm, state, prompt, vdim: int,
                tau: float, eps: float, out=None):
    out = _out(proj, state, vdim, out)
    _ns("rlli_rec", proj).gla_prefill(
        proj, a2, a2_bias, norm, state, prompt.tiles(REC_CHUNK),
        prompt.seqs(REC_CHUNK), vdim, tau, eps, out)
    return out


def hgrn2_decode(proj, bias, lower, norm, state, slots, positions, vdim: int,
                 eps: float, out=None):
    """HGRN2: the same recurrence with k = 1 - decay, silu queries and a
    lower-bounded decay; ``proj`` is q | forget logit | v."""
    out = _out(proj, state, vdim, out)
    _ns("rlli_rec", proj).hgrn2_decode(proj, bias, lower, norm, state, slots,
                                       positions, vdim, eps, out)
    return out


def hgrn2_prefill(proj, bias, lower, norm, state, prompt, vdim: int,
                  eps: float, out=None):
    out = _out(proj, state, vdim, out)
    _ns("rlli_rec", proj).hgrn2_prefill(
        proj, bias, lower, norm, state, prompt.tiles(REC_CHUNK),
        prompt.seqs(REC_CHUNK), vdim, eps, out)
    return out


def rwkv_decode(rkvg, low, w2, w0, bonus, norm, state, slots, positions,
                eps: float, out):
    """RWKV-style recurrence, one new token per sequence: ``rkvg`` [4, rows,
    heads * dim], decay e^(-e^(w2 tanh(low) + w0)), bonus for the present
    token, norm over a head, silu gate."""
    _ns("rlli_rec", rkvg).rwkv_decode(rkvg, low, w2, w0, bonus, norm, state,
                                      slots, positions, eps, out)
    return out


def rwkv_prefill(rkvg, low, w2, w0, bonus, norm, state, prompt, eps: float,
                 out):
    _ns("rlli_rec", rkvg).rwkv_prefill(
        rkvg, low, w2, w0, bonus, norm, state, prompt.tiles(REC_CHUNK),
        prompt.seqs(REC_CHUNK), eps, out)
    return out


def delta_decode(proj, taps, tail, a_rate, dt_bias, norm, state, slots,
                 positions, kv_heads: int, vdim: int, eps: float, out):
    """Gated delta rule, one new token per sequence, convolution of
    q | k | v included.  ``proj``: q | k | v | gate | beta | decay."""
    _ns("rlli_rec", proj).delta_decode(
        proj, taps, tail, a_rate, dt_bias, norm, state, slots, positions,
        kv_heads, vdim, eps, out)
    return out


def delta_prefill(proj, taps, tail, a_rate, dt_bias, norm, state, prompt,
                  kv_heads: int, vdim: int, eps: float, out):
    x = torch.empty((proj.shape[0], taps.shape[1]), dtype=proj.dtype,
                    device=proj.device)
    conv_prompt(proj[:, :taps.shape[1]], taps, tail, prompt, x, silu=True)
    _ns("rlli_rec", proj).delta_prefill(
        proj, x, a_rate, dt_bias, norm, state, prompt.tiles(REC_CHUNK),
        prompt.seqs(REC_CHUNK), kv_heads, vdim, eps, out)
    return out


def mlstm_decode(proj, i_bias, f_bias, norm, state, m, slots, positions,
                 vdim: int, cap: float, eps: float, out):
    """mLSTM, one new token per sequence.  ``proj``: q | k | v | gate | i |
    f; the state's last column is the normalizer, ``m`` the running
    maximum."""
    _ns("rlli_rec", proj).mlstm_decode(proj, i_bias, f_bias, norm, state, m,
                                       slots, positions, vdim, cap, eps, out)
    return out


def mlstm_prefill(proj, i_bias, f_bias, norm, state, m, prompt, vdim: int,
                  cap: float, eps: float, out):
    _ns("rlli_rec", proj).mlstm_prefill(
        proj, i_bias, f_bias, norm, state, m, prompt.tiles(REC_CHUNK),
        prompt.seqs(REC_CHUNK), vdim, cap, eps, out)
    return out


def moe_route(h, router, top: int):
    return _mix(h).moe_route(h, router, top)


def moe_experts(h, router, w_up, w_down, top: int, limit: float):
    """[T, top, W]: one row per chosen expert; the consumer sums them."""
    return _mix(h).moe_experts(h, router, w_up, w_down, top, limit)


def moe_route_softmax(h, router, correction, top: int, groups: int,
                      keep: int):
    return _mix(h).moe_route_softmax(h, router, correction, top, groups, keep)


def moe_relu2(h, router, correction, w_up, w_down, top: int, groups: int,
              keep: int):
    """Squared-relu experts.  Softmax over all routes; ``correction`` shifts
    the choice, which the best ``keep`` of ``groups`` groups of neighbours
    hold; weights sum to one.  Returns (y [T, top, W], ids, weights); routes
    past the experts are identities, whose rows of y are not written."""
    return _mix(h).moe_relu2(h, router, correction, w_up, w_down, top, groups,
                             keep)


# --------------------------------------------------- residual blocks
CONV_SPAN = 16        # prompt rows that one convolution workgroup walks


def block_embed(ids, table, pos_table, positions, x, gain, groups: int,
                eps: float, taps=None, tail=None, slots=None,
                n_decode: int = 0, scale: float = 1.0):
    """Fill the f32 residual with scaled embedding + position and return its
    grouped norm h and, for the first ``n_decode`` rows (one token per
    sequence), h + conv(h) from the sequences' tails.  ``taps`` [branches,
    taps, width] makes that [branches, rows, width]."""
    return _ns("rlli_blk", table).block_embed(
        ids, table, pos_table, positions, x, gain, groups, eps, taps, tail,
        slots, n_decode, scale)


def block_step(x, y, gain, groups: int, eps: float, positions, taps=None,
               tail=None, slots=None, n_decode: int = 0, rows=None,
               keep: bool = True, y2=None, gain1=None, gain2=None,
               part_ids=None, part_w=None, part_h=None, part_limit: int = 0,
               y_bias=None):
    """Add a block's output to the residual; then as block_embed.  ``rows``
    restricts the result (then keep=False).  With ``y2`` half the sum of
    both outputs is added, each normed first (``gain1``, ``gain2``).  With
    ``part_ids`` [T, parts] the sum over y [T, parts, W] is added, where a
    part whose id is ``part_limit`` or more is part_w part_h instead.
    ``y_bias`` [W] goes with a single output."""
    return _ns("rlli_blk", y).block_step(x, y, gain, groups, eps, positions,
                                         taps, tail, slots, n_decode, rows,
                                         keep, y2, gain1, gain2, part_ids,
                                         part_w, part_h, part_limit, y_bias)


def conv_prompt(h, taps, tail, prompt, out, silu: bool = False):
    """out = h + conv(h), or silu(conv(h)), for prompt rows, and their
    sequences' tails.  Branches as in block_embed."""
    _ns("rlli_blk", h).conv_prompt(h, taps, tail, prompt.spans(CONV_SPAN),
                                   prompt.spans(1 << 30), out, silu)


def gate_act(gate_up, out, act: str, limit: float = 0.0):
    """out = act(gate) * up of [rows, gate | up]; act 'clamp_glu': g
    sigmoid(1.702 g) (u + 1) with g <= limit, |u| <= limit."""
    _ns("rlli_blk", gate_up).gate_act(gate_up, out, act, limit)
    return out


def soft_cap(x, cap: float):
    """cap * tanh(x / cap), 32-bit."""
    return _ns("rlli_blk", x).soft_cap(x, cap)


# ------------------------------------------------------------- latents
LATENT_VECTORS = 32   # (row, head) queries of one absorbed prompt tile


def latent_prep(proj, q_norm, kv_norm, eps: float, cache, slots):
    """Norm both latents of ``proj`` (query | key/value | ...), cache the
    second, return the first."""
    return _ns("rlli_lat", proj).latent_prep(proj, q_norm, kv_norm, eps,
                                             cache, slots)


def head_linear(x, w, gate=None, out=None):
    """out[t, h] = w[h] x[t, h] (times sigmoid(gate)); w [heads, n, k]."""
    if out is None:
        out = torch.empty((x.shape[0], w.shape[0] * w.shape[1]),
                          dtype=x.dtype, device=x.device)
    _ns("rlli_lat", w).head_linear(x, w, gate, out)
    return out


def latent_decode(q, gate, cache, positions, block_tables, scale: float,
                  w_uk, w_uv, out):
    """One new token per sequence: absorbed queries over the cached
    latents.  w_uk [heads, rank, dim], w_uv [heads, vdim, rank]."""
    heads = w_uk.shape[0]
    ns = _ns("rlli_lat", q)
    c = ns.latent_attn(head_linear(q, w_uk), cache, block_tables, scale,
                       heads, positions, None, None)
    return head_linear(c, w_uv, gate, out)


def expands(prompt, rank: int, dim: int, vdim: int) -> bool:
    """Whether a step's prompt rows are cheaper with expanded keys and
    values: rebuilding them costs a fixed amount per cached token, a score
    and value row of latent width costs more per (row, token)."""
    absorbed = expanded = 0
    for p in prompt.portions:
        ctx = p.pos0 + p.n
        absorbed += p.n * ctx * 2 * rank
        expanded += ctx * (dim + vdim) * (rank + p.n)
    # the absorbed kernel reaches about half the expanded one's rate
    return 2 * absorbed > expanded


def latent_prefill(q, gate, cache, block_tables, prompt, scale: float, w_uk,
                   w_uv, w_k, w_v, out, expand=None):
    """Prompt rows over the cached latents, their own included: with keys
    and values expanded from the latents (w_k [heads * dim, rank], w_v
    [heads * vdim, rank]) or with absorbed queries, whichever is cheaper
    (``expand`` forces one)."""
    heads, rank, dim = w_uk.shape
    vdim = w_uv.shape[1]
    ns = _ns("rlli_lat", q)
    fast = q.is_cuda and ns.latent_fast(cache, q.dtype == torch.float32)
    attn = _ns("rlli_attn", q) if fast else None
    ok = fast and attn.expanded_ok(dim, vdim) and all(
        t.stride(0) % 4 == 0 and t.data_ptr() % 8 == 0 for t in (gate, out))
    if expand is None:
        expand = ok and expands(prompt, rank, dim, vdim)
    if expand and ok:
        blocks, kv_off, tokens = prompt.gathered(64)
        c = ns.latent_gather(cache, block_tables, blocks, tokens)
        k = torch.nn.functional.linear(c, w_k)
        vt = torch.nn.functional.linear(w_v, c)      # already transposed
        attn.expanded_attn(q, k, vt, gate, prompt.tiles(128), kv_off, heads,
                           heads, scale, out, None, None, 0.0, 0)
        return out
    tiles = prompt.vectors(LATENT_VECTORS, heads) if fast else prompt.tiles(32)
    c = ns.latent_attn(head_linear(q, w_uk), cache, block_tables, scale,
                       heads, None, tiles, prompt.pos0())
    return head_linear(c, w_uv, gate, out)
