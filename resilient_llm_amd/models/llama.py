"""Llama-family model, MI355X-first.

No nn.Module graph: a flat parameter store + an explicit forward written
against the serving ops — fused QKV / gate-up GEMMs through hipBLASLt
(torch.nn.functional.linear), everything between the GEMMs as hand-written
gfx950 kernels (resilient_llm_amd.ops): fused residual-add RMSNorm,
RoPE+paged-KV append, paged GQA decode attention, varlen prefill
attention, fused SwiGLU.  On CPU the same forward runs on the fp32
reference ops — that is the no-GPU test path.

The reference runs no model code at all (model execution lives inside
AWS Bedrock — SURVEY.md §0); targets here come from BASELINE.json:
Llama-3-8B bf16 as the flagship, Llama-3-70B TP=4 per pool.

Weight loading: random init (no-network default) or a safetensors
directory with HF Llama names.
"""

from __future__ import annotations

import dataclasses
import math
import os
from typing import Optional

import torch
import torch.nn.functional as F

from .. import ops
from ..ops import autotune as lt_autotune

# Opt-in: route decode-shaped GEMMs (M<=64) through the custom skinny-M
# MFMA kernel instead of hipBLASLt (A/B lever; see ops/csrc/skinny_gemm.hip)
_USE_SKINNY = os.environ.get("RLLI_SKINNY") == "1"


# Row counts that the measured-GEMM autotuner may tune: the decode graph
# buckets (+ the small row counts prefill's lm_head sees).  Anything else
# (prefill/mixed token counts — unbounded variety) goes straight to
# torch so the tuning cache stays finite.
_LT_ROWS = frozenset({1, 2, 4, 8, 12, 16, 24, 32, 48, 64, 96, 128})


def _linear(x, w):
    if _USE_SKINNY:
        return ops.linear_auto(x, w)
    if x.is_cuda and x.dim() == 2 and x.shape[0] in _LT_ROWS:
        return lt_autotune.tuned_linear(x, w)
    return F.linear(x, w)


@dataclasses.dataclass
class LlamaConfig:
    name: str
    hidden_size: int
    n_layers: int
    n_heads: int
    n_kv_heads: int
    head_dim: int
    intermediate_size: int
    vocab_size: int
    rope_theta: float = 500000.0
    rms_eps: float = 1e-5
    max_position: int = 8192
    tie_embeddings: bool = False
    # token ids that end generation (Llama-3: <|end_of_text|>=128001 and
    # <|eot_id|>=128009); overridable per deployment / by a real tokenizer
    eos_ids: tuple = (2,)

    @property
    def q_size(self) -> int:
        return self.n_heads * self.head_dim

    @property
    def kv_size(self) -> int:
        return self.n_kv_heads * self.head_dim


MODEL_PRESETS: dict[str, LlamaConfig] = {
    "llama-3-8b": LlamaConfig(
        name="llama-3-8b", hidden_size=4096, n_layers=32, n_heads=32,
        n_kv_heads=8, head_dim=128, intermediate_size=14336,
        vocab_size=128256, eos_ids=(128001, 128009)),
    "llama-3-70b": LlamaConfig(
        name="llama-3-70b", hidden_size=8192, n_layers=80, n_heads=64,
        n_kv_heads=8, head_dim=128, intermediate_size=28672,
        vocab_size=128256, eos_ids=(128001, 128009)),
    "llama-3-1b": LlamaConfig(
        # Llama-3.2-1B geometry: small-footprint replica for dense
        # multi-replica serving on one GPU (head_dim 64 path)
        name="llama-3-1b", hidden_size=2048, n_layers=16, n_heads=32,
        n_kv_heads=8, head_dim=64, intermediate_size=8192,
        vocab_size=128256, eos_ids=(128001, 128009)),
    "mistral-7b": LlamaConfig(
        # Mistral-7B-v0.3 geometry (no sliding window: full attention,
        # which is exact for contexts <= max_position)
        name="mistral-7b", hidden_size=4096, n_layers=32, n_heads=32,
        n_kv_heads=8, head_dim=128, intermediate_size=14336,
        vocab_size=32768, rope_theta=1000000.0),
    # CPU-testable models
    "tiny": LlamaConfig(
        name="tiny", hidden_size=256, n_layers=2, n_heads=4, n_kv_heads=2,
        head_dim=64, intermediate_size=512, vocab_size=512,
        max_position=2048),
    "tiny-128": LlamaConfig(
        name="tiny-128", hidden_size=512, n_layers=2, n_heads=4, n_kv_heads=1,
        head_dim=128, intermediate_size=1024, vocab_size=512,
        max_position=2048),
}


class LlamaForCausalLM:
    """Inference-only Llama.  TP sharding plugs in via `shard` (see
    resilient_llm_amd.parallel): rank/world split q/kv heads and the
    intermediate dim column-wise, o/down row-wise, with an all-reduce
    after o_proj and down_proj."""

    EXTENSIONS = ("rlli_hip",)

    def __init__(self, config: LlamaConfig, device: str = "cpu",
                 dtype: torch.dtype = torch.bfloat16,
                 tp_rank: int = 0, tp_world: int = 1,
                 tp_group=None, seed: int = 0,
                 quant: Optional[str] = None) -> None:
        self.config = config
        self.device = torch.device(device)
        self.dtype = dtype
        # quant="fp8": W8A8-fp8 for the three bandwidth-dominant
        # projections (gate_up, down, lm_head) — per-out-channel weight
        # scales + per-row dynamic activation scales emitted by the
        # fused rmsnorm/silu kernels, rowwise torch._scaled_mm compute
        # (hipBLASLt fp8 MFMA).  qkv/o stay bf16: measured 1.0x in fp8
        # at decode shapes (ramp-bound), so quantizing them buys
        # nothing and costs an attention-output quantization step.
        if quant not in (None, "fp8"):
            raise ValueError(f"quant must be None or 'fp8', got {quant!r}")
        self.quant = quant
        self.tp_rank = tp_rank
        self.tp_world = tp_world
        self.tp_group = tp_group
        c = config
        assert c.n_heads % tp_world == 0 and c.n_kv_heads % tp_world == 0, \
            f"TP={tp_world} must divide heads ({c.n_heads}/{c.n_kv_heads})"
        assert c.intermediate_size % tp_world == 0
        self.n_heads = c.n_heads // tp_world
        self.n_kv_heads = c.n_kv_heads // tp_world
        self.inter = c.intermediate_size // tp_world
        self.q_size = self.n_heads * c.head_dim
        self.kv_size = self.n_kv_heads * c.head_dim
        self.scale = 1.0 / math.sqrt(c.head_dim)
        self.params: dict[str, torch.Tensor] = {}
        self._init_weights(seed)
        if self.quant == "fp8":
            self._quantize_weights()
        self.cos_sin = ops.build_cos_sin(c.max_position, c.head_dim,
                                         c.rope_theta, device=self.device)

    # ------------------------------------------------------------ weights
    def _mk(self, name: str, shape: tuple, gen: torch.Generator,
            std: float = 0.02) -> None:
        t = torch.empty(shape, dtype=self.dtype, device=self.device)
        t.normal_(0.0, std, generator=gen)
        self.params[name] = t

    def _full(self, shape: tuple, gen: torch.Generator,
              std: float = 0.02) -> torch.Tensor:
        t = torch.empty(shape, dtype=self.dtype, device=self.device)
        t.normal_(0.0, std, generator=gen)
        return t

    def _init_weights(self, seed: int) -> None:
        """Every rank draws the FULL weight with the same seed and keeps
        its shard — so TP=N computes the same function as TP=1 (the
        gloo/CPU TP tests rely on this)."""
        c = self.config
        r, w = self.tp_rank, self.tp_world
        gen = torch.Generator(device=self.device)
        gen.manual_seed(seed + 1)
        self._mk("embed", (c.vocab_size, c.hidden_size), gen)
        std_o = 0.02 / math.sqrt(2 * c.n_layers)
        for i in range(c.n_layers):
            gen.manual_seed(seed * 1000003 + i * 1009)
            qkv = self._full((c.q_size + 2 * c.kv_size, c.hidden_size), gen)
            qf, kf, vf = torch.split(qkv, [c.q_size, c.kv_size, c.kv_size], dim=0)
            self.params[f"l{i}.qkv"] = torch.cat([
                qf[r * self.q_size:(r + 1) * self.q_size],
                kf[r * self.kv_size:(r + 1) * self.kv_size],
                vf[r * self.kv_size:(r + 1) * self.kv_size]], dim=0).contiguous()
            o = self._full((c.hidden_size, c.q_size), gen, std_o)
            self.params[f"l{i}.o"] = o[:, r * self.q_size:(r + 1) * self.q_size].contiguous()
            gu = self._full((2 * c.intermediate_size, c.hidden_size), gen)
            gf, uf = torch.split(gu, [c.intermediate_size, c.intermediate_size], dim=0)
            self.params[f"l{i}.gate_up"] = torch.cat([
                gf[r * self.inter:(r + 1) * self.inter],
                uf[r * self.inter:(r + 1) * self.inter]], dim=0).contiguous()
            down = self._full((c.hidden_size, c.intermediate_size), gen, std_o)
            self.params[f"l{i}.down"] = down[:, r * self.inter:(r + 1) * self.inter].contiguous()
            self.params[f"l{i}.ln1"] = torch.ones(c.hidden_size, dtype=self.dtype,
                                                  device=self.device)
            self.params[f"l{i}.ln2"] = torch.ones_like(self.params[f"l{i}.ln1"])
        gen.manual_seed(seed + 2)
        self.params["final_ln"] = torch.ones(c.hidden_size, dtype=self.dtype,
                                             device=self.device)
        if c.tie_embeddings:
            self.params["lm_head"] = self.params["embed"]
        else:
            self._mk("lm_head", (c.vocab_size, c.hidden_size), gen)

    def _quantize_weights(self) -> None:
        """Quantize gate_up/down/lm_head to fp8-e4m3 with per-out-channel
        scales and FREE the bf16 originals (8B: ~5.5 GiB back).  Called
        after random init and again after a safetensors load."""
        from ..ops import ref as _ref
        names = [f"l{i}.{n}" for i in range(self.config.n_layers)
                 for n in ("gate_up", "down")] + ["lm_head"]
        for name in names:
            w = self.params.get(name)
            if w is None or w.dtype != self.dtype:
                continue
            q, sc = _ref.quantize_fp8_rowwise(w)
            self.params[name + ".q8"] = q.contiguous()
            self.params[name + ".s"] = sc.to(torch.float32).contiguous()
            if name == "lm_head" and w is self.params.get("embed"):
                pass              # tied: keep the bf16 embed for lookups
            del self.params[name]

    def _linear_fp8(self, x8: torch.Tensor, xs: torch.Tensor,
                    name: str) -> torch.Tensor:
        w8 = self.params[name + ".q8"]
        ws = self.params[name + ".s"]
        if x8.is_cuda:
            return torch._scaled_mm(x8, w8.t(), scale_a=xs.reshape(-1, 1),
                                    scale_b=ws.reshape(1, -1),
                                    out_dtype=torch.bfloat16)
        from ..ops import ref as _ref
        return _ref.scaled_mm_ref(x8, xs, w8, ws)

    def load_safetensors(self, path: str) -> int:
        """Load HF-Llama-named safetensors shards, TP-sharded at load
        each rank takes its column slice of q/k/v and
        gate/up and its row slice of o/down — the exact layout
        ``_init_weights`` produces, so TP=N computes the same function as
        TP=1 on the same checkpoint.  Returns the number of tensors
        consumed.  (The reference runs real models in every pool —
        /root/reference/src/demo_account_sharding.py:202-224.)"""
        import safetensors.torch as st
        c = self.config
        r = self.tp_rank
        loaded = 0
        files = sorted(f for f in os.listdir(path) if f.endswith(".safetensors"))
        if not files:
            raise FileNotFoundError(f"no .safetensors files under {path}")
        raw: dict[str, torch.Tensor] = {}
        for f in files:
            raw.update(st.load_file(os.path.join(path, f)))

        def take(name, rows: Optional[int] = None, cols: Optional[int] = None):
            """Move to device taking only this rank's shard: ``rows`` =
            per-rank output rows (column-parallel), ``cols`` = per-rank
            input columns (row-parallel)."""
            nonlocal loaded
            t = raw[name]
            if rows is not None:
                t = t[r * rows:(r + 1) * rows]
            if cols is not None:
                t = t[:, r * cols:(r + 1) * cols]
            loaded += 1
            return t.to(self.dtype).to(self.device).contiguous()

        self.params["embed"] = take("model.embed_tokens.weight")
        for i in range(c.n_layers):
            p = f"model.layers.{i}."
            q = take(p + "self_attn.q_proj.weight", rows=self.q_size)
            k = take(p + "self_attn.k_proj.weight", rows=self.kv_size)
            v = take(p + "self_attn.v_proj.weight", rows=self.kv_size)
            self.params[f"l{i}.qkv"] = torch.cat([q, k, v], dim=0).contiguous()
            self.params[f"l{i}.o"] = take(p + "self_attn.o_proj.weight",
                                          cols=self.q_size)
            g = take(p + "mlp.gate_proj.weight", rows=self.inter)
            u = take(p + "mlp.up_proj.weight", rows=self.inter)
            self.params[f"l{i}.gate_up"] = torch.cat([g, u], dim=0).contiguous()
            self.params[f"l{i}.down"] = take(p + "mlp.down_proj.weight",
                                             cols=self.inter)
            self.params[f"l{i}.ln1"] = take(p + "input_layernorm.weight")
            self.params[f"l{i}.ln2"] = take(p + "post_attention_layernorm.weight")
        self.params["final_ln"] = take("model.norm.weight")
        if "lm_head.weight" in raw:
            self.params["lm_head"] = take("lm_head.weight")
        else:
            self.params["lm_head"] = self.params["embed"]
        if self.quant == "fp8":
            self._quantize_weights()
        return loaded

    def save_safetensors(self, path: str) -> None:
        if self.quant is not None:
            raise RuntimeError("cannot save a weight-quantized model "
                               "(bf16 originals were freed)")
        """Write the FULL (unsharded) weights in HF-Llama naming — the
        round-trip fixture for the TP-sharded-load tests.  TP=1 only."""
        import safetensors.torch as st
        assert self.tp_world == 1, "save from an unsharded model"
        c = self.config
        out: dict[str, torch.Tensor] = {}
        out["model.embed_tokens.weight"] = self.params["embed"]
        for i in range(c.n_layers):
            p = f"model.layers.{i}."
            qkv = self.params[f"l{i}.qkv"]
            q, k, v = torch.split(qkv, [c.q_size, c.kv_size, c.kv_size], dim=0)
            out[p + "self_attn.q_proj.weight"] = q
            out[p + "self_attn.k_proj.weight"] = k
            out[p + "self_attn.v_proj.weight"] = v
            out[p + "self_attn.o_proj.weight"] = self.params[f"l{i}.o"]
            gu = self.params[f"l{i}.gate_up"]
            g, u = torch.split(gu, [c.intermediate_size, c.intermediate_size], dim=0)
            out[p + "mlp.gate_proj.weight"] = g
            out[p + "mlp.up_proj.weight"] = u
            out[p + "mlp.down_proj.weight"] = self.params[f"l{i}.down"]
            out[p + "input_layernorm.weight"] = self.params[f"l{i}.ln1"]
            out[p + "post_attention_layernorm.weight"] = self.params[f"l{i}.ln2"]
        out["model.norm.weight"] = self.params["final_ln"]
        if self.params["lm_head"] is not self.params["embed"]:
            out["lm_head.weight"] = self.params["lm_head"]
        os.makedirs(path, exist_ok=True)
        st.save_file({k: v.contiguous().cpu() for k, v in out.items()},
                     os.path.join(path, "model.safetensors"))

    def param_bytes(self) -> int:
        seen = set()
        total = 0
        for t in self.params.values():
            if id(t) not in seen:
                seen.add(id(t))
                total += t.numel() * t.element_size()
        return total

    # ------------------------------------------------------------ compute
    def _all_reduce(self, x: torch.Tensor) -> torch.Tensor:
        if self.tp_world > 1:
            import torch.distributed as dist
            dist.all_reduce(x, group=self.tp_group)
        return x

    def _layer(self, i: int, x: torch.Tensor, residual: Optional[torch.Tensor],
               positions: torch.Tensor, kv_cache, slot_mapping: torch.Tensor,
               attn_fn) -> tuple[torch.Tensor, torch.Tensor]:
        p = self.params
        c = self.config
        if residual is None:
            residual = x.clone()
            h = ops.rmsnorm(x, p[f"l{i}.ln1"], c.rms_eps)
        else:
            h = ops.rmsnorm_residual_(x, residual, p[f"l{i}.ln1"], c.rms_eps)
        qkv = _linear(h, p[f"l{i}.qkv"])
        k_cache, v_cache = kv_cache.layer(i)
        # rope + cache append happen inside attn_fn (the decode path fuses
        # them into the attention kernel itself)
        attn_out = attn_fn(i, qkv, k_cache, v_cache)   # [T, q_size]
        h = self._all_reduce(_linear(attn_out, p[f"l{i}.o"]))
        if self.quant == "fp8":
            h2q, h2s = ops.rmsnorm_residual_fp8(h, residual, p[f"l{i}.ln2"],
                                                c.rms_eps)
            gu = self._linear_fp8(h2q, h2s, f"l{i}.gate_up")
            dq, ds = ops.silu_mul_fp8(gu)
            mlp = self._all_reduce(self._linear_fp8(dq, ds, f"l{i}.down"))
            return mlp, residual
        h2 = ops.rmsnorm_residual_(h, residual, p[f"l{i}.ln2"], c.rms_eps)
        gu = _linear(h2, p[f"l{i}.gate_up"])
        mlp = self._all_reduce(_linear(ops.silu_mul(gu), p[f"l{i}.down"]))
        return mlp, residual

    def forward_prefill(self, input_ids: torch.Tensor, positions: torch.Tensor,
                        kv_cache, slot_mapping: torch.Tensor,
                        cu_seqlens: torch.Tensor) -> torch.Tensor:
        """Returns logits for the LAST token of each sequence:
        [n_seqs, vocab]."""
        def attn(i, qkv, k_cache, v_cache):
            ops.rope_kv_append_qkv_(qkv, positions, self.cos_sin, k_cache,
                                    v_cache, slot_mapping, self.n_heads)
            return ops.prefill_attn_qkv(qkv, cu_seqlens, self.scale,
                                        self.n_heads, self.n_kv_heads,
                                        self.config.head_dim)
        return self._forward(input_ids, positions, kv_cache, slot_mapping,
                             attn, last_idx=cu_seqlens[1:].long() - 1)

    def forward_mixed(self, input_ids: torch.Tensor, positions: torch.Tensor,
                      kv_cache, slot_mapping: torch.Tensor, n_decode: int,
                      block_tables_dec, seq_lens_dec,
                      chunk_row0, chunk_pos0, chunk_nrows, chunk_btrow,
                      block_tables_pre, sample_idx) -> torch.Tensor:
        """Mixed batch: rows [0, n_decode) are decode tokens, the rest
        are prefill-chunk tokens attending over the paged cache
        (chunked prefill).  Returns logits for ``sample_idx`` rows."""
        def attn(i, qkv, k_cache, v_cache):
            ops.rope_kv_append_qkv_(qkv, positions, self.cos_sin, k_cache,
                                    v_cache, slot_mapping, self.n_heads)
            out = ops.prefill_paged_attn(
                qkv, k_cache, v_cache, chunk_row0, chunk_pos0, chunk_nrows,
                chunk_btrow, block_tables_pre, self.scale, self.n_heads)
            if n_decode:
                out_d = ops.decode_attn_qkv(
                    qkv[:n_decode], k_cache, v_cache, block_tables_dec,
                    seq_lens_dec, self.scale, self.n_heads)
                out[:n_decode] = out_d
            return out
        return self._forward(input_ids, positions, kv_cache, slot_mapping,
                             attn, last_idx=sample_idx)

    def forward_decode(self, input_ids: torch.Tensor, positions: torch.Tensor,
                       kv_cache, slot_mapping: torch.Tensor,
                       block_tables: torch.Tensor,
                       seq_lens: torch.Tensor) -> torch.Tensor:
        """One token per sequence; returns [batch, vocab] logits."""
        def attn(i, qkv, k_cache, v_cache):
            return ops.decode_attn_rope_qkv(
                qkv, positions, self.cos_sin, k_cache, v_cache, slot_mapping,
                block_tables, seq_lens, self.scale, self.n_heads)
        return self._forward(input_ids, positions, kv_cache, slot_mapping,
                             attn, last_idx=None)

    def _forward(self, input_ids, positions, kv_cache, slot_mapping, attn_fn,
                 last_idx) -> torch.Tensor:
        p = self.params
        x = F.embedding(input_ids.long(), p["embed"])
        residual = None
        for i in range(self.config.n_layers):
            x, residual = self._layer(i, x, residual, positions, kv_cache,
                                      slot_mapping, attn_fn)
        if self.quant == "fp8":
            h8, hs = ops.rmsnorm_residual_fp8(x, residual, p["final_ln"],
                                              self.config.rms_eps)
            if last_idx is not None:
                h8 = h8[last_idx]
                hs = hs[last_idx]
            return self._linear_fp8(h8, hs, "lm_head")
        h = ops.rmsnorm_residual_(x, residual, p["final_ln"],
                                  self.config.rms_eps)
        if last_idx is not None:
            h = h[last_idx]
        return _linear(h, p["lm_head"])   # bf16 logits feed ops.sample
