"""HIP decode engine: sequences the hand-written CDNA4 kernels for one
pipeline stage's per-token decode step.

This is the MI355X-native replacement for the reference's per-token PyTorch
forward (/root/reference/src/sub/submodels.py:170-282 driven by
gptserver.py:788-1110).  One engine serves every in-flight sample: the
sample slot and sequence position are *device* scalars, so the whole block
stack is captured once as a hipGraph and replayed per token regardless of
which sample is flowing through (reference swaps per-sample cache objects
into the modules instead — gptserver.py:975-978).

Supported natively: RMSNorm/LayerNorm, rope/learned positions, GQA
attention (head_size multiple of 32, head_size*q_per_kv >= 64), LLaMA
(SwiGLU) / Gemma / GPT-NeoX MLPs, sequential and parallel residual.
MoE decodes natively (device-side routing); fp8+MoE is refused.
"""

from __future__ import annotations

import os
from typing import Optional

import torch

from ..config import ModelConfig
from ..models.model import KVCachePool
from . import require_hip_ops

__all__ = ["DecodeEngine", "engine_supported"]


def engine_supported(config: ModelConfig) -> bool:
    if config.mlp_class_name == "LLaMAMoE" and (
        config.n_expert > 64 or config.n_expert_per_token > 8
        or config.norm_class_name != "RMSNorm"
    ):
        return False
    if config.head_size % 32 != 0 or config.head_size * config.q_per_kv < 64:
        return False
    if config.head_size not in (64, 128, 256):
        return False
    if config.q_per_kv not in (1, 2, 4, 8, 16):
        return False  # attention kernel instantiations (e.g. falcon-7b's
        # 71 q-heads per kv head run on the torch path)
    if config.n_embd % 8 != 0 or (config.intermediate_size or 0) % 8 != 0:
        return False
    return True


def quantize_fp8_rowwise(w: torch.Tensor):
    """bf16 [M,K] -> (fp8 e4m3 tensor, fp32 per-row scales).  OCP e4m3
    (torch.float8_e4m3fn == gfx950's fp8) with absmax/448 scaling."""
    wf = w.float()
    s = (wf.abs().amax(dim=1).clamp(min=1e-12) / 448.0).float()
    q = (wf / s[:, None]).to(torch.float8_e4m3fn)
    return q.contiguous(), s.contiguous()


class _BlockWeights:
    """Contiguous bf16 views of one block's parameters."""

    def __init__(self, block, config: ModelConfig):
        def p(t):
            if t is None:
                return None
            assert t.dtype == torch.bfloat16, "engine requires bf16 weights"
            return t.detach().contiguous()

        self.norm1_w = p(block.norm_1.weight)
        self.norm1_b = p(getattr(block.norm_1, "bias", None))
        self.attn_w = p(block.attn.attn.weight)
        self.attn_b = p(block.attn.attn.bias)
        self.proj_w = p(block.attn.proj.weight)
        self.proj_b = p(block.attn.proj.bias)
        if block.norm_2 is not None:
            self.norm2_w = p(block.norm_2.weight)
            self.norm2_b = p(getattr(block.norm_2, "bias", None))
        else:
            self.norm2_w = self.norm2_b = None
        mlp = block.mlp
        if config.mlp_class_name == "LLaMAMoE":
            # stacked expert slabs: the router index (device memory)
            # offsets into these at graph-replay time
            self.gate_w = p(mlp.gate.weight)
            self.fc1_w = torch.stack(
                [p(e.fc_1.weight) for e in mlp.experts]).contiguous()
            self.fc2_w = torch.stack(
                [p(e.fc_2.weight) for e in mlp.experts]).contiguous()
            self.mlp_proj_w = torch.stack(
                [p(e.proj.weight) for e in mlp.experts]).contiguous()
            self.mlp_proj_b = None
        elif config.mlp_class_name in ("LLaMAMLP", "GemmaMLP"):
            self.fc1_w = p(mlp.fc_1.weight)
            self.fc2_w = p(mlp.fc_2.weight)
            self.mlp_proj_w = p(mlp.proj.weight)
            self.mlp_proj_b = p(mlp.proj.bias)
        else:  # GptNeoxMLP
            self.fc_w = p(mlp.fc.weight)
            self.fc_b = p(mlp.fc.bias)
            self.mlp_proj_w = p(mlp.proj.weight)
            self.mlp_proj_b = p(mlp.proj.bias)

    def quantize_fp8(self, config) -> None:
        """Attach fp8 copies + per-row scales for the decode GEMVs."""
        if config.mlp_class_name == "LLaMAMoE":
            raise ValueError("fp8 weights are not supported for MoE stages")
        self.attn_w8, self.attn_s = quantize_fp8_rowwise(self.attn_w)
        self.proj_w8, self.proj_s = quantize_fp8_rowwise(self.proj_w)
        self.mlp_proj_w8, self.mlp_proj_s = quantize_fp8_rowwise(
            self.mlp_proj_w)
        if config.mlp_class_name in ("LLaMAMLP", "GemmaMLP"):
            self.fc1_w8, self.fc1_s = quantize_fp8_rowwise(self.fc1_w)
            self.fc2_w8, self.fc2_s = quantize_fp8_rowwise(self.fc2_w)
        else:
            self.fc_w8, self.fc_s = quantize_fp8_rowwise(self.fc_w)


class DecodeEngine:
    """Drives the HIP kernels for a stage (Starter or Secondary module)."""

    def __init__(
        self,
        stage,
        kv_pool: KVCachePool,
        n_chunks: int = 16,
        use_graphs: bool = True,
        expected_s: "int | None" = None,
    ) -> None:
        # adaptive split-S: 16 chunks up to 4k contexts (measured best at
        # short S; the one-launch block-local kernel is used there anyway),
        # then one wave per 32 keys capped at 256 chunks — 8 kv-heads x
        # 256 chunks = 2048 waves = 8/CU, the full wave occupancy (128
        # chunks measured only ~0.6 TB/s of KV streaming at S=8192: half
        # the waves, 4 serial tiles each)
        # expected_s: the caller's upper bound on the sequence length this
        # engine will actually decode at (prompt + tokens).  The one-launch
        # block-local attention (grid = n_kv_heads blocks) wins at short S
        # by the launch floor but serializes at S >~ 500 (measured: +2% at
        # S~166, -14% at S~1900 vs split-S) — when the caller knows the
        # generation runs past the crossover, force the split-S + combine
        # path even at max_seq <= 4096
        self.force_split = 1 if (expected_s is not None
                                 and expected_s >= 512) else 0
        default_chunks = max(16, min(256, stage.max_seq_length // 32))
        if stage.max_seq_length <= 4096 and not self.force_split:
            default_chunks = 16
        if n_chunks == 16:
            n_chunks = default_chunks
        n_chunks = int(os.environ.get("MDI_ATTN_CHUNKS", n_chunks))
        n_chunks = max(4, (n_chunks // 4) * 4)  # block-shared q staging
        self.weight_dtype = os.environ.get("MDI_WEIGHT_DTYPE", "bf16")
        self.kv_dtype = os.environ.get("MDI_KV_DTYPE", "bf16")
        self.ops = require_hip_ops()
        self.config: ModelConfig = stage.config
        cfg = self.config
        if not engine_supported(cfg):
            raise ValueError(f"config {cfg.name!r} unsupported by DecodeEngine")
        self.stage = stage
        self.kv_pool = kv_pool
        self.n_chunks = n_chunks
        self.device = next(stage.parameters()).device
        self.is_starter = hasattr(stage, "lm_head")
        self.use_graphs = use_graphs and self.device.type == "cuda"

        dev = self.device
        self.blocks = [_BlockWeights(b, cfg) for b in stage.transformer.h]
        self.fp8 = (self.weight_dtype == "fp8"
                    and self.device.type == "cuda")
        if self.fp8:
            for w in self.blocks:
                w.quantize_fp8(cfg)
        if self.is_starter:
            self.wte = stage.transformer.wte.weight.detach().contiguous()
            self.lnf_w = stage.transformer.ln_f.weight.detach().contiguous()
            self.lnf_b = getattr(stage.transformer.ln_f, "bias", None)
            if self.lnf_b is not None:
                self.lnf_b = self.lnf_b.detach().contiguous()
            self.head_w = stage.lm_head.weight.detach().contiguous()
            if self.fp8:
                self.head_w8, self.head_s = quantize_fp8_rowwise(self.head_w)
            self.head_b = stage.lm_head.bias
            if self.head_b is not None:
                self.head_b = self.head_b.detach().contiguous()
            self.wpe = None
            if cfg.pos_embedding == "learned":
                self.wpe = stage.transformer.wpe.weight.detach().contiguous()

        # rope tables fp32 (stage buffers, already on device)
        self.cos = stage.cos.detach().to(torch.float32).contiguous()
        self.sin = stage.sin.detach().to(torch.float32).contiguous()

        # ---- workspace ----------------------------------------------------
        bf = dict(device=dev, dtype=torch.bfloat16)
        E, I = cfg.n_embd, cfg.intermediate_size
        n_head, hs = cfg.n_head, cfg.head_size
        self.x = torch.zeros(E, **bf)        # residual stream (graph input)
        self.qkv = torch.zeros(cfg.qkv_dim, **bf)
        self.y = torch.zeros(n_head * hs, **bf)   # attention output
        self.a = torch.zeros(E, **bf)        # proj(attn) (+x)
        self.act = torch.zeros(I, **bf)
        self.m_out = torch.zeros(E, **bf)
        if cfg.mlp_class_name == "LLaMAMoE":
            self.xn = torch.zeros(E, **bf)
            self.gate_logits = torch.zeros(cfg.n_expert, **bf)
            self.moe_eidx = torch.zeros(cfg.n_expert_per_token, device=dev,
                                        dtype=torch.int32)
            self.moe_escale = torch.zeros(cfg.n_expert_per_token, device=dev,
                                          dtype=torch.float32)
        self.part_o = torch.zeros(
            n_head * n_chunks * hs, device=dev, dtype=torch.float32
        )
        self.part_ml = torch.zeros(
            n_head * n_chunks * 2, device=dev, dtype=torch.float32
        )
        if self.is_starter:
            self.logits = torch.zeros(cfg.padded_vocab_size, **bf)
            self.token = torch.zeros(1, device=dev, dtype=torch.int32)
            self.pos_emb = torch.zeros(E, **bf)

        if self.is_starter:
            # fused sampler state
            self.sample_scratch = torch.zeros(520, device=dev,
                                              dtype=torch.int32)
            self.sample_out = torch.zeros(1, device=dev, dtype=torch.int32)

        # device-side slot/pos scalars (graph-replayable)
        self.slot = torch.zeros(1, device=dev, dtype=torch.int32)
        self.pos_table = torch.zeros(
            kv_pool.n_slots, device=dev, dtype=torch.int32
        )
        self.pos = torch.zeros(1, device=dev, dtype=torch.int32)

        # fp8 (OCP e4m3) KV cache: halves KV-read bandwidth at long
        # context and halves cache memory per sample.  Per-row scales;
        # written only by the HIP kernels, so it requires the HIP prefill
        # path (torch prefill would need to append bf16 rows).
        self.kv8 = (
            self.kv_dtype == "fp8"
            and self.device.type == "cuda"
            and self.supports_hip_prefill
        )
        if self.kv_dtype == "fp8" and not self.kv8:
            import warnings

            warnings.warn(
                f"MDI_KV_DTYPE=fp8 ignored for {cfg.name!r}: the fp8 KV "
                "cache needs the HIP prefill path (RMSNorm + LLaMA/Gemma "
                "MLP, sequential residual)"
            )
        if self.kv8:
            kv_pool.to_fp8()

        # fused attention+proj (one launch, in-launch granule hand-off):
        # the proj weight stream overlaps the attention compute instead of
        # serializing behind it (attn_proj_kernel in decode_kernels.hip).
        # MEASURED OFF by default: on Llama-3-8B the attention role
        # stretches ~2x under the co-resident staging traffic (23 us fused
        # vs 9.4 + 8.7 split once the split proj got its 4-deep load
        # pipeline); opt in with MDI_FUSE_ATTN_PROJ=1.
        K_attn = cfg.n_head * cfg.head_size
        self._fuse_attn_proj = (
            not self.fp8
            and not self.kv8
            and not cfg.parallel_residual
            and stage.max_seq_length <= 4096
            and K_attn % 128 == 0
            and K_attn // 2 <= 4096
            and os.environ.get("MDI_FUSE_ATTN_PROJ", "0") == "1"
        )
        if self._fuse_attn_proj:
            # per-layer hand-off scratch: [K/2 y pairs][16 flag slots]
            self.y_gran = torch.zeros(
                len(self.blocks), K_attn // 2 + 16, device=dev,
                dtype=torch.int32,
            )

        self._r_qkv = self._rows(cfg.qkv_dim, E, "MDI_ROWS_QKV")
        self._r_proj = self._rows(E, cfg.n_head * cfg.head_size,
                                  "MDI_ROWS_PROJ")
        self._r_down = self._rows(E, I, "MDI_ROWS_DOWN")
        self._r_head = self._rows(cfg.padded_vocab_size, E, "MDI_ROWS_HEAD")

        if self.is_starter:
            # per-slot current-token table for fully-fused step graphs
            self.token_table = torch.zeros(kv_pool.n_slots, device=dev,
                                           dtype=torch.int32)

        self._graph_blocks: Optional[torch.cuda.CUDAGraph] = None
        self._graph_env: Optional[torch.cuda.CUDAGraph] = None
        self._graph_tail: Optional[torch.cuda.CUDAGraph] = None
        self._graph_standalone: Optional[torch.cuda.CUDAGraph] = None
        self._graph_starter: Optional[torch.cuda.CUDAGraph] = None
        self._graph_tail_sample: Optional[torch.cuda.CUDAGraph] = None
        self._fused_params = None

    # ---------------------------------------------------------------------
    # slot/pos bookkeeping
    # ---------------------------------------------------------------------
    def set_slot_pos(self, slot: int, pos: int) -> None:
        """Host-side bookkeeping (prefill / sample init)."""
        self.pos_table[slot] = pos

    def clear_scratch(self) -> None:
        """Zero granule hand-off buffers (stale (slot, pos) tags from a
        previous run would otherwise satisfy a consumer sweep early)."""
        if getattr(self, "y_gran", None) is not None:
            self.y_gran.zero_()
        for bufs in getattr(self, "_lane_bufs", None) or []:
            g = bufs.get("y_gran")
            if g is not None:
                g.zero_()

    def _stage_pos(self) -> None:
        # pos <- pos_table[slot]   (inside the graph: slot is a device
        # value; one tiny HIP launch instead of a copy + index_select)
        self.ops.stage_slot(self.slot, pos_out=self.pos,
                            pos_table=self.pos_table)

    def _stage_pos_token(self) -> None:
        # pos <- pos_table[slot]; token <- token_table[slot] in ONE launch
        self.ops.stage_slot(self.slot, pos_out=self.pos,
                            token_out=self.token,
                            pos_table=self.pos_table,
                            token_table=self.token_table)

    # ---------------------------------------------------------------------
    # kernel sequence (eager; also what gets captured)
    # ---------------------------------------------------------------------
    @property
    def _nk(self) -> int:
        """fused-norm kind: 1 RMSNorm, 2 LayerNorm."""
        return 1 if self.config.norm_class_name == "RMSNorm" else 2

    @staticmethod
    def _rows(M: int, K: int, env: str = "") -> int:
        """Output rows per wave for the decode GEMV, from an in-graph A/B
        sweep on MI355X (Llama-3-8B shapes): long-K shapes want 4-row
        ILP; for everything else MORE blocks wins — many blocks per CU
        pipeline the per-kernel memory ramp, so rows=1 beat rows=2/4 on
        the qkv (6144x4096) and proj/down shapes by 3-15%. Env override
        for tuning."""
        if env and os.environ.get(env):
            return int(os.environ[env])
        if M >= 65536:
            return 4  # lm_head: grid caps at 4096 blocks; row ILP wins
        if K >= 16384:
            return 1  # direct-x long-K (70B down): max blocks wins
        if M <= 16384:
            return 1
        return 2

    def sample_into_token(self, temperature: float, top_k, seed: int,
                          top_p: float = 1.0) -> torch.Tensor:
        """Fused on-GPU sampling from self.logits into self.sample_out.
        (scratch is self-cleaning; the gumbel stream is keyed by
        (seed, slot, pos) — reproducible and schedule-independent.)"""
        self.ops.sample(
            self.sample_out, self.logits, self.sample_scratch,
            float(temperature), int(top_k or 0), temperature > 0.0,
            int(seed) & 0x7FFFFFFF, self.pos, self.slot, 0, float(top_p),
        )
        return self.sample_out

    def _run_blocks(self) -> None:
        """x -> x through all local blocks (decode, one token).

        All pre-norms are fused into the GEMV staging pass and residual
        adds into GEMV epilogues — a llama block is 6 kernels total (qkv,
        rope+kv, attn x2, proj+res, swiglu, down+res)."""
        cfg = self.config
        ops = self.ops
        eps = cfg.norm_eps
        nk = self._nk
        scale = 1.0 / (cfg.head_size ** 0.5)
        for li, w in enumerate(self.blocks):
            # qkv = Wqkv @ norm1(x); rope + kv-append are fused inside the
            # attention kernel (qkv stays raw)
            if self.fp8:
                ops.gemv_fp8(self.qkv, w.attn_w8, w.attn_s, self.x,
                             w.attn_b, None, 0, w.norm1_w, w.norm1_b, nk,
                             eps, self._r_qkv)
            else:
                ops.gemv(self.qkv, w.attn_w, self.x, w.attn_b, None, 0,
                         w.norm1_w, w.norm1_b, nk, eps, self._r_qkv)
            if self._fuse_attn_proj:
                # attention + proj + residual add in ONE launch; the proj
                # rows stream into LDS while the attention blocks run
                ops.attn_proj(self.a, self.qkv, self.kv_pool.k,
                              self.kv_pool.v, self.cos, self.sin, self.pos,
                              self.slot, li, scale, w.proj_w, w.proj_b,
                              self.x, self.y_gran[li])
                self._mlp(self.a, w, self.a, w.norm2_w, w.norm2_b)
                continue
            ops.attn_decode(
                self.y, self.part_o, self.part_ml, self.qkv, self.kv_pool.k,
                self.kv_pool.v, self.cos, self.sin, self.pos, self.slot, li,
                self.n_chunks, scale,
                kscale=self.kv_pool.kscale, vscale=self.kv_pool.vscale,
                force_split=self.force_split,
            )
            if cfg.parallel_residual:
                # x = x + proj(y) + mlp(norm2(x) or norm1(x))
                if self.fp8:
                    ops.gemv_fp8(self.a, w.proj_w8, w.proj_s, self.y,
                                 w.proj_b, None, 0, None, None, 0, eps,
                                 self._r_proj)
                else:
                    ops.gemv(self.a, w.proj_w, self.y, w.proj_b, None, 0,
                             None, None, 0, eps, self._r_proj)
                nw = w.norm1_w if cfg.shared_attention_norm else w.norm2_w
                nb = w.norm1_b if cfg.shared_attention_norm else w.norm2_b
                self._mlp(self.x, w, self.a, nw, nb)
                ops.add(self.x, self.x, self.m_out)
            else:
                # a = x + proj(y); x = a + mlp(norm2(a))
                if self.fp8:
                    ops.gemv_fp8(self.a, w.proj_w8, w.proj_s, self.y,
                                 w.proj_b, self.x, 1, None, None, 0, eps,
                                 self._r_proj)
                else:
                    ops.gemv(self.a, w.proj_w, self.y, w.proj_b, self.x, 1,
                             None, None, 0, eps, self._r_proj)
                self._mlp(self.a, w, self.a, w.norm2_w, w.norm2_b)
                # _mlp wrote x = res + down(act) directly
        # (sequential path leaves the stream in self.x)

    def _mlp(self, inp, w, res, norm_w, norm_b) -> None:
        """act = act_fn(fc(norm(inp))); writes x/m_out = res + proj(act).

        Sequential path: out buffer is self.x (the new residual stream).
        Parallel path: out buffer is self.m_out (summed by caller)."""
        cfg = self.config
        eps = cfg.norm_eps
        nk = self._nk
        if cfg.mlp_class_name == "LLaMAMoE":
            # router: gate logits -> (top-k experts, softmax weights),
            # then k expert swiglu+down passes selected by DEVICE-side
            # indices (the whole sequence is graph-capturable; reference
            # model.py:823-853 semantics).  The norm runs ONCE as its own
            # kernel — the bf16-rounded x_norm must feed the router
            # exactly as in the torch reference, or near-tied experts
            # get routed differently.
            ops = self.ops
            ops.rmsnorm(self.xn, inp, norm_w, eps)
            ops.gemv(self.gate_logits, w.gate_w, self.xn, None, None, 0,
                     None, None, 0, eps, 1)
            ops.moe_gate_topk(self.moe_eidx, self.moe_escale,
                              self.gate_logits, cfg.n_expert_per_token)
            E, I = cfg.n_embd, cfg.intermediate_size
            out = self.m_out if cfg.parallel_residual else self.x
            res_j = res
            for j in range(cfg.n_expert_per_token):
                ops.gemv_swiglu(self.act, w.fc1_w, w.fc2_w, self.xn, False,
                                None, None, 0, eps,
                                eidx=self.moe_eidx[j:j + 1],
                                estride=I * E,
                                escale=self.moe_escale[j:j + 1])
                ops.gemv(out, w.mlp_proj_w, self.act, None, res_j, 1,
                         None, None, 0, eps, self._r_down,
                         eidx=self.moe_eidx[j:j + 1], estride=E * I)
                res_j = out
            return
        if cfg.mlp_class_name in ("LLaMAMLP", "GemmaMLP"):
            gelu_gate = cfg.mlp_class_name == "GemmaMLP"
            if self.fp8:
                self.ops.gemv_swiglu_fp8(self.act, w.fc1_w8, w.fc1_s,
                                         w.fc2_w8, w.fc2_s, inp, gelu_gate,
                                         norm_w, norm_b, nk, eps)
            else:
                self.ops.gemv_swiglu(self.act, w.fc1_w, w.fc2_w, inp,
                                     gelu_gate, norm_w, norm_b, nk, eps)
        elif self.fp8:
            self.ops.gemv_fp8(self.act, w.fc_w8, w.fc_s, inp, w.fc_b, None,
                              2, norm_w, norm_b, nk, eps, 0)
        else:
            self.ops.gemv(self.act, w.fc_w, inp, w.fc_b, None, 2,
                          norm_w, norm_b, nk, eps)  # gelu
        out = self.m_out if cfg.parallel_residual else self.x
        if self.fp8:
            self.ops.gemv_fp8(out, w.mlp_proj_w8, w.mlp_proj_s, self.act,
                              w.mlp_proj_b, res, 1, None, None, 0, eps,
                              self._r_down)
        else:
            self.ops.gemv(out, w.mlp_proj_w, self.act, w.mlp_proj_b, res, 1,
                          None, None, 0, eps, self._r_down)

    def _embed(self) -> None:
        cfg = self.config
        emb_scale = (cfg.n_embd ** 0.5) if cfg.scale_embeddings else 1.0
        self.ops.embed(self.x, self.wte, self.token, emb_scale)
        if self.wpe is not None:
            self.ops.embed(self.pos_emb, self.wpe, self.pos, 1.0)
            self.ops.add(self.x, self.x, self.pos_emb)

    def _tail_seq(self) -> None:
        # logits = lm_head @ ln_f(x): one fused kernel
        if self.fp8:
            self.ops.gemv_fp8(self.logits, self.head_w8, self.head_s,
                              self.x, self.head_b, None, 0, self.lnf_w,
                              self.lnf_b, self._nk, self.config.norm_eps,
                              self._r_head)
        else:
            self.ops.gemv(self.logits, self.head_w, self.x, self.head_b,
                          None, 0, self.lnf_w, self.lnf_b, self._nk,
                          self.config.norm_eps, self._r_head)

    # ---------------------------------------------------------------------
    # public decode API
    # ---------------------------------------------------------------------
    def capture_graphs(self) -> None:
        """Capture the per-token block stack (and tail) as hipGraphs."""
        if not self.use_graphs or self._graph_blocks is not None:
            return
        torch.cuda.synchronize()
        # warm-up in a side stream (allocator requirement for capture)
        s = torch.cuda.Stream()
        s.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(s):
            for _ in range(2):
                self._stage_pos()
                if self.is_starter:
                    self._embed()
                self._run_blocks()
                if self.is_starter:
                    self._tail_seq()
        torch.cuda.current_stream().wait_stream(s)
        torch.cuda.synchronize()
        # zero any cache rows the warm-up touched
        self.kv_pool.k.zero_()
        self.kv_pool.v.zero_()
        self.clear_scratch()

        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            self._stage_pos()
            if self.is_starter:
                self._embed()
            self._run_blocks()
        self._graph_blocks = g
        if self.is_starter:
            gt = torch.cuda.CUDAGraph()
            with torch.cuda.graph(gt):
                self._tail_seq()
            self._graph_tail = gt
        torch.cuda.synchronize()

    # ------------------------------------------------------------------
    # HIP prefill: torch GEMMs + hand-written rope-append and causal flash
    # attention (no S^2 score materialization)
    # ------------------------------------------------------------------
    @property
    def supports_hip_prefill(self) -> bool:
        cfg = self.config
        return (cfg.norm_class_name == "RMSNorm"
                and cfg.mlp_class_name in ("LLaMAMLP", "GemmaMLP")
                and not cfg.parallel_residual)

    @torch.inference_mode()
    def prefill_hidden(self, x: torch.Tensor, slot: int,
                       pos0: int = 0) -> torch.Tensor:
        """Run the local blocks over a [T, n_embd] prompt chunk, filling the
        KV pool at positions pos0..pos0+T-1."""
        import torch.nn.functional as F

        cfg = self.config
        ops = self.ops
        T = x.size(0)
        scale = 1.0 / (cfg.head_size ** 0.5)
        Y = torch.empty(T, cfg.n_head * cfg.head_size, device=self.device,
                        dtype=torch.bfloat16)
        xn = torch.empty_like(x)
        for li, w in enumerate(self.blocks):
            ops.rmsnorm(xn, x, w.norm1_w, cfg.norm_eps)
            qkv = F.linear(xn, w.attn_w, w.attn_b)
            ops.rope_prefill_append(qkv, self.kv_pool.k, self.kv_pool.v,
                                    self.cos, self.sin, pos0, slot, li,
                                    kscale=self.kv_pool.kscale,
                                    vscale=self.kv_pool.vscale)
            ops.prefill_attn(Y, qkv, self.kv_pool.k, self.kv_pool.v, pos0,
                             slot, li, scale,
                             kscale=self.kv_pool.kscale,
                             vscale=self.kv_pool.vscale)
            # residual rides the GEMM epilogue (addmm beta=1) when there is
            # no bias; act(gate)*up is one fused launch instead of two
            if w.proj_b is None:
                a = torch.addmm(x, Y, w.proj_w.t())
            else:
                a = x + F.linear(Y, w.proj_w, w.proj_b)
            hn = xn
            ops.rmsnorm(hn, a, w.norm2_w, cfg.norm_eps)
            gelu_gate = cfg.mlp_class_name == "GemmaMLP"
            gate = F.linear(hn, w.fc1_w)
            up = F.linear(hn, w.fc2_w)
            ops.swiglu_mul(up, gate, up, gelu_gate)
            if w.mlp_proj_b is None:
                x = torch.addmm(a, up, w.mlp_proj_w.t())
            else:
                x = a + F.linear(up, w.mlp_proj_w, w.mlp_proj_b)
        return x

    @torch.inference_mode()
    def prefill_prompt(self, tokens: torch.Tensor, slot: int,
                       pos0: int = 0) -> torch.Tensor:
        """Starter: embed prompt tokens then run the local blocks."""
        import torch.nn.functional as F

        x = F.embedding(tokens.long().view(-1), self.wte)
        if self.config.scale_embeddings:
            x = x * (self.config.n_embd ** 0.5)
        return self.prefill_hidden(x, slot, pos0)

    # ------------------------------------------------------------------
    # fully-fused per-token step graphs (bench hot path)
    # ------------------------------------------------------------------
    def _sample_seq(self, temperature: float, top_k: int, seed: int,
                    top_p: float = 1.0, out=None, advance: str = "",
                    pos_bias: int = 0) -> None:
        """Fused sampling; `advance` folds the step bookkeeping into the
        sampler's unpack launch: "token" writes token_table[slot],
        "token+pos" additionally advances pos_table[slot].

        pos_bias keys the draw by the DRAWN token's sequence index: the
        standalone step graph (embed->blocks->tail->sample) reads pos
        before its advance, so it passes 1; the pipeline tail-first
        graphs read the already-advanced pos and pass 0.  With matching
        keys the standalone and pipeline token streams are identical."""
        self.ops.sample(self.sample_out if out is None else out,
                        self.logits, self.sample_scratch,
                        float(temperature), int(top_k or 0),
                        temperature > 0.0, int(seed) & 0x7FFFFFFF,
                        self.pos, self.slot, 0, float(top_p),
                        token_table=self.token_table if advance else None,
                        pos_table=self.pos_table
                        if advance == "token+pos" else None,
                        adv_slot=self.slot if advance else None,
                        adv_pos=1 if advance == "token+pos" else 0,
                        pos_bias=pos_bias)

    def _advance_pos(self) -> None:
        # pos_table[slot] += 1 (in-graph, one tiny launch)
        self.ops.stage_slot(self.slot, pos_table_mut=self.pos_table,
                            adv_pos=1)

    # activation/workspace tensors that are private to one in-flight
    # sample step; everything else (weights, KV pool, pos/token tables,
    # rope caches) is shared across lanes
    _LANE_ATTRS = ("x", "qkv", "y", "a", "act", "m_out", "part_o",
                   "part_ml", "logits", "token", "pos_emb",
                   "sample_scratch", "sample_out", "slot", "pos", "xn",
                   "gate_logits", "moe_eidx", "moe_escale", "y_gran")

    def _set_lane(self, lane: int) -> None:
        for a, t_ in self._lane_bufs[lane].items():
            setattr(self, a, t_)

    @property
    def n_lanes(self) -> int:
        return len(getattr(self, "_lane_graphs", None) or [1])

    def ensure_fused_graphs(self, temperature: float, top_k, seed: int,
                            n_lanes: int = 1) -> None:
        """Capture the three starter step graphs for fixed sampling params:
        standalone (embed->blocks->tail->sample), pipeline-starter
        (tail->sample->embed->blocks), and tail+sample only (drain rounds).

        n_lanes > 1 captures the standalone step N times over N private
        workspace sets, each replayed on its own HIP stream: different
        in-flight samples (different KV slots) then overlap on the GPU,
        hiding the per-kernel launch floor that dominates small models.
        Token streams are unchanged — sampling is (seed, slot, pos)-keyed
        and samples share no per-step state."""
        params = (float(temperature), int(top_k or 0), int(seed),
                  int(n_lanes))
        if not self.use_graphs or not self.is_starter:
            return
        if self._fused_params == params and self._graph_standalone is not None:
            return
        t, k, sd, n_lanes = params
        torch.cuda.synchronize()
        s = torch.cuda.Stream()
        s.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(s):
            for _ in range(2):
                self._stage_pos_token()
                self._embed()
                self._run_blocks()
                self._tail_seq()
                self._sample_seq(t, k, sd, advance="token+pos", pos_bias=1)
        torch.cuda.current_stream().wait_stream(s)
        torch.cuda.synchronize()
        self.kv_pool.k.zero_()
        self.kv_pool.v.zero_()
        self.pos_table.zero_()
        self.token_table.zero_()
        self.clear_scratch()

        base = {a: getattr(self, a) for a in self._LANE_ATTRS
                if getattr(self, a, None) is not None}
        self._lane_bufs = [dict(base)]
        for _l in range(1, n_lanes):
            self._lane_bufs.append(
                {a: torch.zeros_like(t_) for a, t_ in base.items()})
        self._lane_graphs = []
        for l in range(n_lanes):
            self._set_lane(l)
            g = torch.cuda.CUDAGraph()
            with torch.cuda.graph(g):
                self._stage_pos_token()
                self._embed()
                self._run_blocks()
                self._tail_seq()
                self._sample_seq(t, k, sd, advance="token+pos", pos_bias=1)
            self._lane_graphs.append(g)
        self._set_lane(0)
        self._lane_streams = [torch.cuda.Stream()
                              for _ in range(n_lanes)]
        self._graph_standalone = self._lane_graphs[0]

        g2 = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g2):
            self._stage_pos()
            self._tail_seq()
            # the sampler writes the drawn token into BOTH token_table
            # and the embed input scalar, and the blocks run with the
            # pre-advance pos; pos advances at the end of the graph
            self._sample_seq(t, k, sd, out=self.token, advance="token")
            self._embed()
            self._run_blocks()
            self._advance_pos()
        self._graph_starter = g2

        g3 = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g3):
            self._stage_pos()
            self._tail_seq()
            self._sample_seq(t, k, sd, advance="token")
        self._graph_tail_sample = g3
        self._fused_params = params
        torch.cuda.synchronize()

    def standalone_step(self, slot: int) -> None:
        """One full decode token for `slot` (token_table-chained)."""
        self.slot.fill_(slot)
        self._graph_standalone.replay()

    # ---- multi-stream lanes (standalone multi-sample overlap) ----------
    def lanes_begin(self) -> None:
        """Order every lane stream after the current stream (prefill and
        host-side staging complete before lane replays start)."""
        cur = torch.cuda.current_stream()
        for st in self._lane_streams:
            st.wait_stream(cur)

    def lanes_join(self) -> None:
        """Order the current stream after every lane stream (no host
        sync; D2H readers on the current stream see the lane writes)."""
        cur = torch.cuda.current_stream()
        for st in self._lane_streams:
            cur.wait_stream(st)

    def standalone_lane_step(self, lane: int, slot: int) -> None:
        """standalone_step on lane `lane`'s private stream/workspace;
        steps on different lanes run concurrently on the GPU."""
        st = self._lane_streams[lane]
        with torch.cuda.stream(st):
            self._lane_bufs[lane]["slot"].fill_(slot)
            self._lane_graphs[lane].replay()

    def starter_step(self, x_in: torch.Tensor, slot: int) -> torch.Tensor:
        """Pipeline starter: tail(x_in)+sample+next head; returns self.x."""
        if x_in.data_ptr() != self.x.data_ptr():
            self.x.copy_(x_in.view(-1), non_blocking=True)
        self.slot.fill_(slot)
        self._graph_starter.replay()
        return self.x

    def tail_sample_step(self, x_in: torch.Tensor, slot: int) -> None:
        if x_in.data_ptr() != self.x.data_ptr():
            self.x.copy_(x_in.view(-1), non_blocking=True)
        self.slot.fill_(slot)
        self._graph_tail_sample.replay()

    def decode_step_head(self, token: torch.Tensor, slot: int) -> torch.Tensor:
        """Starter head role: token -> activations (writes self.x).

        ``token``: scalar int tensor on device (or host int).  Returns the
        activation vector to forward down the ring (bf16, n_embd).
        """
        self.token.fill_(int(token)) if not torch.is_tensor(token) else \
            self.token.copy_(token.view(1).to(torch.int32), non_blocking=True)
        self.slot.fill_(slot)
        if self._graph_blocks is not None:
            self._graph_blocks.replay()
        else:
            self._stage_pos()
            if self.is_starter:
                self._embed()
            self._run_blocks()
        self.pos_table[slot] += 1
        return self.x

    # ------------------------------------------------------------------
    # envelope serve (pipelined secondary): slot comes from the message
    # header ON DEVICE, so the host never reads a header in the decode
    # loop (a per-hop hdr.cpu() would sync the device)
    # ------------------------------------------------------------------
    def ensure_env_graph(self) -> None:
        """Capture header-routed decode: route(hdr)->stage->blocks->advance.
        Requires a spare KV slot (the last one) for stop/flush envelopes.
        Must run BEFORE prefill (capture warm-up scribbles the caches)."""
        if self._graph_env is not None or not self.use_graphs:
            if not hasattr(self, "env_hdr"):
                self.env_hdr = torch.zeros(4, device=self.device,
                                           dtype=torch.int32)
            return
        assert self.kv_pool.n_slots >= 2, "env serve needs a spare KV slot"
        self.env_hdr = torch.zeros(4, device=self.device, dtype=torch.int32)
        dummy = self.kv_pool.n_slots - 1

        def seq():
            self.ops.route_env(self.env_hdr, self.slot, self.pos_table,
                               dummy)
            self._stage_pos()
            self._run_blocks()
            self._advance_pos()

        torch.cuda.synchronize()
        s = torch.cuda.Stream()
        s.wait_stream(torch.cuda.current_stream())
        with torch.cuda.stream(s):
            for _ in range(2):
                seq()
        torch.cuda.current_stream().wait_stream(s)
        torch.cuda.synchronize()
        self.kv_pool.k.zero_()
        self.kv_pool.v.zero_()
        self.pos_table.zero_()
        self.clear_scratch()
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g):
            seq()
        self._graph_env = g
        torch.cuda.synchronize()

    def env_step(self, hdr: torch.Tensor, payload: torch.Tensor) -> torch.Tensor:
        """One header-routed decode step; returns self.x (the activations
        to forward).  hdr/payload are device tensors (recv-ring views);
        everything is enqueued on the current stream — zero host syncs."""
        self.env_hdr.copy_(hdr, non_blocking=True)
        self.x.copy_(payload.view(-1), non_blocking=True)
        if self._graph_env is not None:
            self._graph_env.replay()
        else:
            dummy = self.kv_pool.n_slots - 1
            self.ops.route_env(self.env_hdr, self.slot, self.pos_table,
                               dummy)
            self._stage_pos()
            self._run_blocks()
            self._advance_pos()
        return self.x

    def decode_step_mid(self, x: torch.Tensor, slot: int) -> torch.Tensor:
        """Secondary role: activations in -> activations out."""
        if x.data_ptr() != self.x.data_ptr():
            self.x.copy_(x.view(-1), non_blocking=True)
        self.slot.fill_(slot)
        if self._graph_blocks is not None:
            self._graph_blocks.replay()
        else:
            self._stage_pos()
            self._run_blocks()
        self.pos_table[slot] += 1
        return self.x

    def tail(self, x: Optional[torch.Tensor] = None) -> torch.Tensor:
        """Starter tail role: activations -> logits (bf16, padded vocab)."""
        if x is not None and x.data_ptr() != self.x.data_ptr():
            self.x.copy_(x.view(-1), non_blocking=True)
        if self._graph_tail is not None:
            self._graph_tail.replay()
        else:
            self._tail_seq()
        return self.logits
