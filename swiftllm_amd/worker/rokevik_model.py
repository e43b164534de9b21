"""RokevikModel — the data-plane worker for the Rokevik design.

The worker protocol, the token-level `step`, the block pool, the block managers, hipGraph replay of decode steps and
swapping are SteppedModel's (stepped_model.py); this file adds what is Rokevik's:

  * the layout of a block, a slice per layer RUN (a looped layer has its own in every pass): an attention layer's keys and values;
    for a latent attention layer ONE row per token — the normed latent and the rotated shared key part as the key, the latent
    again (transposed) as the value. Rows may be wider than the heads (served_row_sizes), so that the matrix-core attention
    serves every size;
  * the layout of a state slot (StateSlotManager): the fp32 state of every minGRU run;
  * the stack on several fp32 streams: per sublayer
        y (, y2) = sublayer(h)
        X_t <- sum_s mix[s, t] X_s + out[t] (y + y2);  h = groupnorm(sum_s in[s] X_s)      one fused launch
    (kernels/hyper_stream.py; a model without streams is the case S = 1 of ones), then the summed streams, their norm, the
    vocabulary projection and the cap of the logits. Projections run in the compute dtype (bfloat16 / float16, or true float32).
"""
from typing import List

import torch

from swiftllm_amd.engine_config import EngineConfig
from swiftllm_amd.model_config import RokevikModelConfig

from .kernels.hyper_stream import embed_streams, hyper_step
from .kernels.linear import pack_weight, packable
from .kernels.rms_stream import StateRef
from .kernels.sampling import softcap_logits
from .kernels.window_attn import PoolSlice, served_row_sizes
from .layers.kekapel_layer import _project
from .layers.lorulix_layer import StepContext
from .layers.rokevik_layer import RokevikAttention, RokevikFeedForward, RokevikLatentAttention, RokevikMinGru
from .rokevik_weight import load_rokevik_weights
from .state_slots import StateSlotManager
from .stepped_model import SteppedModel


class _Sublayer:
    """One update of the streams: y = op(norm(sum_s in[s] X_s)), then the streams' step with `streams`."""
    __slots__ = ("op", "norm", "streams", "ends_run")

    def __init__(self, op, norm, streams, ends_run):
        self.op, self.norm, self.streams, self.ends_run = op, norm, streams, ends_run


class RokevikModel(SteppedModel):
    CONFIG_CLASS = RokevikModelConfig

    @torch.inference_mode()
    def __init__(self, engine_config: EngineConfig):
        self.sublayers: List[_Sublayer] = []
        self.pool_slices = {}
        self.row_sizes = {}
        super().__init__(engine_config)
        # the design has no position table: a sequence is bounded by what its block-table row can map
        self.max_seq_len = min(self.model_config.max_position_embeddings,
                               engine_config.max_blocks_per_seq * engine_config.block_size)

    def _layout_pool(self):
        """Row sizes, and offsets (in elements) of every caching layer run's keys and values inside a block."""
        cfg, bs = self.model_config, self.engine_config.block_size
        off = 0
        self.pool_slices, self.row_sizes = {}, {}
        for run in cfg.layer_runs:
            mx = cfg.layers[run.layer].mixer
            if mx.kind == "mingru":
                continue
            key, value = (mx.k_size, mx.v_size) if mx.kind == "latent_attention" else (mx.head_dim, mx.value_dim)
            kd, vd = self.row_sizes[run.index] = served_row_sizes(key, value, self.dtype)
            k_off = off
            off += mx.num_kv_heads * kd * bs
            self.pool_slices[run.index] = PoolSlice(k_off, off)
            off += mx.num_kv_heads * vd * bs
            off += -off % 8         # every slice starts on a 16-byte boundary
        self.block_elems = max(off, 8)      # (a model without attention layers still has a block table)

    def _build(self):
        cfg, ecfg = self.model_config, self.engine_config
        self.weight = load_rokevik_weights(cfg, self.dtype, ecfg.model_path, ecfg.use_dummy, self.device)
        skinny = bool(getattr(ecfg, "use_skinny_gemm", False)) and self.dtype != torch.float32
        if skinny and getattr(ecfg, "pack_decode_weights", False):
            for t in self.weight.projection_tensors():
                if packable(t):
                    pack_weight(t)
        self._skinny = skinny
        # one slot per sequence that runs: as many as a batch holds
        self.state = StateSlotManager(ecfg.max_batch_size, self.device) if cfg.has_state else None
        self.sublayers = []
        for run in cfg.layer_runs:
            lcfg, lw = cfg.layers[run.layer], self.weight.layers[run.layer]
            if lcfg.type == "mingru":
                op = RokevikMinGru(lcfg, lw, skinny, self.state.add_region(lcfg.mixer.width))
            else:
                kind = RokevikAttention if lcfg.type == "attention" else RokevikLatentAttention
                op = kind(lcfg, lw, cfg.norm_eps, skinny, self.pool_slices[run.index], self.max_seq_len,
                          self.row_sizes[run.index])
            self.sublayers.append(_Sublayer(op, lw.norm1, lw.streams1, lcfg.mlp is None))
            if lcfg.mlp is not None:
                self.sublayers.append(_Sublayer(RokevikFeedForward(lcfg, lw, skinny), lw.norm2, lw.streams2, True))
        if self.state is not None:
            self.state.allocate()

    @torch.inference_mode()
    def _run_stack(self, dev: dict, use_pool: bool) -> torch.Tensor:
        """Embedding -> every sublayer -> the fp32 streams [T, streams, width]."""
        cfg, w = self.model_config, self.weight
        eps, groups = cfg.norm_eps, cfg.norm_groups
        st = None
        if self.state is not None:
            st = StateRef(self.state.pool, dev["tok_pos"], dev["tok_start"], dev["tok_state"], dev["tok_seq"],
                          dev["seq_row0"], dev["seq_cnt"])
        ctx = StepContext(self.kv_pool if use_pool else None, self.gpu_block_manager.block_table if use_pool else None,
                          dev["tok_seq"], dev["tok_pos"], (dev["tile_row0"], dev["tile_cnt"]), st,
                          (dev["chunk_row0"], dev["chunk_cnt"], dev["seq_chunk0"]))
        x = embed_streams(dev["input_ids"], w.embed, max(cfg.num_streams, 1))
        tap = self.layer_tap
        subs = self.sublayers
        h = hyper_step(x, read=subs[0].streams.read, norm=subs[0].norm, groups=groups, eps=eps, out_dtype=self.dtype)
        for i, s in enumerate(subs):
            y, y2 = s.op.forward(h, ctx)
            nxt = subs[i + 1] if i + 1 < len(subs) else None
            h = hyper_step(x, y, s.streams, y2, s.op.y_bias, nxt.streams.read if nxt else None, nxt.norm if nxt else None,
                           groups, eps)
            if tap is not None and s.ends_run:
                tap.append(x.sum(dim=1))
        return x

    @torch.inference_mode()
    def _logits(self, x: torch.Tensor, rows: torch.Tensor) -> torch.Tensor:
        """The model's norm of the summed streams of the asked-for rows and the vocabulary projection -> [rows, vocab]: in the
        compute dtype, or fp32 when the logits are capped."""
        cfg, w = self.model_config, self.weight
        h = hyper_step(x, norm=w.final_norm, groups=cfg.norm_groups, eps=cfg.norm_eps, out_dtype=self.dtype, row_idx=rows)
        logits = _project(h, w.head, self._skinny)
        return softcap_logits(logits, cfg.logit_softcap) if cfg.logit_softcap else logits
