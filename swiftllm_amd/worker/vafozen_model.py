"""VafozenModel — the data-plane worker for the Vafozen design.

The worker protocol, the token-level `step`, the block pool, the block managers, hipGraph replay of decode steps and
swapping are SteppedModel's (stepped_model.py); this file adds what is Vafozen's:

  * the layout of a block: the keys and values of every layer with an attention, in rows that may be wider than the heads
    (served_row_sizes), so that the matrix-core attention serves every size;
  * the layout of a state slot (StateSlotManager): the carried inputs of the convolutions and of the token shift, the fp32 states
    of the recurrences;
  * the stack: per layer y = mixer(h) + ff(h) (worker/layers/vafozen_layer.py), then ONE fused launch
        x += y + bias;  h = x / rms(x) * (1 + w)
    (kernels/hyper_stream.py with a single stream). The stream x is fp32, projections run in the compute dtype (bfloat16 / float16,
    or true float32).
"""
from typing import List

import torch

from swiftllm_amd.engine_config import EngineConfig
from swiftllm_amd.model_config import VafozenModelConfig

from .kernels.hyper_stream import StreamWeights, hyper_step
from .kernels.layernorm import embed_positions
from .kernels.linear import pack_weight, packable
from .kernels.rms_stream import StateRef
from .kernels.window_attn import PoolSlice, served_row_sizes
from .layers.kekapel_layer import _project
from .layers.lorulix_layer import StepContext
from .layers.vafozen_layer import VafozenLayer
from .state_slots import StateSlotManager
from .stepped_model import SteppedModel
from .vafozen_weight import load_vafozen_weights


class VafozenModel(SteppedModel):
    CONFIG_CLASS = VafozenModelConfig

    @torch.inference_mode()
    def __init__(self, engine_config: EngineConfig):
        self.layers: List[VafozenLayer] = []
        self.pool_slices = {}
        self.row_sizes = {}
        super().__init__(engine_config)
        # the design has no position table: a sequence is bounded by what its block-table row can map
        self.max_seq_len = min(self.model_config.max_position_embeddings,
                               engine_config.max_blocks_per_seq * engine_config.block_size)

    def _layout_pool(self):
        """Row sizes, and offsets (in elements) of every attention's keys and values inside a block."""
        cfg, bs = self.model_config, self.engine_config.block_size
        off = 0
        self.pool_slices, self.row_sizes = {}, {}
        for i, layer in enumerate(cfg.layers):
            mx = layer.attention
            if mx is None:
                continue
            kd, vd = self.row_sizes[i] = served_row_sizes(mx.head_dim, mx.value_dim, self.dtype)
            k_off = off
            off += mx.num_kv_heads * kd * bs
            self.pool_slices[i] = PoolSlice(k_off, off)
            off += mx.num_kv_heads * vd * bs
            off += -off % 8         # every slice starts on a 16-byte boundary
        self.block_elems = max(off, 8)      # (a model without attention still has a block table)

    def _build(self):
        cfg, ecfg = self.model_config, self.engine_config
        self.weight = load_vafozen_weights(cfg, self.dtype, ecfg.model_path, ecfg.use_dummy, self.device)
        skinny = bool(getattr(ecfg, "use_skinny_gemm", False)) and self.dtype != torch.float32
        if skinny and getattr(ecfg, "pack_decode_weights", False):
            for t in self.weight.projection_tensors():
                if packable(t):
                    pack_weight(t)
        self._skinny = skinny
        self._plain = StreamWeights.plain(self.device)
        # one slot per sequence that runs: as many as a batch holds
        self.state = StateSlotManager(ecfg.max_batch_size, self.device)
        self.layers = [VafozenLayer(lcfg, lw, cfg.norm_eps, skinny, self.state, self.pool_slices.get(i), self.row_sizes.get(i),
                                    self.max_seq_len) for i, (lcfg, lw) in enumerate(zip(cfg.layers, self.weight.layers))]
        self.state.allocate()

    @torch.inference_mode()
    def _run_stack(self, dev: dict, use_pool: bool) -> torch.Tensor:
        """Embedding -> every layer -> the fp32 stream [T, 1, width]."""
        cfg, w = self.model_config, self.weight
        eps, plain = cfg.norm_eps, self._plain
        st = StateRef(self.state.pool, dev["tok_pos"], dev["tok_start"], dev["tok_state"], dev["tok_seq"], dev["seq_row0"],
                      dev["seq_cnt"], (dev["tile_row0"], dev["tile_cnt"], dev["seq_tile0"]))
        ctx = StepContext(self.kv_pool if use_pool else None, self.gpu_block_manager.block_table if use_pool else None,
                          dev["tok_seq"], dev["tok_pos"], (dev["tile_row0"], dev["tile_cnt"]), st)
        x, _ = embed_positions(dev["input_ids"], dev["tok_pos"], w.embed, None, cfg.embedding_scale, keep_copy=False)
        x = x.unsqueeze(1)
        tap, layers = self.layer_tap, w.layers
        h = hyper_step(x, norm=layers[0].norm1 if layers else w.final_norm, eps=eps, out_dtype=self.dtype)
        for i, layer in enumerate(self.layers):
            y = layer.forward(h, ctx)
            h = hyper_step(x, y, plain, y_bias=layers[i].y_bias, norm=layers[i + 1].norm1 if i + 1 < len(layers) else None, eps=eps)
            if tap is not None:
                tap.append(x[:, 0].clone())
        return x

    @torch.inference_mode()
    def _logits(self, x: torch.Tensor, rows: torch.Tensor) -> torch.Tensor:
        """The model's norm of the asked-for rows and the vocabulary projection -> [rows, vocab] in the compute dtype."""
        h = hyper_step(x, norm=self.weight.final_norm, eps=self.model_config.norm_eps, out_dtype=self.dtype, row_idx=rows)
        return _project(h, self.weight.head, self._skinny)
