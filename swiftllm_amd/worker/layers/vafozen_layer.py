"""A Vafozen layer: mixer(h) + ff(h) of one normed input as one product on the way in, the mixers, and one product on the way out.
Everything in between writes its part of one row per token (`VafozenLayerWeight.ins`); adding the result to the fp32 stream and the
next input's norm are the model's fused step (kernels/hyper_stream.py)."""
import torch

from ..kernels.linear_scan import DECAY_EXP_EXP, DECAY_SIGMOID_POWER, linear_recurrence, low_rank_decay
from ..kernels.linear import linear_grouped
from ..kernels.moe import gated_rows
from ..kernels.rms_stream import token_shift_mix
from ..kernels.rope_kv import qkv_conv_rope_and_store_kv
from ..kernels.ssd import state_space_mixer
from ..kernels.window_attn import MASK_CHUNK, MASK_WINDOW, AttentionSpec, masked_attention
from .kekapel_layer import _project, _project_partials
from .lorulix_layer import StepContext


class _Left:
    """The softmax attention of a side-by-side layer: biases, convolutions or q/k norm, rotation and KV store in one launch (the
    layer's left factor rides on the cached values), then attention over the pool into the layer's row, gated where the design
    says so. row_sizes: key and value row sizes in the pool (kernels/window_attn.py: served_row_sizes)."""

    def __init__(self, layer_config, weight, eps: float, pool_slice, max_positions: int, row_sizes, tail_off: int):
        mx = self.mixer = layer_config.mixer.left
        self.v_mult = layer_config.mixer.left_scale
        self.w, self.eps, self.pool_slice, self.max_positions, self.tail_off = weight, eps, pool_slice, max_positions, tail_off
        self.spec = AttentionSpec(mx.num_q_heads, mx.num_kv_heads, row_sizes[0], row_sizes[1], mx.scale, window=mx.chunk,
                                  mask_kind=MASK_CHUNK if mx.chunk else MASK_WINDOW, softcap=mx.softcap, slopes=weight.slopes,
                                  out_dim=mx.value_dim)

    def forward(self, proj: torch.Tensor, row: torch.Tensor, ctx: StepContext):
        mx, w, sp = self.mixer, self.w, self.spec
        q = qkv_conv_rope_and_store_kv(proj[:, w.cols["qkv"]], w.qkv_b, w.conv, w.q_norm, w.k_norm, w.freq, mx.rot, ctx.pool,
                                       self.pool_slice, ctx.block_table, ctx.state, self.tail_off, mx.num_q_heads, mx.num_kv_heads,
                                       mx.head_dim, mx.value_dim, sp.head_dim, sp.value_dim, self.eps, self.v_mult)
        out = row[:, w.ins["left"]]
        if ctx.pool is None:    # memory profiling: no cached keys to read
            out.zero_()
            return
        masked_attention(q, ctx.pool, self.pool_slice, ctx.block_table, ctx.tok_seq, ctx.tok_pos, sp, ctx.tiles, self.max_positions,
                         out=out, gate=proj[:, w.cols["gate"]] if mx.convolved else None)


class _LinearAttention:
    """Gated linear attention: decays from the low-rank rows of the fused projection, the recurrence on the sequence's state, head
    norm and gate."""

    def __init__(self, layer_config, weight, eps: float, state_off: int):
        self.mixer, self.mult = layer_config.mixer.right, layer_config.mixer.right_scale
        self.w, self.eps, self.state_off = weight, eps, state_off

    def forward(self, h: torch.Tensor, proj: torch.Tensor, row: torch.Tensor, ctx: StepContext, skinny: bool):
        mx, w = self.mixer, self.w
        decay = low_rank_decay(proj[:, w.cols["decay"]], None, w.decay_2, w.decay_b, DECAY_SIGMOID_POWER, 1.0 / mx.tau)
        q, k, v, g = (proj[:, w.cols["right_" + n]] for n in "qkvg")
        linear_recurrence(q, k, v, decay, ctx.state, self.state_off, mx.num_heads, mx.key_dim,
                          mx.value_dim, q_scale=mx.key_dim ** -0.5,
                          finish=(row[:, w.ins["right"]], w.right_norm, g, self.eps, self.mult))


class _TimeMixing:
    """Time mixing: five token-shifted mixes of the input, their projections and decays, the recurrence with the bonus, head norm and
    gate."""

    def __init__(self, layer_config, weight, eps: float, tail_off: int, state_off: int):
        self.mixer, self.mult = layer_config.mixer.right, layer_config.mixer.right_scale
        self.w, self.eps, self.tail_off, self.state_off = weight, eps, tail_off, state_off

    def forward(self, h: torch.Tensor, proj: torch.Tensor, row: torch.Tensor, ctx: StepContext, skinny: bool):
        mx, w = self.mixer, self.w
        mixes = token_shift_mix(h, w.mu, ctx.state, self.tail_off)
        rkvg = linear_grouped(mixes[:4], w.shifted, skinny)
        r, k, v, g = (rkvg[:, i * mx.inner:(i + 1) * mx.inner] for i in range(4))
        decay = low_rank_decay(mixes[4], w.decay_1, w.decay_2, w.decay_b, DECAY_EXP_EXP, tanh=True)
        linear_recurrence(r, k, v, decay, ctx.state, self.state_off, mx.num_heads, mx.key_dim,
                          mx.value_dim, bonus=w.bonus, finish=(row[:, w.ins["right"]], w.right_norm, g, self.eps, self.mult))


class _StateSpace:
    def __init__(self, layer_config, weight, eps: float, tail_off: int, state_off: int):
        self.mixer, self.w, self.eps, self.tail_off, self.state_off = layer_config.mixer, weight, eps, tail_off, state_off

    def forward(self, h: torch.Tensor, proj: torch.Tensor, row: torch.Tensor, ctx: StepContext, skinny: bool):
        w = self.w
        state_space_mixer(proj[:, w.cols["in"]], w.conv, w.conv_b, w.a_log, w.dt_bias, w.d_skip, w.right_norm, ctx.state,
                          self.tail_off, self.state_off, self.mixer, self.eps, out=row[:, w.ins["mixer"]])


class VafozenLayer:
    def __init__(self, layer_config, weight, eps: float, skinny: bool, state, pool_slice, row_sizes, max_positions: int):
        """state: the StateSlotManager that hands out the regions this layer carries from token to token."""
        mx = layer_config.mixer
        self.w, self.skinny, self.mlp = weight, skinny, layer_config.mlp
        self.left = None
        if layer_config.type == "mamba2":
            tail = state.add_region(2 * (mx.conv_taps - 1) * mx.conv_channels)
            self.right = _StateSpace(layer_config, weight, eps, tail, state.add_region(mx.state_elems))
            return
        lf, rt = mx.left, mx.right
        tail = state.add_region(2 * max(lf.conv_taps - 1, 0) * lf.channels)
        self.left = _Left(layer_config, weight, eps, pool_slice, max_positions, row_sizes, tail)
        if layer_config.type == "parallel":
            self.right = _LinearAttention(layer_config, weight, eps, state.add_region(rt.state_elems))
        else:
            shift = state.add_region(2 * weight.mu.shape[1])
            self.right = _TimeMixing(layer_config, weight, eps, shift, state.add_region(rt.state_elems))

    def forward(self, h: torch.Tensor, ctx: StepContext):
        """-> the layer's result, rows or SplitKPartials."""
        w = self.w
        proj = _project(h, w.proj, self.skinny)
        make = torch.zeros if w.row_gaps else torch.empty       # (columns of no piece meet zero weights: they must be finite)
        row = make((h.shape[0], w.row_size), dtype=h.dtype, device=h.device)
        if self.left is not None:
            self.left.forward(proj, row, ctx)
        self.right.forward(h, proj, row, ctx, self.skinny)
        if self.mlp is not None:
            gated_rows(row[:, w.ins["ff"]], proj[:, w.cols["ff_gate"]], proj[:, w.cols["ff_up"]])
        return _project_partials(row, w.out, self.skinny)
