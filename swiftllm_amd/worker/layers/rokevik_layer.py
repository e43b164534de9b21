"""The sublayers of a Rokevik layer, each a function from its normed input to its raw result (and an optional second addend);
mixing the result into the streams and the next input's norm are the model's fused step (kernels/hyper_stream.py)."""
import torch

from ..kernels.min_gru import min_gru
from ..kernels.moe import ACT_SILU, moe_experts, moe_route_grouped
from ..kernels.rope_kv import head_gate_, latent_rope_and_store_kv, qk_norm_rope_and_store_kv
from ..kernels.window_attn import MASK_WINDOW, AttentionSpec, masked_attention
from .kekapel_layer import _project, _silu_unit
from .lorulix_layer import StepContext


class RokevikAttention:
    """(q | k | gate) projection -> biases, q/k norm, rotary, head temperatures, KV store (the values are the biased keys) ->
    capped softmax attention over every earlier key -> head gate -> output projection (its bias is added by the stream step).
    row_sizes: key and value row sizes in the pool (at least the head's; kernels/window_attn.py: served_row_sizes)."""

    def __init__(self, layer_config, weight, eps: float, skinny: bool, pool_slice, max_positions: int, row_sizes):
        mx = self.mixer = layer_config.mixer
        self.w, self.eps, self.skinny, self.pool_slice, self.max_positions = weight, eps, skinny, pool_slice, max_positions
        self.y_bias = weight.o_b
        # the temperatures ride on the queries; the kernel's scale and cap are the configuration's
        self.spec = AttentionSpec(mx.num_q_heads, mx.num_kv_heads, row_sizes[0], row_sizes[1], mx.scale, window=0,
                                  mask_kind=MASK_WINDOW, softcap=mx.softcap)

    def forward(self, h: torch.Tensor, ctx: StepContext):
        mx, w, sp = self.mixer, self.w, self.spec
        n, H, d = h.shape[0], mx.num_q_heads, mx.head_dim
        proj = _project(h, w.proj, self.skinny)
        q = qk_norm_rope_and_store_kv(proj, w.q_b, w.k_b, w.q_norm, w.k_norm, w.temp, w.freq, mx.rot, ctx.pool, self.pool_slice,
                                      ctx.block_table, ctx.tok_seq, ctx.tok_pos, H, mx.num_kv_heads, 0, d, d, self.eps,
                                      sp.head_dim, sp.value_dim)
        if ctx.pool is None:    # memory profiling: the attention's output buffer without its reads
            y = torch.zeros((n, H * sp.value_dim), dtype=h.dtype, device=h.device)
        else:
            y = masked_attention(q, ctx.pool, self.pool_slice, ctx.block_table, ctx.tok_seq, ctx.tok_pos, sp, ctx.tiles,
                                 self.max_positions)
        if sp.value_dim != d:
            y = y.view(n, H, sp.value_dim)[:, :, :d].reshape(n, H * d)
        head_gate_(y, proj[:, w.gate_col:w.gate_col + H], H, d)
        return _project(y, w.o, self.skinny), None


class RokevikLatentAttention:
    """(q | compressed kv | gate) projection -> rotary, latent norm and cache store -> queries folded through the key
    up-projection -> attention of all heads over the one cached row per token (key: latent | rotated part, value: latent) inside
    the window -> value up-projection per head -> head gate -> output projection."""

    def __init__(self, layer_config, weight, eps: float, skinny: bool, pool_slice, max_positions: int, row_sizes):
        mx = self.mixer = layer_config.mixer
        self.w, self.eps, self.skinny, self.pool_slice, self.max_positions = weight, eps, skinny, pool_slice, max_positions
        self.y_bias = None
        self.spec = AttentionSpec(mx.num_q_heads, 1, row_sizes[0], row_sizes[1], mx.scale, window=mx.window,
                                  mask_kind=MASK_WINDOW)

    def forward(self, h: torch.Tensor, ctx: StepContext):
        mx, w, sp = self.mixer, self.w, self.spec
        n, H, d, dr, r, e = h.shape[0], mx.num_q_heads, mx.head_dim, mx.rot_dim, mx.kv_rank, mx.value_dim
        proj = _project(h, w.proj, self.skinny)
        qa = torch.empty((n, H * sp.head_dim), dtype=h.dtype, device=h.device)
        latent_rope_and_store_kv(proj, qa, w.freq, w.c_norm, ctx.pool, self.pool_slice, ctx.block_table, ctx.tok_seq,
                                 ctx.tok_pos, mx, mx.q_size, self.eps, sp.head_dim, sp.value_dim)
        # q_abs[t, h, :] = W_uk,h^T q_unrotated[t, h, :]  -> the first kv_rank columns of every head of qa
        qn = proj[:, :mx.q_size].view(n, H, d + dr)[:, :, :d].transpose(0, 1)           # [H, T, d]
        torch.bmm(qn, w.uk, out=qa.view(n, H, sp.head_dim)[:, :, :r].transpose(0, 1))   # (a strided batched product: no copy)
        if ctx.pool is None:
            att = torch.zeros((n, H * sp.value_dim), dtype=h.dtype, device=h.device)
        else:
            att = masked_attention(qa, ctx.pool, self.pool_slice, ctx.block_table, ctx.tok_seq, ctx.tok_pos, sp, ctx.tiles,
                                   self.max_positions)
        y = torch.empty((n, H * e), dtype=h.dtype, device=h.device)
        torch.bmm(att.view(n, H, sp.value_dim)[:, :, :r].transpose(0, 1), w.uv_t, out=y.view(n, H, e).transpose(0, 1))
        head_gate_(y, proj[:, w.gate_col:w.gate_col + H], H, e)
        return _project(y, w.o, self.skinny), None


class RokevikMinGru:
    """(gate z | candidate | output gate) projection -> the recurrence on the sequence's state -> output projection."""

    def __init__(self, layer_config, weight, skinny: bool, state_off: int):
        self.mixer, self.w, self.skinny, self.state_off = layer_config.mixer, weight, skinny, state_off
        self.y_bias = None

    def forward(self, h: torch.Tensor, ctx: StepContext):
        w = self.w
        proj = _project(h, w.proj, self.skinny)
        y = min_gru(proj, w.z_b, w.x_b, ctx.state, ctx.chunks, self.state_off, self.mixer.width)
        return _project(y, w.o, self.skinny), None


class RokevikFeedForward:
    """Sigmoid router -> SiLU gated experts on inputs scaled by their scores; the experts' results of decode-sized steps and the
    shared expert's leave separately (the stream step adds them up)."""

    def __init__(self, layer_config, weight, skinny: bool):
        self.mlp, self.w, self.skinny = layer_config.mlp, weight, skinny
        self.y_bias = None

    def forward(self, h: torch.Tensor, ctx: StepContext):
        mlp, w = self.mlp, self.w
        idx, wts = moe_route_grouped(h, w.router, None, mlp.top_k, normalize=False)
        out = moe_experts(h, idx, wts, w.gate_up, w.down, 0.0, ACT_SILU, weigh_inputs=True, combine=False)
        if w.shared_up_gate is None:
            return out, None
        return out, _project(_silu_unit(h, w.shared_up_gate, self.skinny), w.shared_down, self.skinny)
