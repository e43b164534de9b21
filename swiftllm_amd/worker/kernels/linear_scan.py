"""Recurrences that are linear in a matrix state with a decay per key channel (gated linear attention, time mixing with a bonus for
the current token), and the low-rank decays they take. csrc/linear_scan.hip, csrc/low_rank_decay.hip."""
import torch

from swiftllm_amd import _hip

from .delta_rule import gated_head_rmsnorm
from .rms_stream import StateRef

DECAY_SIGMOID_POWER = 0     # sigmoid(y)^power
DECAY_EXP_EXP = 1           # exp(-exp(y))

# limits of csrc/linear_scan.hip
STEP_MAX_VDIM = 256         # a thread of the one-token kernel owns one or four columns
TILE_MAX_DIM = 320          # key channels of a tile in LDS


def low_rank_decay(x: torch.Tensor, w1: torch.Tensor, w2: torch.Tensor, bias: torch.Tensor, kind: int, power: float = 1.0,
                   tanh: bool = False) -> torch.Tensor:
    """-> fp32 [T, channels]: the decay of y = w2 act(w1 x) + bias; w1 None: x holds the rank rows already. x may be a column slice."""
    _hip.require_gpu_tensor(x, "x")
    n, (channels, rank) = x.shape[0], w2.shape
    assert x.stride(1) == 1 and w2.is_contiguous() and w2.dtype == x.dtype and x.shape[1] == (rank if w1 is None else w1.shape[1])
    assert w1 is None or (w1.is_contiguous() and w1.dtype == x.dtype and w1.shape[0] == rank)
    assert bias.dtype == torch.float32 and bias.is_contiguous() and bias.numel() == channels
    out = torch.empty((n, channels), dtype=torch.float32, device=x.device)
    _hip.call("swl_low_rank_decay", _hip.ptr(out), _hip.ptr(x), x.stride(0), _hip.ptr(w1), _hip.ptr(w2), _hip.ptr(bias), n,
              x.shape[1], rank, channels, 1 if tanh else 0, int(kind), float(power), _hip.dtype_code3(x.dtype), _hip.stream())
    return out


def linear_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, st: StateRef, state_off: int,
                      num_heads: int, dim: int, vdim: int, q_scale: float = 1.0, bonus: torch.Tensor = None,
                      k_scale: torch.Tensor = None, dskip: torch.Tensor = None, num_qk_heads: int = 0, finish=None) -> torch.Tensor:
    """Per head, on the fp32 state [heads, dim, vdim] at state_off inside each sequence's slot: S <- diag(decay) S + k v^T, o = S^T q
    (+ dskip v); with `bonus` (fp32 [heads, dim]): o = (S + diag(bonus) k v^T)^T q of the state before the update. q [T, num_qk_heads
    * dim] (times q_scale), k likewise (times k_scale[t, h], when given), v [T, num_heads * vdim] may be column slices; decay fp32
    [T, num_heads * dim] or [T, num_heads]. st.tiles: the step's tiles.
    finish None: -> o fp32 [T, num_heads * vdim]. finish = (out, norm_w, gate, eps, mult): the head norm of `gated_head_rmsnorm` is
    applied too and the result goes to `out`."""
    _hip.require_gpu_tensor(q, "q")
    n, H = q.shape[0], num_heads
    G = num_qk_heads or H
    assert q.dtype == k.dtype == v.dtype and q.stride(1) == k.stride(1) == v.stride(1) == 1
    assert q.shape[1] == k.shape[1] == G * dim and v.shape[1] == H * vdim and H % G == 0
    assert decay.dtype == torch.float32 and decay.stride(1) == 1 and decay.shape in ((n, H * dim), (n, H))
    per_channel = decay.shape[1] == H * dim
    for t, size in ((bonus, H * dim), (k_scale, n * H), (dskip, H)):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.numel() == size)
    row0, cnt, seq_tile0 = st.tiles
    num_seqs, num_tiles = st.seq_row0.shape[0], row0.shape[0]
    code, stream, dev, f32 = _hip.dtype_code3(q.dtype), _hip.stream(), q.device, torch.float32
    if num_seqs == n and vdim <= STEP_MAX_VDIM:          # every portion is one token
        y = torch.empty((n, H * vdim), dtype=f32, device=dev) if finish is None else None
        out, norm_w, gate, eps, mult = finish if finish is not None else (None, None, None, 0.0, 1.0)
        head_stride = 0
        if finish is not None:
            assert out.shape == gate.shape == (n, H * vdim) and out.dtype == gate.dtype == q.dtype
            assert norm_w.dtype == f32 and norm_w.is_contiguous() and norm_w.numel() in (vdim, H * vdim)
            head_stride = vdim if norm_w.numel() != vdim else 0
        _hip.call("swl_linear_step", _hip.ptr(out), out.stride(0) if out is not None else 0, _hip.ptr(y), H * vdim, _hip.ptr(q),
                  q.stride(0), _hip.ptr(k), k.stride(0), _hip.ptr(v), v.stride(0), _hip.ptr(decay), decay.stride(0),
                  1 if per_channel else 0, _hip.ptr(k_scale), _hip.ptr(bonus), float(q_scale), _hip.ptr(dskip), _hip.ptr(st.pool),
                  st.pool.stride(0), int(state_off), _hip.ptr(st.seq_row0), _hip.ptr(st.tok_pos), _hip.ptr(st.tok_state), num_seqs,
                  H, G, dim, vdim, _hip.ptr(norm_w), head_stride, _hip.ptr(gate), gate.stride(0) if gate is not None else 0,
                  float(eps), float(mult), code, stream)
        return y if finish is None else out
    dp = -(-dim // 16) * 16
    qd = torch.empty((num_tiles, H, 16, dp), dtype=f32, device=dev)
    kd = torch.empty((num_tiles, H, dp, 16), dtype=f32, device=dev)
    total = torch.empty((num_tiles, H, dp), dtype=f32, device=dev)
    intra = torch.empty((num_tiles, H, 16, 16), dtype=f32, device=dev)
    _hip.call("swl_linear_chunks", _hip.ptr(qd), _hip.ptr(kd), _hip.ptr(total), _hip.ptr(intra), _hip.ptr(q), q.stride(0),
              _hip.ptr(k), k.stride(0), _hip.ptr(decay), decay.stride(0), 1 if per_channel else 0, _hip.ptr(k_scale),
              _hip.ptr(bonus), float(q_scale), _hip.ptr(row0), _hip.ptr(cnt), num_tiles, H, G, dim, code, stream)
    o = torch.empty((n, H * vdim), dtype=f32, device=dev)
    _hip.call("swl_linear_scan", _hip.ptr(o), o.stride(0), _hip.ptr(qd), _hip.ptr(kd), _hip.ptr(total), _hip.ptr(intra),
              _hip.ptr(v), v.stride(0), _hip.ptr(dskip), _hip.ptr(st.pool), st.pool.stride(0), int(state_off),
              _hip.ptr(st.seq_row0), _hip.ptr(st.seq_cnt), _hip.ptr(seq_tile0), _hip.ptr(st.tok_pos), _hip.ptr(st.tok_state),
              num_seqs, H, dim, vdim, code, stream)
    if finish is None:
        return o
    out, norm_w, gate, eps, mult = finish
    gated_head_rmsnorm(out, o, gate, norm_w, H, vdim, eps, mult)
    return out
