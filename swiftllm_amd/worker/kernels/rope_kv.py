"""Rotary positions fused with the paged KV store (plain heads, heads with biases and a q/k norm, the compressed rows of latent
attention), and the per-head steps after the softmax: the combination of two score maps, the head gate. csrc/rope_kv.hip."""
import torch

from swiftllm_amd import _hip

from .window_attn import PoolSlice


def rotary_frequencies(rot, device) -> torch.Tensor:
    """The float64 frequency table of a RotaryConfig on the device (None without rotation)."""
    if rot.dims == 0:
        return None
    return torch.tensor(rot.frequencies(), dtype=torch.float64, device=device)


def _pool_ptrs(pool, pool_slice: PoolSlice):
    if pool is None:
        return 0, 0, 0
    assert pool.is_contiguous()
    esize = pool.element_size()
    return pool.data_ptr() + pool_slice.k_offset * esize, pool.data_ptr() + pool_slice.v_offset * esize, pool.shape[1]


def rope_and_store_kv(qkv: torch.Tensor, freq: torch.Tensor, rot_dims: int, pool: torch.Tensor, pool_slice: PoolSlice,
                      block_table: torch.Tensor, tok_seq: torch.Tensor, tok_pos: torch.Tensor, num_q_heads: int,
                      num_k_heads: int, num_v_heads: int, dim: int, vdim: int):
    """Rows [q | k | v (| anything)] of one fused projection: the query heads rotated in place, the key heads rotated into
    the pool, the value heads copied into the pool. pool None (memory profiling): queries only."""
    _hip.require_gpu_tensor(qkv, "qkv")
    assert qkv.dim() == 2 and qkv.stride(1) == 1
    assert qkv.shape[1] >= (num_q_heads + num_k_heads) * dim + num_v_heads * vdim
    assert tok_pos.dtype == torch.int32 and tok_pos.shape[0] == qkv.shape[0]
    assert freq is None or (freq.dtype == torch.float64 and freq.numel() == rot_dims // 2)
    kp, vp, stride = _pool_ptrs(pool, pool_slice)
    if pool is not None:
        assert pool.dtype == qkv.dtype and block_table.is_contiguous() and tok_seq.dtype == torch.int32
    _hip.call("swl_rope_store_kv", _hip.ptr(qkv), _hip.ptr(freq), kp, vp, _hip.ptr(block_table), _hip.ptr(tok_seq),
              _hip.ptr(tok_pos), qkv.shape[0], num_q_heads, num_k_heads, num_v_heads, dim, vdim,
              rot_dims if freq is not None else 0, qkv.stride(0), block_table.shape[1] if block_table is not None else 0,
              stride, _hip.dtype_code3(qkv.dtype), _hip.stream())


def qk_norm_rope_and_store_kv(rows: torch.Tensor, q_b: torch.Tensor, k_b: torch.Tensor, q_norm: torch.Tensor,
                              k_norm: torch.Tensor, q_mult: torch.Tensor, freq: torch.Tensor, rot, pool: torch.Tensor,
                              pool_slice: PoolSlice, block_table: torch.Tensor, tok_seq: torch.Tensor, tok_pos: torch.Tensor,
                              num_q_heads: int, num_k_heads: int, num_v_heads: int, dim: int, vdim: int, eps: float,
                              k_dim: int = 0, v_dim: int = 0) -> torch.Tensor:
    """rows [q | k | v (| anything)] of one fused projection whose biases (fp32, optional) are still to be added -> the queries
    [T, num_q_heads * k_dim]: biased, RMS-normed per head (fp32 weights of `dim` shared by the heads, None: not normed), rotated as
    `rot` (a RotaryConfig) says and multiplied by q_mult[head] (None: 1). The keys go to the pool likewise; the values to the V
    pool — with num_v_heads = 0 the rows hold none and the biased keys, neither normed nor rotated, are the values. k_dim / v_dim:
    row sizes in the pool and in the result (default dim / vdim), columns beyond the head zero. pool None: queries only."""
    _hip.require_gpu_tensor(rows, "rows")
    n = rows.shape[0]
    k_dim, v_dim = k_dim or dim, v_dim or vdim
    assert rows.dim() == 2 and rows.stride(1) == 1 and tok_pos.dtype == torch.int32 and tok_pos.shape[0] == n
    assert rows.shape[1] >= (num_q_heads + num_k_heads) * dim + num_v_heads * vdim
    for t, size in ((q_b, num_q_heads * dim), (k_b, num_k_heads * dim), (q_norm, dim), (k_norm, dim), (q_mult, num_q_heads)):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.numel() == size)
    rot_dims = rot.dims if freq is not None else 0
    assert freq is None or (freq.dtype == torch.float64 and freq.numel() == rot_dims // 2)
    kp, vp, stride = _pool_ptrs(pool, pool_slice)
    if pool is not None:
        assert pool.dtype == rows.dtype and block_table.is_contiguous() and tok_seq.dtype == torch.int32
    q = torch.empty((n, num_q_heads * k_dim), dtype=rows.dtype, device=rows.device)
    _hip.call("swl_qk_norm_rope_store_kv", _hip.ptr(rows), _hip.ptr(q), _hip.ptr(q_b), _hip.ptr(k_b), _hip.ptr(q_norm),
              _hip.ptr(k_norm), _hip.ptr(q_mult), _hip.ptr(freq), kp, vp, _hip.ptr(block_table), _hip.ptr(tok_seq),
              _hip.ptr(tok_pos), n, num_q_heads, num_k_heads, num_v_heads, dim, vdim, rot_dims, 1 if rot.half else 0,
              float(rot.multiplier), rows.stride(0), q.stride(0), k_dim, v_dim, 1 if num_v_heads == 0 else 0,
              block_table.shape[1] if block_table is not None else 0, stride, float(eps), _hip.dtype_code3(rows.dtype),
              _hip.stream())
    return q


def qkv_conv_rope_and_store_kv(rows: torch.Tensor, bias: torch.Tensor, conv_w: torch.Tensor, q_norm: torch.Tensor,
                               k_norm: torch.Tensor, freq: torch.Tensor, rot, pool: torch.Tensor, pool_slice: PoolSlice,
                               block_table: torch.Tensor, st, tail_off: int, num_q_heads: int, num_kv_heads: int, dim: int,
                               vdim: int, k_dim: int, v_dim: int, eps: float, v_mult: float = 1.0) -> torch.Tensor:
    """rows [q | k | v (| anything)] of one fused projection -> the queries [T, num_q_heads * k_dim]; keys and values go to the
    pool. Per channel: + bias (fp32 [q | k | v]), causal convolution over the sequence (conv_w fp32 tap-major [taps, q | k | v],
    carried inputs at tail_off inside the state slot); per q / k head: RMS norm with q_norm / k_norm, rotation; values times v_mult.
    Every step optional (None). st: the step's StateRef. k_dim / v_dim: row sizes in the pool and in the result, columns beyond the
    head zero. pool None (memory profiling): queries only."""
    _hip.require_gpu_tensor(rows, "rows")
    n = rows.shape[0]
    channels = (num_q_heads + num_kv_heads) * dim + num_kv_heads * vdim
    assert rows.dim() == 2 and rows.stride(1) == 1 and rows.shape[1] >= channels and st.tok_pos.shape[0] == n
    for t, size in ((bias, channels), (q_norm, dim), (k_norm, dim)):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.numel() == size)
    assert conv_w is None or (conv_w.dtype == torch.float32 and conv_w.is_contiguous() and conv_w.shape[1] == channels)
    rot_dims = rot.dims if freq is not None else 0
    assert freq is None or (freq.dtype == torch.float64 and freq.numel() == rot_dims // 2)
    kp, vp, stride = _pool_ptrs(pool, pool_slice)
    if pool is not None:
        assert pool.dtype == rows.dtype and block_table.is_contiguous()
    q = torch.empty((n, num_q_heads * k_dim), dtype=rows.dtype, device=rows.device)
    slots = st.pool if conv_w is not None else None
    _hip.call("swl_qkv_conv_rope_store_kv", _hip.ptr(rows), rows.stride(0), _hip.ptr(q), q.stride(0), _hip.ptr(bias),
              _hip.ptr(conv_w), conv_w.shape[0] if conv_w is not None else 0, _hip.ptr(q_norm), _hip.ptr(k_norm), _hip.ptr(freq),
              rot_dims, 1 if rot_dims == 0 or rot.half else 0, float(rot.multiplier) if rot_dims else 1.0, float(v_mult), kp, vp,
              _hip.ptr(block_table), block_table.shape[1] if block_table is not None else 0, stride, _hip.ptr(slots),
              slots.stride(0) if slots is not None else 0, int(tail_off), _hip.ptr(st.tok_pos), _hip.ptr(st.tok_start),
              _hip.ptr(st.tok_state), _hip.ptr(st.tok_seq), n, num_q_heads, num_kv_heads, dim, vdim, k_dim, v_dim, float(eps),
              _hip.dtype_code3(rows.dtype), _hip.stream())
    return q


def latent_rope_and_store_kv(proj: torch.Tensor, qa: torch.Tensor, freq: torch.Tensor, c_norm: torch.Tensor,
                             pool: torch.Tensor, pool_slice: PoolSlice, block_table: torch.Tensor, tok_seq: torch.Tensor,
                             tok_pos: torch.Tensor, mixer, dkv_col: int, eps: float, k_dim: int = 0, v_dim: int = 0):
    """proj rows: the query heads [dim | rot_dim] and, at column dkv_col (< 0: the layer reads another layer's cache), the
    compressed row [kv_rank | rot_dim]. Writes the rotated query parts into qa [T, heads, k_dim] (columns kv_rank .. kv_rank +
    rot_dim) and the normed latent + rotated shared key part into the pool. The layout of the pairs and the multiplier of the
    rotation are mixer.rot's. k_dim / v_dim: row sizes in qa and in the pool (default kv_rank + rot_dim / kv_rank), columns beyond
    zeroed."""
    _hip.require_gpu_tensor(proj, "proj")
    n = proj.shape[0]
    k_dim, v_dim = k_dim or mixer.kv_rank + mixer.rot_dim, v_dim or mixer.kv_rank
    assert proj.dim() == 2 and proj.stride(1) == 1 and qa.is_contiguous() and qa.dtype == proj.dtype
    assert qa.shape == (n, mixer.num_q_heads * k_dim)
    assert freq.dtype == torch.float64 and freq.numel() == mixer.rot_dim // 2
    assert tok_pos.dtype == torch.int32 and tok_pos.shape[0] == n
    kp, vp, stride = _pool_ptrs(pool if dkv_col >= 0 else None, pool_slice)
    if kp:
        assert pool.dtype == proj.dtype and c_norm.dtype == torch.float32 and c_norm.numel() == mixer.kv_rank
    _hip.call("swl_latent_rope_store_kv", _hip.ptr(proj), _hip.ptr(qa), _hip.ptr(freq), _hip.ptr(c_norm), kp, vp,
              _hip.ptr(block_table), _hip.ptr(tok_seq), _hip.ptr(tok_pos), n, mixer.num_q_heads, mixer.head_dim,
              mixer.rot_dim, mixer.kv_rank, proj.stride(0), dkv_col if kp else -1, qa.stride(0),
              block_table.shape[1] if block_table is not None else 0, stride, float(eps), 1 if mixer.rot.half else 0,
              float(mixer.rot.multiplier), k_dim, v_dim, _hip.dtype_code3(proj.dtype), _hip.stream())


def diff_head_combine(maps: torch.Tensor, gate: torch.Tensor, lam: float, mult: float, eps: float, num_heads: int,
                      vdim: int, out_dtype: torch.dtype) -> torch.Tensor:
    """maps fp32 [T, 2 * heads * vdim] (map-major) -> [T, heads * vdim]: unit_rms(a1 - lam * a2) * mult * sigmoid(gate[t, h]).
    gate: [T, heads] logits, possibly a column slice of a wider matrix."""
    _hip.require_gpu_tensor(maps, "maps")
    n = maps.shape[0]
    assert maps.dtype == torch.float32 and maps.is_contiguous() and maps.shape[1] == 2 * num_heads * vdim
    assert gate is None or (gate.shape == (n, num_heads) and gate.stride(1) == 1 and gate.dtype == out_dtype)
    out = torch.empty((n, num_heads * vdim), dtype=out_dtype, device=maps.device)
    _hip.call("swl_diff_head_combine", _hip.ptr(out), _hip.ptr(maps), _hip.ptr(gate), gate.stride(0) if gate is not None else 0,
              float(lam), float(mult), float(eps), n, num_heads, vdim, _hip.dtype_code3(out_dtype), _hip.stream())
    return out


def head_gate_(y: torch.Tensor, gate: torch.Tensor, num_heads: int, vdim: int) -> torch.Tensor:
    """In place: y[t, h, :] *= sigmoid(gate[t, h])."""
    _hip.require_gpu_tensor(y, "y")
    n = y.shape[0]
    assert y.is_contiguous() and y.shape[1] == num_heads * vdim
    assert gate.shape == (n, num_heads) and gate.stride(1) == 1 and gate.dtype == y.dtype
    _hip.call("swl_head_gate", _hip.ptr(y), _hip.ptr(gate), gate.stride(0), n, num_heads, vdim, _hip.dtype_code3(y.dtype),
              _hip.stream())
    return y
