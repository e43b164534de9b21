"""minGRU: an element-wise gated recurrence with per-sequence state slots. csrc/min_gru.hip."""
import torch

from swiftllm_amd import _hip

from ..batch_plan import StepPlan
from .rms_stream import StateRef


def min_gru(proj: torch.Tensor, z_b: torch.Tensor, u_b: torch.Tensor, st: StateRef, chunks, state_off: int,
            width: int) -> torch.Tensor:
    """proj [T, z | u | gate] (rows of the fused projection, biases z_b / u_b fp32 still to be added; a column slice of a wider
    matrix is fine) -> S * silu(gate) [T, width] in proj's dtype, S_t = (1 - a) S + a c per channel with a = sigmoid(z), c = u +
    1/2 for u >= 0 and sigmoid(u) below, in fp32 on the `width` floats at `state_off` of each sequence's slot. chunks =
    (chunk_row0, chunk_cnt, seq_chunk0): the step's portions cut into runs of up to StepPlan.CHUNK tokens; portions of more than
    one run are evaluated in parallel over them (three launches), a step of single runs in one launch."""
    _hip.require_gpu_tensor(proj, "proj")
    n = proj.shape[0]
    assert proj.dim() == 2 and proj.stride(1) == 1 and proj.shape[1] >= 3 * width
    for t in (z_b, u_b):
        assert t is None or (t.dtype == torch.float32 and t.is_contiguous() and t.numel() == width)
    row0, cnt, first = chunks
    nc, ns = row0.shape[0], st.seq_row0.shape[0]
    assert first.shape[0] == ns and 0 <= state_off <= st.pool.shape[1] - width
    code, stream = _hip.dtype_code3(proj.dtype), _hip.stream()
    part = None
    if nc > ns:
        part = torch.empty((nc, 2, width), dtype=torch.float32, device=proj.device)
        _hip.call("swl_min_gru_chunks", _hip.ptr(part), _hip.ptr(proj), proj.stride(0), _hip.ptr(z_b), _hip.ptr(u_b),
                  _hip.ptr(row0), _hip.ptr(cnt), nc, width, code, stream)
        _hip.call("swl_min_gru_carry", _hip.ptr(part), _hip.ptr(st.pool), st.pool.stride(0), int(state_off),
                  _hip.ptr(st.seq_row0), _hip.ptr(st.seq_cnt), _hip.ptr(first), _hip.ptr(st.tok_pos), _hip.ptr(st.tok_state),
                  ns, StepPlan.CHUNK, width, stream)
    out = torch.empty((n, width), dtype=proj.dtype, device=proj.device)
    _hip.call("swl_min_gru_apply", _hip.ptr(out), _hip.ptr(proj), proj.stride(0), _hip.ptr(z_b), _hip.ptr(u_b), _hip.ptr(part),
              _hip.ptr(st.pool), st.pool.stride(0), int(state_off), _hip.ptr(row0), _hip.ptr(cnt), _hip.ptr(st.tok_pos),
              _hip.ptr(st.tok_state), nc, width, code, stream)
    return out
