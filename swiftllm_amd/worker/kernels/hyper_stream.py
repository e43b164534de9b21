"""The fp32 residual of models with hyper-connections: several streams per token, mixed by every sublayer.
csrc/hyper_stream.hip."""
import torch

from swiftllm_amd import _hip

from .linear import SplitKPartials


class StreamWeights:
    """How one sublayer reads and writes the streams (fp32): u = sum_s read[s] X_s; X_t <- sum_s mix[s, t] X_s + write[t] y."""
    __slots__ = ("read", "mix", "write")

    def __init__(self, read: torch.Tensor, mix: torch.Tensor, write: torch.Tensor):
        assert read.dtype == mix.dtype == write.dtype == torch.float32 and mix.is_contiguous()
        assert read.dim() == write.dim() == 1 and mix.shape == (read.numel(), write.numel()) and mix.shape[0] == mix.shape[1]
        self.read, self.mix, self.write = read, mix, write

    @staticmethod
    def plain(device) -> "StreamWeights":
        """One stream: the ordinary residual x + f(x)."""
        one = torch.ones(1, dtype=torch.float32, device=device)
        return StreamWeights(one, one.view(1, 1), one)


def embed_streams(tokens: torch.Tensor, embed: torch.Tensor, streams: int) -> torch.Tensor:
    """-> x fp32 [T, streams, width]: every stream holds embed[tokens[t]]."""
    _hip.require_gpu_tensor(embed, "embed")
    n, width = tokens.shape[0], embed.shape[1]
    assert embed.is_contiguous() and tokens.dtype == torch.int32
    x = torch.empty((n, streams, width), dtype=torch.float32, device=embed.device)
    _hip.call("swl_embed_streams", _hip.ptr(x), _hip.ptr(embed), _hip.ptr(tokens), n, width, streams,
              _hip.dtype_code3(embed.dtype), _hip.stream())
    return x


def hyper_step(x: torch.Tensor, y: torch.Tensor = None, done: StreamWeights = None, y2: torch.Tensor = None,
               y_bias: torch.Tensor = None, read: torch.Tensor = None, norm: torch.Tensor = None, groups: int = 1,
               eps: float = 1e-6, out_dtype: torch.dtype = None, row_idx: torch.Tensor = None) -> torch.Tensor:
    """The step between two sublayers on the streams x [T, S, width], in place. y (+ y2, + y_bias [width] fp32): the result of the
    sublayer whose StreamWeights are `done`; y has one row per token, or k neighbouring ones (the results of its k experts) that
    are summed, or is a product's SplitKPartials, whose fp32 slabs are summed. norm (fp32 [width]): returns the next input, the sum of
    the streams weighted by
    `read` (None: plainly summed), RMS-normed in `groups` equal parts and scaled by `norm`, in y's dtype (out_dtype without a y) —
    of rows row_idx only, when given; then y must be None."""
    _hip.require_gpu_tensor(x, "x")
    n, streams, width = x.shape
    assert x.dtype == torch.float32 and x.is_contiguous() and (y is not None or norm is not None)
    slabs = y if isinstance(y, SplitKPartials) else None
    dtype = y.dtype if y is not None else out_dtype
    parts = 0
    if slabs is not None:
        assert slabs.shape == (n, width) and done.mix.shape[0] == streams
        parts, y = slabs.k_splits, None
    has_y = y is not None or slabs is not None
    if y is not None:
        parts = y.shape[0] // n
        assert y.shape[1] == width and y.shape[0] % n == 0 and y.is_contiguous() and done.mix.shape[0] == streams
        assert y2 is None or (y2.shape == (n, width) and y2.is_contiguous() and y2.dtype == y.dtype)
    assert read is None or (read.dtype == torch.float32 and read.numel() == streams)
    for w in (y_bias, norm):
        assert w is None or (w.dtype == torch.float32 and w.is_contiguous() and w.numel() == width)
    rows = n if row_idx is None else row_idx.shape[0]
    out = torch.empty((rows, width), dtype=dtype, device=x.device) if norm is not None else None
    _hip.call("swl_hyper_step", _hip.ptr(x), _hip.ptr(y), parts, _hip.ptr(slabs.slabs) if slabs is not None else 0, n * width,
              _hip.ptr(y2), _hip.ptr(y_bias), _hip.ptr(done.mix) if has_y else 0, _hip.ptr(done.write) if has_y else 0,
              _hip.ptr(read), _hip.ptr(norm), _hip.ptr(out), _hip.ptr(row_idx), rows, width, streams, int(groups), float(eps),
              _hip.dtype_code3(dtype), _hip.stream())
    return out
