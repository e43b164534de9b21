"""Weight containers and checkpoint reader for Vafozen.

Tensor names are the checkpoint's: `embed`, `final.norm`, `head`, and per layer `l<i>.`: `norm1`, the mixer's `mix.*` (a side-by-side
layer's two mixers under `mix.left.*` / `mix.right.*`) and the feed-forward's `mlp.*`. Linear weights are [out, in].

Every half of a layer reads the same normed input and every result is added to the same stream, so a layer needs ONE matrix on the
way in and ONE on the way out:
  * `proj`: the rows of all projections of the normed input, a piece per consumer (`cols[name]` = its columns in the product),
    pieces on multiples of 8 rows (16-byte boundaries in the product), zero rows between;
  * `out`: the output projections side by side along the input dimension (`ins[name]` likewise). What precedes it writes into one
    row per token; the factors of the two mixers are applied there (left: to the values as they are cached, right: by the head norm).
Time mixing reads token-shifted mixes of the input, so its r / k / v / gate matrices are a stack of their own (`shifted`, [4 inner, width]:
one grouped product).
Low-rank decay matrices are padded with zero rows / columns to a rank that is a power of two from 16 on (what the matrix-core form
takes) in 16-bit models; their rank is the checkpoint tensor's.
Everything that enters fp32 arithmetic — norm weights (the layers' and the model's are stored around zero: kept as 1 + w), biases, q/k
norm weights, convolutions (stored [channels, taps], kept tap-major), mixing vectors, bonus, recurrence constants — is kept in fp32
(exact: the checkpoint holds bfloat16). Shapes are checked against config.json before anything is used.
"""
import math
from typing import List

import torch

from .kekapel_weight import Getter, _checkpoint_getter
from .kernels.rope_kv import rotary_frequencies

_ALIGN = 8


class _Pieces:
    """Matrices stacked along `dim` on multiples of _ALIGN, and where each of them is."""

    def __init__(self, dim: int):
        self.dim, self.parts, self.at, self.size = dim, [], {}, 0

    def add(self, name: str, t: torch.Tensor):
        n = t.shape[self.dim]
        self.at[name] = slice(self.size, self.size + n)
        self.parts.append(t)
        self._pad(t, -n % _ALIGN)
        self.size += n + -n % _ALIGN

    def _pad(self, like: torch.Tensor, n: int):
        if n:
            shape = list(like.shape)
            shape[self.dim] = n
            self.parts.append(torch.zeros(shape, dtype=like.dtype, device=like.device))

    def cat(self, multiple: int = _ALIGN) -> torch.Tensor:
        """One matrix, its size along `dim` a multiple of `multiple`."""
        extra = -self.size % multiple
        self._pad(self.parts[0], extra)
        self.size += extra
        return torch.cat(self.parts, dim=self.dim).contiguous()

    @property
    def has_gaps(self) -> bool:
        """Columns that belong to no piece."""
        return sum(s.stop - s.start for s in self.at.values()) != self.size


class VafozenLayerWeight:
    def __init__(self, layer_id: int):
        self.layer_id = layer_id

    def load(self, get: Getter, cfg, lcfg, dtype, device):
        w, mx, p = cfg.hidden_size, lcfg.mixer, f"l{self.layer_id}."

        def f32(name, shape):
            return get(p + name, shape).to(device=device, dtype=torch.float32).contiguous()

        def mat(name, shape):
            return get(p + name, shape).to(device=device, dtype=dtype).contiguous()

        def low_rank(first, second, channels):
            """-> (W1 [rank, width], W2 [channels, rank])"""
            a, b = mat(first, (None, w)), mat(second, (channels, None))
            rank = a.shape[0]
            if b.shape[1] != rank:
                raise ValueError(f"{p}{first} and {p}{second}: ranks differ ({rank} vs {b.shape[1]})")
            if dtype != torch.float32:
                padded = max(16, 1 << (rank - 1).bit_length())
                a = torch.cat((a, torch.zeros((padded - rank, w), dtype=dtype, device=device)))
                b = torch.cat((b, torch.zeros((channels, padded - rank), dtype=dtype, device=device)), dim=1)
            return a.contiguous(), b.contiguous()

        self.norm1 = 1.0 + f32("norm1", (w,))
        self.y_bias = None
        ins, outs = _Pieces(0), _Pieces(1)
        if lcfg.type == "mamba2":
            ins.add("in", mat("mix.in", (mx.proj_size, w)))
            outs.add("mixer", mat("mix.o", (w, mx.inner)))
            C, H = mx.conv_channels, mx.num_heads
            self.conv = f32("mix.conv", (C, mx.conv_taps)).t().contiguous()      # tap-major
            self.conv_b = f32("mix.conv.b", (C,))
            self.dt_bias, self.a_log, self.d_skip = f32("mix.dt_bias", (H,)), f32("mix.A_log", (H,)), f32("mix.D", (H,))
            self.right_norm = f32("mix.norm", (mx.inner,))
        else:
            lf, rt = mx.left, mx.right
            sizes = {"q": lf.q_size, "k": lf.k_size, "v": lf.v_size}
            q, r = "mix.left.", "mix.right."
            ins.add("qkv", torch.cat([mat(q + n, (s, w)) for n, s in sizes.items()]))
            self.qkv_b = torch.cat([f32(f"{q}{n}.b", (s,)) for n, s in sizes.items()]).contiguous()
            self.y_bias = (mx.left_scale * f32(q + "o.b", (w,))).contiguous()
            outs.add("left", mat(q + "o", (w, lf.o_size)))
            outs.add("right", mat(r + "o", (w, rt.inner)))
            self.q_norm = self.k_norm = self.conv = None
            self.freq = rotary_frequencies(lf.rot, device)
            slopes = lf.slopes()
            self.slopes = torch.tensor(slopes, dtype=torch.float64).to(device=device, dtype=torch.float32) if slopes else None
            if lcfg.type == "parallel":
                self.q_norm, self.k_norm = f32(q + "q.norm", (lf.head_dim,)), f32(q + "k.norm", (lf.head_dim,))
                a1, self.decay_2 = low_rank(r + "a1", r + "a2", rt.keys)
                for n, s in (("q", rt.keys), ("k", rt.keys), ("v", rt.inner), ("g", rt.inner)):
                    ins.add("right_" + n, mat(r + n, (s, w)))
                ins.add("decay", a1)
                self.decay_b = f32(r + "a2.b", (rt.keys,))
                self.right_norm = f32(r + "norm", (rt.value_dim,))
            else:
                if lf.conv_taps:
                    self.conv = torch.cat([f32(f"{q}{n}.conv", (s, lf.conv_taps)) for n, s in sizes.items()]).t().contiguous()
                ins.add("gate", mat(q + "g", (lf.o_size, w)))
                self.mu = torch.stack([f32(f"{r}mu.{s}", (w,)) for s in "rkvgw"]).contiguous()
                self.shifted = torch.cat([mat(r + s, (rt.inner, w)) for s in "rkvg"]).contiguous()
                self.decay_1, self.decay_2 = low_rank(r + "w1", r + "w2", rt.keys)
                self.decay_b = f32(r + "w0", (rt.keys,))
                self.bonus = f32(r + "u", (rt.num_heads, rt.key_dim))
                self.right_norm = f32(r + "norm", (rt.inner,))
        if lcfg.mlp is not None:
            ff = lcfg.mlp.ffn_inter_dim
            ins.add("ff_gate", mat("mlp.gate", (ff, w)))
            ins.add("ff_up", mat("mlp.up", (ff, w)))
            outs.add("ff", mat("mlp.down", (w, ff)))
        self.proj, self.out = ins.cat(32), outs.cat()
        self.cols, self.ins = ins.at, outs.at
        self.row_size, self.row_gaps = outs.size, outs.has_gaps


class VafozenWeight:
    def __init__(self, model_config, dtype: torch.dtype):
        self.model_config = model_config
        self.dtype = dtype
        self.layers = [VafozenLayerWeight(i) for i in range(model_config.num_layers)]

    def load(self, get: Getter, device):
        cfg, dtype = self.model_config, self.dtype
        w = cfg.hidden_size
        self.embed = get("embed", (cfg.vocab_size, w)).to(device=device, dtype=dtype).contiguous()
        self.final_norm = (1.0 + get("final.norm", (w,)).to(device=device, dtype=torch.float32)).contiguous()
        self.head = get("head", (cfg.vocab_size, w)).to(device=device, dtype=dtype).contiguous()
        for layer, lcfg in zip(self.layers, cfg.layers):
            layer.load(get, cfg, lcfg, dtype, device)

    def projection_tensors(self) -> List[torch.Tensor]:
        """The 2-D matrices a step multiplies through `linear` (candidates for the decode GEMMs' packed copies)."""
        out = [self.head]
        for layer in self.layers:
            out += [layer.proj, layer.out] + ([layer.shifted] if hasattr(layer, "shifted") else [])
        return out


def _dummy_getter(seed: int = 0) -> Getter:
    """Random weights of the checkpoint's shapes (benchmarks, memory profiling): matrices ~ N(0, 1/in), weights stored around zero and
    biases small, recurrence constants of order one — a stream that stays finite at any depth. Low-rank decays have rank 64."""
    g = torch.Generator().manual_seed(seed)

    def get(name: str, shape: tuple) -> torch.Tensor:
        leaf = name.split(".")[-1]
        shape = tuple(64 if s is None else s for s in shape)
        if ".mu." in name:
            return torch.rand(shape, generator=g)
        if len(shape) == 2 and leaf != "u":
            return torch.randn(shape, generator=g) / math.sqrt(shape[1])
        if leaf == "w0":
            return -3.0 + torch.rand(shape, generator=g)
        if leaf in ("A_log", "dt_bias", "u"):
            return 0.5 * torch.randn(shape, generator=g)
        if leaf in ("D", "norm") and name != "final.norm":
            return 1.0 + 0.02 * torch.randn(shape, generator=g)
        return 0.02 * torch.randn(shape, generator=g)
    return get


def load_vafozen_weights(model_config, dtype: torch.dtype, model_path: str, use_dummy: bool = False,
                         device="cuda") -> VafozenWeight:
    weight = VafozenWeight(model_config, dtype)
    get = _dummy_getter() if use_dummy else _checkpoint_getter(model_path)
    weight.load(get, torch.device(device))
    return weight
