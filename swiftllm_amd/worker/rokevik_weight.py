"""Weight containers and checkpoint reader for Rokevik.

Tensor names are the checkpoint's: `embed`, `final.norm`, `head`, and per layer `l<i>.`: `norm1 / norm2`, the mixer's `mix.*`, the
feed-forward's `mlp.*` and the stream weights `hc1.* / hc2.*` (`in`, `out`, `mix`). Linear weights are [out, in].

What the loader does with them:
  * matrices that multiply the same input are concatenated into one projection, padded with zero rows to a multiple of 8 rows so
    that every row of its output starts on a 16-byte boundary: attention q | k | head gate; latent attention q | compressed kv |
    head gate; minGRU z | x | gate; experts gate | up, stacked ([experts, 2 ff, width], [experts, width, ff]); the shared expert up | gate (the
    order of the decode GEMM that applies the gate itself);
  * the latent attention's up-projections are kept per head for batched products: uk [H, dim, kv_rank] (queries are folded
    through it) and uv^T [H, kv_rank, vdim] (applied to the attention's output over the latent rows);
  * everything that enters fp32 arithmetic — norm weights, biases, head temperatures, the router, the stream weights — is kept in
    fp32 (exact: the checkpoint holds bfloat16);
  * rotary frequencies: a float64 table per layer on the device, any interpolation included.
Shapes are checked against config.json before anything is used. A looped layer has one set of weights whatever its runs.
"""
import math
from typing import List

import torch

from .kekapel_weight import Getter, _checkpoint_getter
from .kernels.hyper_stream import StreamWeights
from .kernels.rope_kv import rotary_frequencies
from .rosilix_weight import _pad_rows


class RokevikLayerWeight:
    def __init__(self, layer_id: int):
        self.layer_id = layer_id

    def load(self, get: Getter, cfg, lcfg, dtype, device):
        w, mx, p = cfg.hidden_size, lcfg.mixer, f"l{self.layer_id}."

        def f32(name, shape):
            return get(p + name, shape).to(device=device, dtype=torch.float32).contiguous()

        def mat(name, shape):
            return get(p + name, shape).to(device=device, dtype=dtype).contiguous()

        def streams(name):
            s = cfg.num_streams
            if not s:
                return StreamWeights.plain(device)
            return StreamWeights(f32(name + ".in", (s,)), f32(name + ".mix", (s, s)), f32(name + ".out", (s,)))

        self.norm1, self.streams1 = f32("norm1", (w,)), streams("hc1")
        if lcfg.type == "attention":
            H = mx.num_q_heads
            self.freq = rotary_frequencies(mx.rot, device)
            self.proj = _pad_rows(torch.cat((mat("mix.q", (mx.q_size, w)), mat("mix.k", (mx.k_size, w)), mat("mix.g", (H, w))),
                                            dim=0))
            self.gate_col = mx.q_size + mx.k_size
            self.q_b, self.k_b, self.o_b = f32("mix.q.b", (mx.q_size,)), f32("mix.k.b", (mx.k_size,)), f32("mix.o.b", (w,))
            self.q_norm, self.k_norm = f32("mix.q.norm", (mx.head_dim,)), f32("mix.k.norm", (mx.head_dim,))
            self.temp = f32("mix.temp", (H,))
            self.o = mat("mix.o", (w, mx.o_size))
        elif lcfg.type == "latent_attention":
            H = mx.num_q_heads
            self.freq = rotary_frequencies(mx.rot, device)
            self.proj = _pad_rows(torch.cat((mat("mix.q", (mx.q_size, w)), mat("mix.dkv", (mx.dkv_size, w)),
                                             mat("mix.g", (H, w))), dim=0))
            self.gate_col = mx.q_size + mx.dkv_size
            self.c_norm = f32("mix.dkv.norm", (mx.kv_rank,))
            self.uk = mat("mix.uk", (H * mx.head_dim, mx.kv_rank)).view(H, mx.head_dim, mx.kv_rank).contiguous()
            self.uv_t = mat("mix.uv", (H * mx.value_dim, mx.kv_rank)).view(H, mx.value_dim, mx.kv_rank) \
                .transpose(1, 2).contiguous()
            self.o = mat("mix.o", (w, mx.o_size))
        else:
            n = mx.width
            self.proj = _pad_rows(torch.cat((mat("mix.z", (n, w)), mat("mix.x", (n, w)), mat("mix.g", (n, w))), dim=0))
            self.z_b, self.x_b = f32("mix.z.b", (n,)), f32("mix.x.b", (n,))
            self.o = mat("mix.o", (w, n))
        mlp = lcfg.mlp
        if mlp is None:
            return
        self.norm2, self.streams2 = f32("norm2", (w,)), streams("hc2")
        ff = mlp.ffn_inter_dim
        self.router = f32("mlp.router", (mlp.num_experts, w))
        self.gate_up = torch.empty((mlp.num_experts, 2 * ff, w), dtype=dtype, device=device)
        self.down = torch.empty((mlp.num_experts, w, ff), dtype=dtype, device=device)
        for e in range(mlp.num_experts):
            self.gate_up[e, :ff] = mat(f"mlp.e{e}.gate", (ff, w))
            self.gate_up[e, ff:] = mat(f"mlp.e{e}.up", (ff, w))
            self.down[e] = mat(f"mlp.e{e}.down", (w, ff))
        self.shared_up_gate = self.shared_down = None
        if mlp.shared_ffn_inter_dim:
            fs = mlp.shared_ffn_inter_dim
            self.shared_up_gate = torch.cat((mat("mlp.shared.up", (fs, w)), mat("mlp.shared.gate", (fs, w))), dim=0).contiguous()
            self.shared_down = mat("mlp.shared.down", (w, fs))


class RokevikWeight:
    def __init__(self, model_config, dtype: torch.dtype):
        self.model_config = model_config
        self.dtype = dtype
        self.layers = [RokevikLayerWeight(i) for i in range(model_config.num_layers)]

    def load(self, get: Getter, device):
        cfg, dtype = self.model_config, self.dtype
        w = cfg.hidden_size
        self.embed = get("embed", (cfg.vocab_size, w)).to(device=device, dtype=dtype).contiguous()
        self.final_norm = get("final.norm", (w,)).to(device=device, dtype=torch.float32).contiguous()
        self.head = get("head", (cfg.vocab_size, w)).to(device=device, dtype=dtype).contiguous()
        for layer, lcfg in zip(self.layers, cfg.layers):
            layer.load(get, cfg, lcfg, dtype, device)

    def projection_tensors(self) -> List[torch.Tensor]:
        """The 2-D matrices a step multiplies through `linear` (candidates for the decode GEMMs' packed copies)."""
        out = [self.head]
        for layer in self.layers:
            for a in ("proj", "o", "shared_up_gate", "shared_down"):
                t = getattr(layer, a, None)
                if t is not None:
                    out.append(t)
        return out


def _dummy_getter(seed: int = 0) -> Getter:
    """Random weights of the checkpoint's shapes (benchmarks, memory profiling): matrices ~ N(0, 1/in), norm weights and
    temperatures near one, biases small, streams that mix a little — values that stay finite through any depth."""
    g = torch.Generator().manual_seed(seed)

    def get(name: str, shape: tuple) -> torch.Tensor:
        leaf = name.split(".")[-1]
        if ".hc" in name:
            s = shape[0]
            return (0.9 * torch.eye(s) + 0.1 / s) if leaf == "mix" else torch.full(shape, 1.0 / s if leaf == "in" else 0.5)
        if len(shape) == 2:
            return torch.randn(shape, generator=g) / math.sqrt(shape[1])
        return 0.02 * torch.randn(shape, generator=g) + (0.0 if leaf == "b" else 1.0)
    return get


def load_rokevik_weights(model_config, dtype: torch.dtype, model_path: str, use_dummy: bool = False,
                         device="cuda") -> RokevikWeight:
    weight = RokevikWeight(model_config, dtype)
    get = _dummy_getter() if use_dummy else _checkpoint_getter(model_path)
    weight.load(get, torch.device(device))
    return weight
