"""A plain, slow evaluation of the Vafozen design: one function per mechanism, straight from the equations, on ONE sequence given
whole, in the dtype of the weights handed in (float32 or float64; nothing is rounded to 16 bits). It shares no code with
swiftllm_amd: the tests compare the framework's kernels, cache and state handling with it.

Notation: h [T, width] is the one normed input that both halves of a layer read, W["name"] a checkpoint tensor, positions i
(query) and j (key) count from 0, S a recurrent state of one head [key channels, value channels].

    layer:       x <- x + mixer(h) + ff(h),   h = N(x) = (1 + w) x / r(x),  r(x)^2 = mean(x^2) + eps
    parallel:    a softmax attention (biases, weighted q/k norm, scale q.k - slope_h (i - j), keys of the query's own chunk)
                 and a linear attention with a decay per key channel: S <- diag(alpha) S + k v^T, o = S^T q
    parallel_2:  a softmax attention (biases, causal convolutions, rotation by halves, capped scores, element-wise gate)
                 and a time mixing of shifted inputs: o = (S + diag(u) k v^T)^T r, then S <- diag(w) S + k v^T
    mamba2:      S <- exp(-exp(A) dt) S + dt B x^T, y = S^T C + D x, convolution in front, gate and grouped norm behind
    ff:          down(silu(gate h) * up h)
"""
import math

import torch


# ---- pieces --------------------------------------------------------------------------------------------------------------
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def layer_norm1p(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * (1 + w)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def causal_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """u [T, C], w [C, taps]: y_t = sum over lags l of w[:, taps - 1 - l] u_(t - l), where u is zero at negative times."""
    T, C = u.shape
    taps = w.shape[1]
    padded = torch.cat((torch.zeros(taps - 1, C, dtype=u.dtype), u), dim=0)
    out = torch.zeros_like(u)
    for j in range(taps):
        out = out + padded[j:j + T] * w[:, j]
    return out


def rotate_halves(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, d]: dimension i < dims / 2 turns with dimension i + dims / 2 by the angle position * base^(-2 i / dims)."""
    T = x.shape[0]
    half = dims // 2
    pos = torch.arange(T, dtype=torch.float64).view(T, 1)
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64).view(1, half)
    c = torch.cos(pos * freq).to(x.dtype).view(T, 1, half)
    s = torch.sin(pos * freq).to(x.dtype).view(T, 1, half)
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat((u * c - v * s, v * c + u * s, rest), dim=-1)


def head_slope(h: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (h + 1) / heads)


def attend(q, k, v, score, visible):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; score(h, q_h k_h^T) -> scores [T, T]; visible [T, T] bool -> [T, H * dv]."""
    T, H = q.shape[:2]
    rep = H // k.shape[1]
    outs = []
    for h in range(H):
        s = score(h, q[:, h] @ k[:, h // rep].T).masked_fill(~visible, float("-inf"))
        outs.append(torch.softmax(s, dim=-1) @ v[:, h // rep])
    return torch.stack(outs, dim=1).reshape(T, -1)


def causal_mask(T: int, chunk: int = 0) -> torch.Tensor:
    i = torch.arange(T).view(T, 1)
    j = torch.arange(T).view(1, T)
    m = j <= i
    return m & (i // chunk == j // chunk) if chunk else m


def projections(h, W, p):
    return [h @ W[p + n].T + W[p + n + ".b"] for n in ("q", "k", "v")]


# ---- mixers --------------------------------------------------------------------------------------------------------------
def distance_attention(h, W, p, mx, eps):
    """The left half of `parallel`."""
    T, H, G, d, dv = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = projections(h, W, p)
    q = unit_rms(q.view(T, H, d), eps) * W[p + "q.norm"]
    k = unit_rms(k.view(T, G, d), eps) * W[p + "k.norm"]
    dist = (torch.arange(T).view(T, 1) - torch.arange(T).view(1, T)).to(h.dtype)
    out = attend(q, k, v.view(T, G, dv), lambda hh, qk: qk * mx["scale"] - head_slope(hh, H) * dist,
                 causal_mask(T, (mx.get("mask") or {}).get("size", 0)))
    return out @ W[p + "o"].T + W[p + "o.b"]


def linear_scan(q, k, v, decay):
    """q, k, decay [T, H, d], v [T, H, dv]: S <- diag(decay) S + k v^T, o = S^T q -> [T, H, dv]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = []
    for t in range(T):
        S = decay[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out.append((S * q[t].unsqueeze(-1)).sum(dim=1))
    return torch.stack(out)


def bonus_scan(r, k, v, decay, u):
    """o = (S + diag(u) k v^T)^T r with the state of the tokens before, then S <- diag(decay) S + k v^T. u [H, d]."""
    T, H, d = r.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=r.dtype)
    out = []
    for t in range(T):
        kv = k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out.append(((S + u.unsqueeze(-1) * kv) * r[t].unsqueeze(-1)).sum(dim=1))
        S = decay[t].unsqueeze(-1) * S + kv
    return torch.stack(out)


def gated_linear_attention(h, W, p, mx, eps):
    """The right half of `parallel`."""
    T, H, d, dv = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ W[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, d)
    v = (h @ W[p + "v"].T).view(T, H, dv)
    z = h @ W[p + "a1"].T @ W[p + "a2"].T + W[p + "a2.b"]
    alpha = torch.sigmoid(z).pow(1.0 / mx["tau"]).view(T, H, d)
    o = unit_rms(linear_scan(q, k, v, alpha), eps) * W[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def convolved_attention(h, W, p, mx):
    """The left half of `parallel_2`."""
    T, H, G, d, dv = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (causal_conv(u, W[p + n + ".conv"]) for n, u in zip("qkv", projections(h, W, p)))
    q = rotate_halves(q.view(T, H, d), mx["rot"]["dims"], mx["rot"]["base"])
    k = rotate_halves(k.view(T, G, d), mx["rot"]["dims"], mx["rot"]["base"])
    cap = mx["softcap"]
    out = attend(q, k, v.view(T, G, dv), lambda hh, qk: cap * torch.tanh(qk * mx["scale"] / cap), causal_mask(T))
    return (out * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T + W[p + "o.b"]


def time_mixing(h, W, p, mx, eps):
    """The right half of `parallel_2`."""
    T, H, d = h.shape[0], mx["heads"], mx["dim"]
    prev = torch.cat((torch.zeros_like(h[:1]), h[:-1]), dim=0)
    mix = {s: h + (prev - h) * W[f"{p}mu.{s}"] for s in "rkvgw"}
    r, k, v = ((mix[s] @ W[p + s].T).view(T, H, d) for s in "rkv")
    w = torch.exp(-torch.exp(torch.tanh(mix["w"] @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"])).view(T, H, d)
    o = unit_rms(bonus_scan(r, k, v, w, W[p + "u"]), eps).reshape(T, H * d)
    return (o * W[p + "norm"] * silu(mix["g"] @ W[p + "g"].T)) @ W[p + "o"].T


def state_space(h, W, p, mx, eps):
    """The mixer `mamba2`."""
    T = h.shape[0]
    H, P, N, G = mx["heads"], mx["vdim"], mx["state"], mx["groups"]
    inner = H * P
    proj = h @ W[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, W[p + "conv"]) + W[p + "conv.b"])
    x = xbc[:, :inner].view(T, H, P)
    group = torch.arange(H) // (H // G)
    B = xbc[:, inner:inner + G * N].view(T, G, N)[:, group]
    C = xbc[:, inner + G * N:].view(T, G, N)[:, group]
    dt = torch.log1p(torch.exp(-(dt + W[p + "dt_bias"]).abs())) + (dt + W[p + "dt_bias"]).clamp_min(0)      # softplus
    decay = torch.exp(-torch.exp(W[p + "A_log"]) * dt)
    y = linear_scan(C, B * dt.unsqueeze(-1), x, decay.unsqueeze(-1).expand(T, H, N)) + W[p + "D"].unsqueeze(-1) * x
    parts = mx["norm_groups"]
    y = (y.reshape(T, inner) * silu(z)).view(T, parts, inner // parts)
    return (unit_rms(y, eps).reshape(T, inner) * W[p + "norm"]) @ W[p + "o"].T


def parallel(h, W, p, mx, eps):
    return mx["left_scale"] * distance_attention(h, W, p + "left.", mx["left"], eps) \
        + mx["right_scale"] * gated_linear_attention(h, W, p + "right.", mx["right"], eps)


def parallel_2(h, W, p, mx, eps):
    return mx["left_scale"] * convolved_attention(h, W, p + "left.", mx["left"]) \
        + mx["right_scale"] * time_mixing(h, W, p + "right.", mx["right"], eps)


MIXERS = {"parallel": parallel, "parallel_2": parallel_2, "mamba2": state_space}


# ---- the model -----------------------------------------------------------------------------------------------------------
def gated_unit(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def forward(config: dict, W: dict, tokens, taps: list = None) -> torch.Tensor:
    """-> logits [T, vocab]; `taps`, when given, receives the stream after every layer."""
    eps = config["norm"]["eps"]
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        h = layer_norm1p(x, W[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, W, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp"):
            y = y + gated_unit(h, W, p + "mlp.")
        x = x + y
        if taps is not None:
            taps.append(x.clone())
    return layer_norm1p(x, W["final.norm"], eps) @ W["head"].T


# ---- random models for the tests -----------------------------------------------------------------------------------------
def tensor_shapes(config: dict, rank: int = 5) -> dict:
    """name -> shape of every tensor a checkpoint of `config` holds. rank: of the low-rank decay projections (a layer's own under
    the test-only key mixer.right.rank)."""
    w = config["width"]
    out = {"embed": (config["vocab"], w), "final.norm": (w,), "head": (config["vocab"], w)}
    for i, layer in enumerate(config["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        out[p + "norm1"] = (w,)
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            out.update({p + "mlp.gate": (ff, w), p + "mlp.up": (ff, w), p + "mlp.down": (w, ff)})
        if layer["type"] == "mamba2":
            inner, gn = mx["heads"] * mx["vdim"], mx["groups"] * mx["state"]
            p += "mix."
            out.update({p + "in": (2 * inner + 2 * gn + mx["heads"], w), p + "conv": (inner + 2 * gn, mx["conv"]),
                        p + "conv.b": (inner + 2 * gn,), p + "dt_bias": (mx["heads"],), p + "A_log": (mx["heads"],),
                        p + "D": (mx["heads"],), p + "norm": (inner,), p + "o": (w, inner)})
            continue
        lf, rt = mx["left"], mx["right"]
        sizes = {"q": lf["heads"] * lf["dim"], "k": lf["kv_heads"] * lf["dim"], "v": lf["kv_heads"] * lf["vdim"]}
        q = p + "mix.left."
        for n, size in sizes.items():
            out.update({q + n: (size, w), q + n + ".b": (size,)})
        out.update({q + "o": (w, lf["heads"] * lf["vdim"]), q + "o.b": (w,)})
        r = p + "mix.right."
        rk = rt.get("rank", rank)
        if layer["type"] == "parallel":
            out.update({q + "q.norm": (lf["dim"],), q + "k.norm": (lf["dim"],)})
            kd, vd = rt["heads"] * rt["dim"], rt["heads"] * rt["vdim"]
            out.update({r + "q": (kd, w), r + "k": (kd, w), r + "v": (vd, w), r + "g": (vd, w), r + "o": (w, vd),
                        r + "norm": (rt["vdim"],), r + "a1": (rk, w), r + "a2": (kd, rk), r + "a2.b": (kd,)})
        else:
            out.update({q + n + ".conv": (size, lf["conv"]) for n, size in sizes.items()})
            out[q + "g"] = (lf["heads"] * lf["vdim"], w)
            n = rt["heads"] * rt["dim"]
            out.update({f"{r}mu.{s}": (w,) for s in "rkvgw"})
            out.update({r + s: (n, w) for s in "rkvg"})
            out.update({r + "w1": (rk, w), r + "w2": (n, rk), r + "w0": (n,), r + "u": (rt["heads"], rt["dim"]),
                        r + "norm": (n,), r + "o": (w, n)})
    return out


def random_weights(config: dict, seed: int = 0) -> dict:
    """Random tensors with bfloat16-representable values (float32), sized so that every mechanism matters in the output:
    recurrences that neither vanish nor blow up, gates and decays away from their flat ends."""
    g = torch.Generator().manual_seed(seed)

    def n(shape):
        return torch.randn(shape, generator=g)

    W = {}
    for name, shape in tensor_shapes(config).items():
        leaf = name.split(".")[-1]
        if leaf == "norm1" or name == "final.norm":
            t = 0.2 * n(shape)
        elif leaf == "norm":
            t = 1.0 + 0.2 * n(shape)
        elif leaf == "conv":
            t = n(shape) / shape[1] ** 0.5
        elif ".mu." in name:
            t = torch.rand(shape, generator=g)
        elif leaf == "A_log":
            t = -1.0 + 1.5 * torch.rand(shape, generator=g)
        elif leaf == "dt_bias":
            t = -2.0 + 2.0 * torch.rand(shape, generator=g)
        elif leaf == "w0":
            t = -3.0 + 3.0 * torch.rand(shape, generator=g)
        elif leaf == "D":
            t = 0.5 + torch.rand(shape, generator=g)
        elif leaf == "u":
            t = 0.5 + 0.5 * n(shape)
        elif leaf == "b":
            t = 0.3 * n(shape)
        elif leaf in ("a2", "w2"):
            t = 2.0 * n(shape) / shape[1] ** 0.5
        elif len(shape) == 2:
            t = n(shape) / shape[1] ** 0.5
        else:
            t = n(shape)
        W[name] = t.to(torch.bfloat16).to(torch.float32)
    return W


def write_checkpoint(path: str, config: dict, W: dict):
    """config.json and model.safetensors (bfloat16) in the folder `path`."""
    import json
    import os
    import struct
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
        json.dump(config, f)
    header, blobs, off = {}, [], 0
    for name, t in W.items():
        raw = t.to(torch.bfloat16).contiguous().view(torch.int16).numpy().tobytes()
        header[name] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [off, off + len(raw)]}
        blobs.append(raw)
        off += len(raw)
    head = json.dumps(header).encode()
    head += b" " * (-len(head) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(head)))
        f.write(head)
        for b in blobs:
            f.write(b)


# ---- configurations for the tests ----------------------------------------------------------------------------------------
def parallel_layer(heads=4, kv_heads=2, dim=16, vdim=24, chunk=20, scale=0.3, g_heads=3, g_dim=12, g_vdim=20, tau=8.0, rank=5,
                   left_scale=0.7, right_scale=1.3, ff=48):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        left["mask"] = {"size": chunk}
    return {"type": "parallel", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": left, "left_scale": left_scale, "right_scale": right_scale,
                      "right": {"heads": g_heads, "dim": g_dim, "vdim": g_vdim, "tau": tau, "rank": rank}}}


def parallel2_layer(heads=4, kv_heads=2, dim=16, vdim=20, conv=3, rot_dims=12, base=10000.0, scale=0.25, softcap=5.0, r_heads=3,
                    r_dim=12, rank=7, left_scale=1.1, right_scale=0.6, ff=48):
    return {"type": "parallel_2", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "scale": scale,
                               "softcap": softcap, "rot": {"base": base, "dims": rot_dims}},
                      "left_scale": left_scale, "right_scale": right_scale,
                      "right": {"heads": r_heads, "dim": r_dim, "rank": rank}}}


def mamba_layer(heads=4, vdim=12, state=20, groups=2, conv=3, norm_groups=3, ff=40):
    return {"type": "mamba2", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}}


def make_config(layers=None, width=40, vocab=61, eps=1e-5, scale=3.0, max_positions=None):
    if layers is None:
        layers = [parallel_layer(), parallel2_layer(), mamba_layer(), parallel2_layer(conv=4, ff=0), parallel_layer(chunk=33)]
    cfg = {"architecture": "Vafozen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "layers": layers}
    if max_positions:
        cfg["max_positions"] = max_positions
    return cfg
