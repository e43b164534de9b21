"""A plain, slow evaluation of the Rokevik design: one function per mechanism, straight from the equations, on ONE sequence
given whole, in the dtype of the weights handed in (float32 or float64; nothing is rounded to 16 bits). It shares no code with
swiftllm_amd: the tests compare the framework's kernels, cache and state handling with it.

Notation: W["name"] is a checkpoint tensor, X [S, T, width] the S streams, h [T, width] a sublayer's input, positions i (query)
and j (key) count from 0.

    streams:    u = sum_s a_s X_s;  y = f(N(u));  X_t <- sum_s M[s, t] X_s + b_t y   (a, b, M per sublayer; the model reads sum_s X_s)
    norm:       N splits the vector into equal parts, every part over its own sqrt(mean square + eps), the whole times w
    attention:  q, k with biases, per-head weighted RMS norm, rotate-half rotary; values are the biased projected keys;
                score c tanh(scale temp_h q.k / c), softmax over j <= i, heads times sigmoid(gate), biased output projection
    latent:     c = normed compressed row, one rotated key part for all heads (angles by parts interpolated), keys U_k c and
                values U_v c per head, softmax over 0 <= i - j < window, heads times sigmoid(gate)
    min GRU:    S <- (1 - z) S + z g(u), z = sigmoid(.), g(u) = u + 1/2 for u >= 0 and sigmoid(u) below; W_o (S silu(gate))
    experts:    sum over the top experts of f_e(s_e h) with s = sigmoid(router h), plus the shared expert
"""
import math

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    T, width = x.shape
    return rms(x.reshape(T, groups, width // groups), eps).reshape(T, width) * w


def silu(z):
    return z * torch.sigmoid(z)


def rotary_frequencies(rot):
    """-> (frequencies, multiplier of cos and sin); with `scaling`, slow dimensions are slowed down by `factor`, fast ones kept."""
    dims, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def turns_at(t):
        return dims * math.log(sc["original"] / (2 * math.pi * t)) / (2 * math.log(base))
    lo = max(math.floor(turns_at(sc["fast"])), 0)
    hi = min(math.ceil(turns_at(sc["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate_half(x, pos, rot):
    """x [T, heads, d]: dimension i < dims / 2 turns with dimension i + dims / 2."""
    if not rot or rot["dims"] == 0:
        return x
    f, mult = rotary_frequencies(rot)
    half = rot["dims"] // 2
    ang = pos.double()[:, None] * torch.tensor(f, dtype=torch.float64)[None, :]
    c, s = (torch.cos(ang) * mult).to(x.dtype)[:, None, :], (torch.sin(ang) * mult).to(x.dtype)[:, None, :]
    u, v, rest = x[..., :half], x[..., half:2 * half], x[..., 2 * half:]
    return torch.cat((u * c - v * s, v * c + u * s, rest), dim=-1)


def softmax_heads(q, k, v, scale, visible, softcap=0.0, temp=None):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for h in range(H):
        s = (q[:, h] @ k[:, h // (H // G)].T) * scale
        if temp is not None:
            s = s * temp[h]
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(~visible, float("-inf"))
        out.append(torch.softmax(s, dim=-1) @ v[:, h // (H // G)])
    return torch.stack(out, dim=1)


def causal(T, window=0):
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    return (j <= i) & ((i - j < window) if window else torch.ones(T, T, dtype=torch.bool))


def gate_heads(o, h, Wg):
    return (o * torch.sigmoid(h @ Wg.T)[:, :, None]).reshape(o.shape[0], -1)


def attention_mixer(h, W, p, mx, eps):
    T = h.shape[0]
    H, G, d = mx["heads"], mx["kv_heads"], mx["dim"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, d)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, d)
    v = k
    pos = torch.arange(T)
    q = rotate_half(rms(q, eps) * W[p + "q.norm"], pos, mx.get("rot"))
    k = rotate_half(rms(k, eps) * W[p + "k.norm"], pos, mx.get("rot"))
    o = softmax_heads(q, k, v, mx["scale"], causal(T), mx.get("softcap") or 0.0, W[p + "temp"])
    return gate_heads(o, h, W[p + "g"]) @ W[p + "o"].T + W[p + "o.b"]


def latent_rows(h, W, p, mx, eps):
    """-> (latent [T, r], rotated shared key part [T, 1, dr])."""
    T, r = h.shape[0], mx["kv_rank"]
    z = h @ W[p + "dkv"].T
    c = rms(z[:, :r], eps) * W[p + "dkv.norm"]
    return c, rotate_half(z[:, r:].reshape(T, 1, -1), torch.arange(T), mx["rot"])


def latent_mixer(h, W, p, mx, eps):
    T = h.shape[0]
    H, d, dr, e = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    q = (h @ W[p + "q"].T).view(T, H, d + dr)
    q = torch.cat((q[..., :d], rotate_half(q[..., d:], torch.arange(T), mx["rot"])), dim=-1)
    c, kr = latent_rows(h, W, p, mx, eps)
    k = torch.cat(((c @ W[p + "uk"].T).view(T, H, d), kr.expand(T, H, dr)), dim=-1)
    v = (c @ W[p + "uv"].T).view(T, H, e)
    o = softmax_heads(q, k, v, mx["scale"], causal(T, (mx.get("mask") or {}).get("size", 0)))
    return gate_heads(o, h, W[p + "g"]) @ W[p + "o"].T


def min_gru_states(z, u, start=None):
    """z, u [T, n]: gate values in (0, 1) and raw candidates -> the states after every token."""
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    S = torch.zeros_like(z[0]) if start is None else start
    out = []
    for t in range(z.shape[0]):
        S = (1 - z[t]) * S + z[t] * cand[t]
        out.append(S)
    return torch.stack(out)


def min_gru_mixer(h, W, p, mx, eps):
    z = torch.sigmoid(h @ W[p + "z"].T + W[p + "z.b"])
    u = h @ W[p + "x"].T + W[p + "x.b"]
    return (min_gru_states(z, u) * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def expert(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def route(z, top):
    s = torch.sigmoid(z)
    idx = s.topk(top, dim=-1).indices
    return idx, s.gather(1, idx)


def moe_ff(h, W, p, mlp):
    idx, w = route(h @ W[p + "router"].T, mlp["router"]["top"])
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        for j in range(idx.shape[1]):
            rows = (idx[:, j] == e).nonzero()[:, 0]
            if rows.numel():
                out[rows] += expert(w[rows, j:j + 1] * h[rows], W, f"{p}e{e}.")
    if mlp.get("shared"):
        out = out + expert(h, W, p + "shared.")
    return out


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer, "mingru": min_gru_mixer}


def layer_order(cfg):
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    return list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n))


def hyper_step(X, y, mix, out):
    """X [S, T, w] -> the streams after a sublayer that returned y: X_t = sum_s mix[s, t] X_s + out[t] y, from the old streams."""
    return torch.stack([sum(mix[s, t] * X[s] for s in range(X.shape[0])) + out[t] * y for t in range(X.shape[0])])


def forward(cfg, W, tokens, taps=None):
    """-> logits [T, vocab]; taps (a list): the sum of the streams after every layer run."""
    eps, groups, S = cfg["norm"]["eps"], cfg["norm"].get("groups", 1), cfg.get("streams")
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    X = x.expand(S or 1, *x.shape)
    for i in layer_order(cfg):
        layer, p = cfg["layers"][i], f"l{i}."

        def update(X, q, f):
            if not S:
                return X + f(group_norm(X[0], W[f"{p}norm{q}"], groups, eps))
            u = sum(W[f"{p}hc{q}.in"][s] * X[s] for s in range(S))
            return hyper_step(X, f(group_norm(u, W[f"{p}norm{q}"], groups, eps)), W[f"{p}hc{q}.mix"], W[f"{p}hc{q}.out"])
        X = update(X, 1, lambda h: MIXERS[layer["type"]](h, W, p + "mix.", layer["mixer"], eps))
        if layer.get("mlp"):
            X = update(X, 2, lambda h: moe_ff(h, W, p + "mlp.", layer["mlp"]))
        if taps is not None:
            taps.append(X.sum(0))
    z = group_norm(X.sum(0), W["final.norm"], groups, eps) @ W["head"].T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(z / cap) if cap else z


# ---- random models for the tests -------------------------------------------------------------------------------------------
def tensor_shapes(cfg):
    """name -> shape of every tensor a checkpoint of `cfg` holds."""
    w, S = cfg["width"], cfg.get("streams")
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,), "head": (cfg["vocab"], w)}
    for i, layer in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", layer["mixer"]
        m = p + "mix."
        out[p + "norm1"] = (w,)
        if layer["type"] == "attention":
            H, G, d = mx["heads"], mx["kv_heads"], mx["dim"]
            out.update({m + "q": (H * d, w), m + "q.b": (H * d,), m + "k": (G * d, w), m + "k.b": (G * d,), m + "q.norm": (d,),
                        m + "k.norm": (d,), m + "temp": (H,), m + "g": (H, w), m + "o": (w, H * d), m + "o.b": (w,)})
        elif layer["type"] == "latent_attention":
            H, d, dr, e, r = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
            out.update({m + "q": (H * (d + dr), w), m + "dkv": (r + dr, w), m + "dkv.norm": (r,), m + "uk": (H * d, r),
                        m + "uv": (H * e, r), m + "g": (H, w), m + "o": (w, H * e)})
        else:
            n = mx["width"]
            out.update({m + "z": (n, w), m + "z.b": (n,), m + "x": (n, w), m + "x.b": (n,), m + "g": (n, w), m + "o": (w, n)})
        mlp = layer.get("mlp")
        if mlp:
            out[p + "norm2"] = (w,)
            units = [(f"{p}mlp.e{e}.", mlp["expert"]["ff"]) for e in range(mlp["router"]["experts"])]
            if mlp.get("shared"):
                units.append((p + "mlp.shared.", mlp["shared"]["ff"]))
            for u, ff in units:
                out.update({u + "gate": (ff, w), u + "up": (ff, w), u + "down": (w, ff)})
            out[p + "mlp.router"] = (mlp["router"]["experts"], w)
        if S:
            for q in ("1", "2") if mlp else ("1",):
                out.update({f"{p}hc{q}.in": (S,), f"{p}hc{q}.out": (S,), f"{p}hc{q}.mix": (S, S)})
    return out


def random_weights(cfg, seed=0):
    """Random tensors with bfloat16-representable values (float32), sized so that every mechanism matters in the output."""
    g = torch.Generator().manual_seed(seed)
    W = {}
    for name, shape in tensor_shapes(cfg).items():
        leaf, rand = name.split(".")[-1], torch.randn(shape, generator=g)
        if ".hc" in name:
            if leaf == "mix":
                t = 0.8 * torch.eye(shape[0]) + 0.2 * torch.rand(shape, generator=g)
            else:
                t = 0.4 + 0.6 * torch.rand(shape, generator=g)
        elif "norm" in leaf:
            t = 1.0 + 0.2 * rand
        elif leaf == "temp":
            t = 0.6 + 0.9 * torch.rand(shape, generator=g)
        elif name.endswith("z.b"):
            t = -1.5 + 1.5 * rand        # (slow and fast channels)
        elif leaf == "b":
            t = 0.3 * rand
        elif leaf == "embed":
            t = rand
        elif leaf == "router":
            t = 2.0 * rand / shape[1] ** 0.5
        else:
            t = rand / shape[1] ** 0.5
        W[name] = t.to(torch.bfloat16).to(torch.float32)
    return W


def write_checkpoint(path, cfg, W):
    """config.json and model.safetensors (bfloat16) in the folder `path`."""
    import json
    import os

    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return str(path)


# ---- configurations for the tests ------------------------------------------------------------------------------------------
def moe(ff=24, experts=5, top=2, shared=16):
    mlp = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared}
    return mlp


def attention_layer(heads=4, kv_heads=2, dim=16, rot_dims=8, base=300.0, scale=None, softcap=20.0, mlp="moe"):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale}
    if softcap:
        mx["softcap"] = softcap
    if rot_dims:
        mx["rot"] = {"dims": rot_dims, "base": base}
    return {"type": "attention", "mixer": mx, "mlp": moe() if mlp == "moe" else mlp}


def latent_layer(heads=3, dim=12, rot_dim=8, vdim=10, kv_rank=20, window=24, base=5000.0, scale=None, factor=4.0, original=64,
                 fast=16.0, slow=1.0, mlp="moe"):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
          "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"dims": rot_dim, "base": base}}
    if window:
        mx["mask"] = {"size": window}
    if factor:
        mx["rot"]["scaling"] = {"factor": factor, "original": original, "fast": fast, "slow": slow}
    return {"type": "latent_attention", "mixer": mx, "mlp": moe() if mlp == "moe" else mlp}


def min_gru_layer(width=56, mlp="moe"):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": moe() if mlp == "moe" else mlp}


def make_config(layers=None, width=48, vocab=61, eps=1e-5, groups=3, streams=3, loop=(1, 3, 2), logit_softcap=12.0):
    if layers is None:
        layers = [latent_layer(), attention_layer(), min_gru_layer(), latent_layer(heads=2, window=7, mlp=None)]
    cfg = {"architecture": "Rokevik", "layers": layers, "width": width, "vocab": vocab, "norm": {"eps": eps, "groups": groups}}
    if streams:
        cfg["streams"] = streams
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    if logit_softcap:
        cfg["logit_softcap"] = logit_softcap
    return cfg
