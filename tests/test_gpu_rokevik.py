"""Rokevik on the GPU against the plain implementation in tests/rokevik_oracle.py: every mechanism alone, whole prompts,
token-by-token decoding, portions down to two tokens, unequal batches, reused blocks and state slots, far keys, keys at page
borders and at both sides of a window's edge, the first tokens of a sequence, long decoding, odd sizes, hipGraph replays,
swapping, and greedy generation through the Engine and its scheduler. Configurations and weights are made here (small, random,
seeded)."""
import asyncio
import random

import pytest
import torch

import rokevik_oracle as O

pytestmark = pytest.mark.gpu

F32_TOL = 3e-5      # relative rms error of fp32 logits (true fp32 products, fp32 statistics)
BF16_TOL = 8e-2     # the same in bfloat16 (bf16 products and activations, fp32 streams, statistics and recurrences)
EPS = 1e-5


def f64(W):
    return {k: v.double() for k, v in W.items()}


def make_model(path, cfg, W, dtype="float32", num_blocks=48, max_seqs=4, cpu_blocks=0, graph=False, max_len=512):
    from swiftllm_amd import EngineConfig, build_model
    O.write_checkpoint(str(path), cfg, W)
    ecfg = EngineConfig(model_path=str(path), use_dummy=False, block_size=16, gpu_mem_utilization=0.9,
                        num_cpu_blocks=cpu_blocks, max_seqs_in_block_table=max_seqs, max_blocks_per_seq=-(-max_len // 16),
                        max_batch_size=max_seqs, max_tokens_in_batch=1024, dtype=dtype, use_hip_graph=graph)
    model = build_model(ecfg)
    model.load_weights()
    model.init_kvcache_and_swap(num_blocks)
    return model


def row_err(got, want):
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt().clamp_min(1e-9)


def rel_err(got, want):
    return float(row_err(got, want).max())


def close(got, want, dtype, tol=None):
    """fp32 runs are held to the tolerance everywhere; 16-bit runs at the median and at most positions (rounding moves a
    router's close calls, and a token that goes to another expert differs by more than rounding)."""
    e = row_err(got, want)
    if dtype in ("float32", torch.float32):
        return float(e.max()) < (tol or F32_TOL)
    tol = tol or BF16_TOL
    return float(e.median()) < tol / 2 and float((e < tol).double().mean()) >= 0.75


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def entry(seq, toks, start, want=None):
    from swiftllm_amd.worker.batch_plan import StepEntry
    return StepEntry(seq, toks, start, tuple(range(len(toks))) if want is None else tuple(want))


def run_in_portions(model, seq, toks, sizes):
    """Feed toks to sequence `seq` in portions of the given sizes (the last size repeats); -> logits of every position."""
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[min(i, len(sizes) - 1)], len(toks) - at)
        out.append(model.step([entry(seq, toks[at:at + n], at)]).clone())
        at += n
        i += 1
    return torch.cat(out)


# ---- the streams -------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("S,width,groups,n", [(1, 48, 1, 5), (2, 160, 2, 9), (3, 50, 5, 4), (4, 1024, 4, 7), (2, 36, 6, 3),
                                              (5, 40, 1, 3), (8, 2052, 3, 4), (3, 33, 3, 6), (2, 4096, 1, 2), (4, 4100, 10, 2),
                                              (13, 44, 2, 3)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
def test_streams_step(S, width, groups, n, dtype):
    from swiftllm_amd.worker.kernels.hyper_stream import StreamWeights, embed_streams, hyper_step
    g = torch.Generator().manual_seed(S * width)
    X, y, y2 = torch.randn(n, S, width, generator=g), torch.randn(n, width, generator=g), torch.randn(n, width, generator=g)
    mix, out, read = torch.randn(S, S, generator=g), torch.randn(S, generator=g), torch.randn(S, generator=g)
    w, bias = 1 + 0.2 * torch.randn(width, generator=g), torch.randn(width, generator=g)
    X[:, :, :width // groups] *= 30.0          # (the first part of the norm is much larger than the others)
    y, y2 = y.to(dtype), y2.to(dtype)
    d = lambda t: t.double()        # noqa: E731
    Xs = d(X).transpose(0, 1)
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    sw = StreamWeights(read.cuda(), mix.cuda(), out.cuda())
    for second, with_bias in ((True, True), (False, False), (True, False)):
        total = d(y) + (d(y2) if second else 0) + (d(bias) if with_bias else 0)
        new = O.hyper_step(Xs, total, d(mix), d(out))
        h_want = O.group_norm(sum(d(read)[s] * new[s] for s in range(S)), d(w), groups, EPS)
        x = X.cuda().clone()
        h = hyper_step(x, y.cuda(), sw, y2.cuda() if second else None, bias.cuda() if with_bias else None, read.cuda(), w.cuda(),
                       groups, EPS)
        assert (x.cpu().double() - new.transpose(0, 1)).abs().max() < 1e-5 * float(new.abs().max())
        assert h.dtype == dtype and (h.cpu().double() - h_want).abs().max() < tol * float(h_want.abs().max())
        x2 = X.cuda().clone()
        assert hyper_step(x2, y.cuda(), sw, y2.cuda() if second else None, bias.cuda() if with_bias else None) is None
        assert torch.equal(x2, x)
    # a result in three rows per token (a token's experts), summed
    y3 = torch.randn(n, 3, width, generator=g).to(dtype)
    new = O.hyper_step(Xs, d(y3).sum(1) + d(y2), d(mix), d(out))
    x = X.cuda().clone()
    hyper_step(x, y3.view(n * 3, width).cuda(), sw, y2.cuda())
    assert (x.cpu().double() - new.transpose(0, 1)).abs().max() < 1e-5 * float(new.abs().max())
    # the norm alone: of all rows with a weighted sum, of some rows of the plain sum (the model's last norm); nothing is written
    x = X.cuda().clone()
    h = hyper_step(x, read=read.cuda(), norm=w.cuda(), groups=groups, eps=EPS, out_dtype=dtype)
    want = O.group_norm(sum(d(read)[s] * Xs[s] for s in range(S)), d(w), groups, EPS)
    assert (h.cpu().double() - want).abs().max() < tol * float(want.abs().max())
    rows = torch.tensor([n - 1, 0, 1], dtype=torch.int32)
    h = hyper_step(x, norm=w.cuda(), groups=groups, eps=EPS, out_dtype=dtype, row_idx=rows.cuda())
    want = O.group_norm(Xs.sum(0)[rows.long()], d(w), groups, EPS)
    assert (h.cpu().double() - want).abs().max() < tol * float(want.abs().max())
    assert torch.equal(x.cpu(), X)
    emb = torch.randn(11, width, generator=g).to(dtype)
    ids = torch.tensor([3, 10, 0, 3], dtype=torch.int32)
    assert torch.equal(embed_streams(ids.cuda(), emb.cuda(), S).cpu(), emb[ids.long()].float()[:, None, :].expand(4, S, width))


def test_a_plain_residual_is_one_stream_of_ones():
    from swiftllm_amd.worker.kernels.hyper_stream import StreamWeights, hyper_step
    g = torch.Generator().manual_seed(0)
    x, y, w = torch.randn(3, 1, 64, generator=g), torch.randn(3, 64, generator=g), torch.ones(64)
    sw = StreamWeights.plain(torch.device("cuda"))
    dev = x.cuda().clone()
    hyper_step(dev, y.cuda(), sw, read=sw.read, norm=w.cuda(), eps=EPS)
    assert torch.allclose(dev.cpu()[:, 0], x[:, 0] + y)


# ---- rotation, norm and store ------------------------------------------------------------------------------------------------
class Pages:
    """A pool of pages full of finite garbage and a block table in which another sequence owns the first blocks."""

    def __init__(self, k_elems, v_elems, dtype, num_blocks=40, off=24, max_blocks=None):
        from swiftllm_amd.worker.block_manager import BlockManager
        from swiftllm_amd.worker.kernels.window_attn import PoolSlice
        self.mgr = BlockManager("GPU", num_blocks, 3, max_blocks or num_blocks, 16, "cuda")
        self.mgr.allocate_blocks_for_seqs([1], [37])
        self.slice = PoolSlice(off, off + k_elems * 16)
        self.k_elems, self.v_elems = k_elems, v_elems
        self.pool = torch.full((num_blocks, off + (k_elems + v_elems) * 16 + 16), 3e4, dtype=dtype, device="cuda")

    def rows(self, seq, at, n):
        self.mgr.allocate_blocks_for_seqs([seq], [at + n])
        pos = torch.arange(at, at + n, dtype=torch.int32, device="cuda")
        return torch.full((n,), seq, dtype=torch.int32, device="cuda"), pos

    def token(self, seq, pos, G, kd, vd):
        """-> (key rows [G, kd], value rows [G, vd]) of one position as the pool holds them"""
        page = self.pool[int(self.mgr.block_table[seq][pos // 16])].cpu().double()
        k0, v0, o = self.slice.k_offset, self.slice.v_offset, pos % 16
        return page[k0:k0 + G * kd * 16].view(G, 16, kd)[:, o], page[v0:v0 + G * vd * 16].view(G, vd, 16)[:, :, o]


ROPE_CASES = [  # H, G, d, rot dims, half, key row, value row, interpolated
    (4, 2, 64, 16, True, 64, 64, False), (6, 3, 80, 32, True, 96, 96, True), (3, 1, 10, 6, True, 10, 10, False),
    (5, 5, 24, 24, True, 32, 32, False), (2, 1, 128, 128, True, 128, 128, True), (4, 4, 16, 0, True, 32, 32, False),
    (3, 3, 48, 16, False, 48, 48, False), (7, 1, 12, 12, False, 15, 13, True), (2, 2, 200, 64, True, 288, 256, False),
    (9, 3, 8, 8, True, 8, 8, False), (1, 1, 112, 48, True, 128, 128, False)]


@pytest.mark.parametrize("H,G,d,rd,half,kd,vd,scaled", ROPE_CASES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_norm_rotation_and_store_with_keys_as_values(H, G, d, rd, half, kd, vd, scaled, dtype):
    from swiftllm_amd.model_config import RotaryConfig
    from swiftllm_amd.worker.kernels.rope_kv import qk_norm_rope_and_store_kv, rotary_frequencies
    g = torch.Generator().manual_seed(d + H)
    n, extra, start = 21, 5, 20030
    rot_cfg = {"dims": rd, "base": 777.0}
    if scaled:
        rot_cfg["scaling"] = {"factor": 4.0, "original": 300, "fast": 20.0, "slow": 2.0}
    rot = RotaryConfig(rot_cfg, d, half=half)
    stride = (H + G) * d + extra
    stride += -stride % 8
    rows = torch.randn(n, stride, generator=g).to(dtype)
    qb, kb = torch.randn(H * d, generator=g), torch.randn(G * d, generator=g)
    qw, kw, temp = 1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g), 0.5 + torch.rand(H, generator=g)
    pages = Pages(G * kd, G * vd, dtype, num_blocks=1300, max_blocks=1290)
    seq, pos = pages.rows(2, start, n)
    freq = rotary_frequencies(rot, torch.device("cuda"))
    q = qk_norm_rope_and_store_kv(rows.cuda(), qb.cuda(), kb.cuda(), qw.cuda(), kw.cuda(), temp.cuda(), freq, rot, pages.pool,
                                  pages.slice, pages.mgr.block_table, seq, pos, H, G, 0, d, d, EPS, kd, vd)
    r = rows.double()
    qr, kr = r[:, :H * d].view(n, H, d) + qb.double().view(H, d), r[:, H * d:(H + G) * d].view(n, G, d) + kb.double().view(G, d)

    def turn(x):
        if rd and not half:     # interleaved pairs, from the halves: gather evens and odds, turn, scatter back
            perm = torch.tensor(list(range(0, rd, 2)) + list(range(1, rd, 2)) + list(range(rd, d)))
            y = torch.empty_like(x)
            y[..., perm] = O.rotate_half(x[..., perm], pos.cpu(), rot_cfg)
            return y
        return O.rotate_half(x, pos.cpu(), rot_cfg)
    q_want = turn(O.rms(qr, EPS) * qw.double()) * temp.double()[:, None]
    k_want = turn(O.rms(kr, EPS) * kw.double())
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    got = q.cpu().double().view(n, H, kd)
    assert (got[..., :d] - q_want).abs().max() < tol and bool((got[..., d:] == 0).all())
    for t in (0, 1, 2, 15, 20):
        k, v = pages.token(2, start + t, G, kd, vd)
        assert (k[:, :d] - k_want[t]).abs().max() < tol and bool((k[:, d:] == 0).all())
        assert (v[:, :d] - kr[t]).abs().max() < tol and bool((v[:, d:] == 0).all())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_store_with_value_columns_and_without_norm(dtype):
    """The same kernel for projections that have values of their own, no norm, no biases and no factor."""
    from swiftllm_amd.model_config import RotaryConfig
    from swiftllm_amd.worker.kernels.rope_kv import qk_norm_rope_and_store_kv, rotary_frequencies
    for H, G, d, e, kd, vd, rd in ((4, 2, 32, 24, 32, 24, 16), (3, 3, 10, 6, 16, 9, 4)):
        g = torch.Generator().manual_seed(d)
        n = 19
        rows = torch.randn(n, (H + G) * d + G * e, generator=g).to(dtype)
        rot = RotaryConfig({"dims": rd, "base": 50.0}, d, half=True)
        pages = Pages(G * kd, G * vd, dtype)
        seq, pos = pages.rows(0, 7, n)
        q = qk_norm_rope_and_store_kv(rows.cuda(), None, None, None, None, None, rotary_frequencies(rot, torch.device("cuda")), rot,
                                      pages.pool, pages.slice, pages.mgr.block_table, seq, pos, H, G, G, d, e, EPS, kd, vd)
        r = rows.double()
        qk = O.rotate_half(r[:, :(H + G) * d].view(n, H + G, d), pos.cpu(), {"dims": rd, "base": 50.0})
        tol = 1e-5 if dtype == torch.float32 else 2e-2
        assert (q.cpu().double().view(n, H, kd)[..., :d] - qk[:, :H]).abs().max() < tol
        for t in range(n):
            k, v = pages.token(0, 7 + t, G, kd, vd)
            assert (k[:, :d] - qk[t, H:]).abs().max() < tol and bool((k[:, d:] == 0).all())
            assert torch.equal(v[:, :e].reshape(-1), r[t, (H + G) * d:]) and bool((v[:, e:] == 0).all())


# ---- mixers alone ------------------------------------------------------------------------------------------------------------
class MixerBench:
    """One mixer of the product with weights loaded by the product's loader, on a hand-made pool and hand-made state slots that
    hold garbage; `pad`: the pool's rows as the worker would choose them for the dtype."""

    def __init__(self, layer, W, dtype, width=64, num_blocks=48, pad=True):
        from swiftllm_amd.model_config import RokevikModelConfig
        from swiftllm_amd.worker.kernels.window_attn import served_row_sizes
        from swiftllm_amd.worker.layers import rokevik_layer as L
        from swiftllm_amd.worker.rokevik_weight import RokevikLayerWeight
        self.cfg = RokevikModelConfig(O.make_config(layers=[layer], width=width, loop=None, groups=1))
        self.dtype = dtype
        lcfg = self.cfg.layers[0]
        mx = lcfg.mixer
        lw = RokevikLayerWeight(0)
        lw.load(lambda name, shape: W[name].clone(), self.cfg, lcfg, dtype, torch.device("cuda"))
        self.y_bias = None
        if mx.kind == "mingru":
            self.pages = Pages(8, 8, dtype, num_blocks)
            self.op = L.RokevikMinGru(lcfg, lw, False, 4)
            self.slots = torch.full((3, mx.width + 9), float("nan"), device="cuda")
            return
        need = (mx.k_size, mx.v_size) if mx.kind == "latent_attention" else (mx.head_dim, mx.value_dim)
        sizes = served_row_sizes(*need, dtype) if pad else need
        self.pages = Pages(mx.num_kv_heads * sizes[0], mx.num_kv_heads * sizes[1], dtype, num_blocks)
        kind = L.RokevikAttention if mx.kind == "attention" else L.RokevikLatentAttention
        self.op = kind(lcfg, lw, self.cfg.norm_eps, False, self.pages.slice, 512, sizes)
        self.slots = None
        if self.op.y_bias is not None:
            self.y_bias = self.op.y_bias.cpu().double()

    def context(self, parts, tiled):
        """parts: (sequence, start, count) of every portion of the step."""
        from swiftllm_amd.worker.batch_plan import StepEntry, plan_step
        from swiftllm_amd.worker.kernels.rms_stream import StateRef
        from swiftllm_amd.worker.layers.lorulix_layer import StepContext
        plan = plan_step([StepEntry(s, [0] * c, at) for s, at, c in parts])
        for s, at, c in parts:
            self.pages.mgr.allocate_blocks_for_seqs([s], [at + c])
        plan.tok_state = torch.tensor([2 * s for s, at, c in parts for _ in range(c)]).numpy()
        dev = {name: torch.from_numpy(getattr(plan, name).astype("int32")).cuda() for name in plan.SEGMENTS}
        st = None
        if self.slots is not None:
            st = StateRef(self.slots, dev["tok_pos"], dev["tok_start"], dev["tok_state"], dev["tok_seq"], dev["seq_row0"],
                          dev["seq_cnt"])
        return StepContext(self.pages.pool, self.pages.mgr.block_table, dev["tok_seq"], dev["tok_pos"],
                           (dev["tile_row0"], dev["tile_cnt"]) if tiled else None, st,
                           (dev["chunk_row0"], dev["chunk_cnt"], dev["seq_chunk0"]))

    def run(self, h, portions, tiled=True, seq=2):
        """-> the mixer's output of every token of one sequence, fed in the given portions (the last size repeats)."""
        n, out, at, i = h.shape[0], [], 0, 0
        while at < n:
            c = min(portions[min(i, len(portions) - 1)], n - at)
            y, _ = self.op.forward(h[at:at + c].to(self.dtype).cuda(), self.context([(seq, at, c)], tiled))
            out.append(y.cpu().double())
            at += c
            i += 1
        y = torch.cat(out)
        return y if self.y_bias is None else y + self.y_bias

    def run_together(self, hs, steps, tiled=True):
        """hs: the inputs of sequences 0, 2 (…); steps: per step the tokens each brings (0: sits out)."""
        seqs = [0, 2][:len(hs)]
        at, got = [0] * len(hs), [[] for _ in hs]
        for counts in steps:
            parts = [(seqs[i], at[i], c) for i, c in enumerate(counts) if c]
            rows = torch.cat([hs[i][at[i]:at[i] + c] for i, c in enumerate(counts) if c])
            y, _ = self.op.forward(rows.to(self.dtype).cuda(), self.context(parts, tiled))
            o = 0
            for i, c in enumerate(counts):
                got[i].append(y[o:o + c].cpu().double())
                o += c
                at[i] += c
        return [torch.cat(g) + (0 if self.y_bias is None else self.y_bias) for g in got]


def one_layer(layer, seed, width=64):
    cfg = O.make_config(layers=[layer], width=width, loop=None, groups=1)
    return O.random_weights(cfg, seed)


def mixer_tol(dtype, want):
    return (2e-4 if dtype == torch.float32 else 4e-2) * max(1.0, float(want.abs().max()))


def check_mixer(layer, n, width=64, dtype=torch.float32, cuts=((1000,), (5, 1, 2, 30, 2), (1,)), tiled=True, pad=True, seed=0):
    W = one_layer(layer, seed + n, width)
    if dtype != torch.float32:
        W = {k: v.to(dtype).float() for k, v in W.items()}
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(n)).to(dtype).float()
    want = O.MIXERS[layer["type"]](h.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    for portions in cuts:
        got = MixerBench(layer, W, dtype, width, pad=pad).run(h, portions, tiled)
        assert (got - want).abs().max() < mixer_tol(dtype, want), portions


@pytest.mark.parametrize("H,G,d,rd,cap,n", [(4, 2, 16, 8, 20.0, 150), (3, 1, 10, 10, 3.0, 70), (5, 5, 24, 0, None, 33),
                                            (6, 2, 12, 4, 45.0, 1), (9, 3, 48, 16, 5.0, 40), (1, 1, 136, 32, 2.0, 20)])
def test_attention_alone(H, G, d, rd, cap, n):
    check_mixer(O.attention_layer(heads=H, kv_heads=G, dim=d, rot_dims=rd, softcap=cap, scale=0.37, mlp=None), n)


@pytest.mark.parametrize("H,G,d,rd,cap,n", [(4, 2, 64, 16, 20.0, 150), (6, 3, 80, 32, 8.0, 90), (8, 2, 32, 32, None, 70),
                                            (4, 4, 16, 8, 5.0, 50), (3, 1, 128, 64, 30.0, 80), (10, 5, 112, 16, 10.0, 40)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
def test_attention_on_the_matrix_cores(H, G, d, rd, cap, n, dtype):
    layer = O.attention_layer(heads=H, kv_heads=G, dim=d, rot_dims=rd, softcap=cap, mlp=None)
    check_mixer(layer, n, 128, dtype, cuts=((17, 1, 2, 40),))
    check_mixer(layer, n, 128, dtype, cuts=((17, 1, 2, 40),), tiled=False, pad=False)


@pytest.mark.parametrize("H,d,dr,e,r,win,n", [(3, 16, 8, 24, 32, 24, 150), (5, 8, 4, 8, 12, 1, 40), (1, 24, 16, 40, 20, None, 33),
                                              (6, 4, 2, 6, 7, 16, 45), (2, 16, 16, 16, 16, 33, 1), (4, 12, 6, 10, 18, 100, 130)])
def test_latent_attention_alone(H, d, dr, e, r, win, n):
    check_mixer(O.latent_layer(heads=H, dim=d, rot_dim=dr, vdim=e, kv_rank=r, window=win, scale=0.3, mlp=None), n)
    check_mixer(O.latent_layer(heads=H, dim=d, rot_dim=dr, vdim=e, kv_rank=r, window=win, factor=None, mlp=None), n, seed=1)


@pytest.mark.parametrize("H,d,dr,e,r,win,n", [(7, 32, 16, 48, 120, 37, 150), (4, 64, 32, 64, 96, None, 90),
                                              (17, 16, 16, 32, 48, 7, 64), (2, 64, 8, 128, 176, 50, 70), (40, 8, 32, 16, 32, 20, 40),
                                              (5, 24, 24, 40, 60, 33, 80), (6, 32, 64, 32, 512, 48, 60)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
def test_latent_attention_on_the_matrix_cores(H, d, dr, e, r, win, n, dtype):
    layer = O.latent_layer(heads=H, dim=d, rot_dim=dr, vdim=e, kv_rank=r, window=win, mlp=None)
    check_mixer(layer, n, 128, dtype, cuts=((17, 1, 2, 40), (1,)))
    check_mixer(layer, n, 128, dtype, cuts=((17, 1, 2, 40),), tiled=False, pad=False)


@pytest.mark.parametrize("tiled,dtype", [(False, torch.float32), (True, torch.bfloat16)])
@pytest.mark.parametrize("n,target", [(400, 3), (400, 15), (400, 16), (400, 0)])
def test_a_far_key_among_hundreds_and_at_page_borders(tiled, dtype, n, target):
    """The query projection turns the askers' direction into the key of the answering direction (no rotation), which only token
    `target` has: one score stands out among hundreds, for askers near and hundreds of positions away, in prompts and decoded."""
    d = 32
    layer = O.attention_layer(heads=2, kv_heads=1, dim=d, rot_dims=0, scale=0.5, softcap=40.0, mlp=None)
    W = one_layer(layer, 7)
    g = torch.Generator().manual_seed(n)
    ask, answer = torch.randn(64, generator=g), torch.randn(64, generator=g)
    turned = W["l0.mix.k"] @ torch.outer(answer, ask) / (ask @ ask)
    W["l0.mix.q"] = turned.repeat(2, 1) + 0.02 * W["l0.mix.q"]
    W["l0.mix.q.b"] *= 0.01
    W["l0.mix.k.b"] *= 0.01
    W["l0.mix.q.norm"], W["l0.mix.k.norm"], W["l0.mix.temp"] = torch.ones(d), torch.ones(d), torch.tensor([1.0, 1.25])
    h = 0.3 * torch.randn(n, 64, generator=g)
    h[target] = answer
    askers = [t for t in range(target + 1, n) if t % 2 == 0]
    h[askers] += ask
    W = {k: v.to(dtype).float() for k, v in W.items()}
    h = h.to(dtype).float()
    want = O.attention_mixer(h.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    hidden = h.clone()
    hidden[target] = h[target + 1]
    other = O.attention_mixer(hidden.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    assert (other[askers] - want[askers]).abs().max(dim=-1).values.min() > 4 * mixer_tol(dtype, want)
    for portions in ((n - 30, 1), (97, 2, 1, 16), (n,)):
        got = MixerBench(layer, W, dtype).run(h, portions, tiled)
        assert (got - want).abs().max() < mixer_tol(dtype, want), portions


@pytest.mark.parametrize("tiled,dtype", [(False, torch.float32), (True, torch.bfloat16)])
@pytest.mark.parametrize("window", [1, 2, 16, 17, 31, 45])
def test_keys_just_inside_and_just_outside_the_window(tiled, dtype, window):
    """Marked tokens whose latent answers every query: a query sees the mark when it is window - 1 back and not when it is
    window back, at every place of a page, in prompts, portions and decoding."""
    H, d, dr, r, n = 2, 32, 16, 32, 180
    layer = O.latent_layer(heads=H, dim=d, rot_dim=dr, vdim=24, kv_rank=r, window=window, scale=0.05, factor=None, mlp=None)
    W = one_layer(layer, 11)
    g = torch.Generator().manual_seed(window)
    u, m = torch.randn(64, generator=g), torch.randn(64, generator=g)
    u, m = u / u.norm() * 8, m / m.norm() * 8
    h = u + 0.3 * torch.randn(n, 64, generator=g)           # every token asks
    marks = [5, 47, 48, 111, 150]
    for t in marks:
        h[t] = h[t] + 2 * m                                   # (and the marked ones answer)
    c_u, _ = O.latent_rows(u[None].double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    c_m, _ = O.latent_rows((u + 2 * m)[None].double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    a = (c_m - c_u)[0].float()
    a = a - c_u[0].float() * (a @ c_u[0].float()) / (c_u[0].float() @ c_u[0].float())
    q = (W["l0.mix.q"] @ u).view(H, d + dr)[:, :d]
    uk = W["l0.mix.uk"].view(H, d, r)
    for hd in range(H):
        uk[hd] += 9.0 / 0.05 * torch.outer(q[hd] / q[hd].norm() ** 2, a / (a @ c_m[0].float()))
    W["l0.mix.uk"] = uk.reshape(H * d, r).contiguous()
    W = {k: v.to(dtype).float() for k, v in W.items()}
    h = h.to(dtype).float()
    want = O.latent_mixer(h.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    for portions in ((n - 40, 1), (37, 2, 1, 16, 2), (n,)):
        got = MixerBench(layer, W, dtype).run(h, portions, tiled)
        assert (got - want).abs().max() < mixer_tol(dtype, want), portions
    # the case is sharp: one token more or less in the window would show at the marks' edges
    for other_window, at in ((window + 1, [t + window for t in marks if t + window < n]),
                             (window - 1, [t + window - 1 for t in marks if t + window - 1 < n])):
        if other_window < 1:
            continue
        mx = dict(layer["mixer"], mask={"size": other_window})
        other = O.latent_mixer(h.double(), f64(W), "l0.mix.", mx, EPS)
        assert (other[at] - want[at]).abs().max() > 5 * mixer_tol(dtype, want)


@pytest.mark.parametrize("width,n", [(56, 150), (33, 70), (288, 100), (1, 40), (1030, 64), (48, 1), (64, 700)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_min_gru_alone(width, n, dtype):
    """Slots hold NaN before a sequence starts; long portions run in parallel over their chunks, short ones walk."""
    cuts = ((1000,), (33, 2, 1, 64, 100), (2,)) if n <= 150 else ((1000,), (333, 2, 65))
    check_mixer(O.min_gru_layer(width=width, mlp=None), n, 64, dtype, cuts=cuts)


def test_min_gru_remembers_the_first_token_and_forgets_at_once():
    """Channels whose gate is nearly shut carry the first token's candidate to the end; channels whose gate is wide open hold the
    last token only — whole, in portions and decoded."""
    layer = O.min_gru_layer(width=64, mlp=None)
    W = one_layer(layer, 3)
    W["l0.mix.z"] = 0.01 * W["l0.mix.z"]
    W["l0.mix.z.b"] = torch.where(torch.arange(64) % 2 == 0, -9.0, 9.0)
    g = torch.Generator().manual_seed(1)
    h = torch.randn(300, 64, generator=g)
    h[0] *= 300.0
    want = O.min_gru_mixer(h.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    lost = h.clone()
    lost[0] = h[1]
    other = O.min_gru_mixer(lost.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
    assert (other[-1] - want[-1]).abs().max() > 20 * mixer_tol(torch.float32, want[1:])
    for portions in ((1000,), (1, 64, 1), (100, 2, 33), (1,)):
        got = MixerBench(layer, W, torch.float32).run(h, portions)
        assert (got[1:] - want[1:]).abs().max() < mixer_tol(torch.float32, want[1:]), portions


@pytest.mark.parametrize("layer", [O.attention_layer(mlp=None), O.latent_layer(mlp=None), O.min_gru_layer(width=40, mlp=None)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_two_sequences_of_a_step_do_not_meet(layer, dtype):
    W = {k: v.to(dtype).float() for k, v in one_layer(layer, 21).items()}
    g = torch.Generator().manual_seed(2)
    hs = [torch.randn(n, 64, generator=g).to(dtype).float() for n in (130, 77)]
    got = MixerBench(layer, W, dtype).run_together(hs, [(70, 1), (1, 40), (0, 3), (2, 33), (57, 0)])
    for h, y in zip(hs, got):
        want = O.MIXERS[layer["type"]](h.double(), f64(W), "l0.mix.", layer["mixer"], EPS)
        assert (y - want).abs().max() < mixer_tol(dtype, want)


# ---- experts -----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("experts,top,ff,shared,width,n", [(5, 2, 24, 16, 48, 9), (7, 1, 48, 96, 64, 200), (3, 3, 16, 0, 64, 40),
                                                           (6, 2, 12, 20, 44, 70), (16, 4, 32, 32, 128, 3), (1, 1, 8, 8, 32, 17),
                                                           (9, 1, 80, 112, 160, 1)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_experts_with_weighted_inputs(experts, top, ff, shared, width, n, dtype):
    from swiftllm_amd.model_config import RokevikModelConfig
    from swiftllm_amd.worker.layers.rokevik_layer import RokevikFeedForward
    from swiftllm_amd.worker.rokevik_weight import RokevikLayerWeight
    layer = O.min_gru_layer(width=8, mlp=O.moe(ff=ff, experts=experts, top=top, shared=shared))
    cfg = O.make_config(layers=[layer], width=width, loop=None, groups=1)
    W = O.random_weights(cfg, 4)
    mcfg = RokevikModelConfig(cfg)
    lw = RokevikLayerWeight(0)
    lw.load(lambda name, shape: W[name].clone(), mcfg, mcfg.layers[0], dtype, torch.device("cuda"))
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(5)).to(dtype)
    a, b = RokevikFeedForward(mcfg.layers[0], lw, False).forward(h.cuda(), None)
    got = a.float().view(n, -1, width).sum(1) + (b.float() if b is not None else 0)      # (decode-sized: a row per expert)
    want = O.moe_ff(h.double(), f64(W), "l0.mlp.", layer["mlp"])
    e = (got.cpu().double() - want).abs().max(dim=-1).values / want.abs().max()
    if dtype == torch.float32:
        assert float(e.max()) < 1e-5
    else:
        assert float(e.median()) < 2e-2 and float((e < 4e-2).double().mean()) > 0.9
    assert (b is None) == (shared == 0)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
def test_gated_unit_with_row_weights(dtype):
    from swiftllm_amd.worker.kernels.moe import ACT_CLAMPED, ACT_SILU_UP_FIRST, gated_unit
    g = torch.Generator().manual_seed(3)
    for rows, ff in ((7, 40), (5, 33), (300, 8)):
        gu, w = torch.randn(rows, 2 * ff, generator=g).to(dtype), torch.rand(rows, generator=g) + 0.1
        for in_w in (w, None):
            z = gu.double() * (in_w.double()[:, None] if in_w is not None else 1)
            want = O.silu(z[:, :ff]) * z[:, ff:]
            got = gated_unit(gu.cuda(), ff, in_w=in_w.cuda() if in_w is not None else None)
            assert (got.cpu().double() - want).abs().max() < (1e-5 if dtype == torch.float32 else 4e-2)
        got = gated_unit(gu.cuda(), ff, ACT_SILU_UP_FIRST)
        z = gu.double()
        assert (got.cpu().double() - O.silu(z[:, ff:]) * z[:, :ff]).abs().max() < (1e-5 if dtype == torch.float32 else 4e-2)
        a, b = z[:, :ff].clamp(max=1.5), z[:, ff:].clamp(-1.5, 1.5)
        got = gated_unit(gu.cuda(), ff, ACT_CLAMPED, 1.5)
        assert (got.cpu().double() - a * torch.sigmoid(1.702 * a) * (b + 1)).abs().max() < (1e-5 if dtype == torch.float32 else 4e-2)


@pytest.mark.parametrize("n,width,ff", [(1, 128, 64), (32, 256, 96), (50, 128, 64), (200, 128, 32), (7, 100, 30)])
@pytest.mark.parametrize("packed", [True, False])
def test_fused_silu_unit(n, width, ff, packed):
    """The one-launch form of the shared expert's first half, the medium and large forms, and the shapes none of them serves."""
    from swiftllm_amd.worker.kernels.linear import pack_weight, packable
    from swiftllm_amd.worker.layers.kekapel_layer import _silu_unit
    g = torch.Generator().manual_seed(n)
    h = torch.randn(n, width, generator=g).bfloat16()
    w = (torch.randn(2 * ff, width, generator=g) / width ** 0.5).bfloat16().cuda()
    if packed and packable(w):
        pack_weight(w)
    z = h.double() @ w.cpu().double().T
    want = z[:, :ff] * O.silu(z[:, ff:])
    assert (_silu_unit(h.cuda(), w, True).cpu().double() - want).abs().max() < 1e-2 * max(1.0, float(want.abs().max()))
    got = _silu_unit(h.float().cuda(), w.float(), False)
    assert (got.cpu().double() - want).abs().max() < 1e-4


def test_capped_logits_and_fp32_argmax():
    from swiftllm_amd.worker.kernels.sampling import argmax_rows, softcap_logits
    g = torch.Generator().manual_seed(6)
    for dtype in (torch.float32, torch.bfloat16):
        x = (30 * torch.randn(5, 1024, generator=g)).to(dtype)
        got = softcap_logits(x.cuda(), 15.0)
        assert got.dtype == torch.float32
        assert (got.cpu().double() - 15 * torch.tanh(x.double() / 15)).abs().max() < 1e-5
    y = torch.randn(9, 2048, generator=g)
    y[3, 17] = y[3, 1999] = 50.0                    # a tie: the lowest index
    y[4, 2047], y[5, 0] = 60.0, 60.0
    assert argmax_rows(y.cuda()).tolist() == [int(r.argmax()) if i != 3 else 17 for i, r in enumerate(y)]
    assert argmax_rows(y.cuda()[:, :61]).tolist() == y[:, :61].argmax(1).tolist()


# ---- the whole model ---------------------------------------------------------------------------------------------------------
@pytest.fixture(scope="module")
def default_case():
    cfg = O.make_config()
    W = O.random_weights(cfg, seed=3)
    toks = tokens_for(cfg, 90, 1)
    streams = []
    logits = O.forward(cfg, f64(W), toks, streams)
    return cfg, W, toks, logits, streams


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_logits_and_every_layer(tmp_path, default_case, dtype):
    cfg, W, toks, want, streams = default_case
    model = make_model(tmp_path / "m", cfg, W, dtype)
    assert type(model).__name__ == "RokevikModel"
    model.layer_tap = []
    got = model.step([entry(0, toks, 0)])
    assert len(model.layer_tap) == len(streams) == 6            # (four layers, two of them run twice)
    for x, ref in zip(model.layer_tap, streams):
        if dtype == "float32":
            assert (x.cpu().double() - ref).abs().max() < 3e-4
        else:
            assert float((x.cpu().double() - ref).abs().median()) < 0.1
    assert close(got, want, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decoding_and_portions_match_the_whole_prompt(tmp_path, default_case, dtype):
    cfg, W, toks, want, _ = default_case
    model = make_model(tmp_path / "m", cfg, W, dtype)
    assert close(run_in_portions(model, 0, toks, [1]), want, dtype)                     # token by token from the first
    assert close(run_in_portions(model, 1, toks, [2]), want, dtype)                     # pairs
    assert close(run_in_portions(model, 2, toks, [3, 2, 16, 1, 31, 2, 17, 1]), want, dtype)
    model.free_seqs_resources([0, 1, 2])
    assert close(run_in_portions(model, 0, toks, [58, 1]), want, dtype)                 # a prompt, then decoding
    if dtype == "bfloat16":     # the same positions whole and cut: the cut must not show beyond rounding
        whole = model.step([entry(1, toks, 0)])
        model.free_seqs_resources([1])
        parts = run_in_portions(model, 1, toks, [15, 2, 1, 33])
        assert float(row_err(parts, whole.float()).median()) < BF16_TOL / 2


def test_decode_graph_replays_match_eager_steps(tmp_path, default_case):
    cfg, W, toks, want, _ = default_case
    model = make_model(tmp_path / "m", cfg, W, "float32", graph=True)
    other = tokens_for(cfg, 70, 2)
    want_other = O.forward(cfg, f64(W), other)
    a = [model.step([entry(0, toks[:30], 0), entry(1, other[:11], 0)])]
    got0, got1 = [a[0][:30]], [a[0][30:]]
    for i in range(40):     # two sequences decode together: one captured graph, replayed with other positions and slots
        lg = model.step([entry(0, toks[30 + i:31 + i], 30 + i), entry(1, other[11 + i:12 + i], 11 + i)]).clone()
        got0.append(lg[:1])
        got1.append(lg[1:])
        torch.cuda.synchronize()
    assert model.graph_captures == 1
    assert rel_err(torch.cat(got0), want[:70]) < F32_TOL
    assert rel_err(torch.cat(got1), want_other[:51]) < F32_TOL


def test_decode_graph_replays_in_bfloat16(tmp_path):
    """Matrix-core shapes: the captured step against eager steps of the same model, replay after replay."""
    layers = [O.attention_layer(heads=4, kv_heads=2, dim=64, rot_dims=16, mlp=O.moe(32, 8, 2, 32)),
              O.latent_layer(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, window=20, mlp=O.moe(32, 8, 2, 32)),
              O.min_gru_layer(width=128, mlp=O.moe(32, 8, 1, 32))]
    cfg = O.make_config(layers=layers, width=128, groups=2, loop=(0, 3, 2), vocab=96)
    W = O.random_weights(cfg, 17)
    toks = [tokens_for(cfg, 60, 5), tokens_for(cfg, 44, 6), tokens_for(cfg, 35, 7)]
    runs = []
    for graph in (True, False):
        model = make_model(tmp_path / f"m{graph}", cfg, W, "bfloat16", graph=graph)
        model.step([entry(i, t[:20], 0, want=[]) for i, t in enumerate(toks)])
        runs.append([model.step([entry(i, t[20 + k:21 + k], 20 + k) for i, t in enumerate(toks)]).clone() for k in range(15)])
        torch.cuda.synchronize()
    assert all(torch.equal(a, b) for a, b in zip(*runs))


def _serve(model, reqs, cuts, rows_total):
    """Up to rows_total live requests, portions beside decoded tokens, requests that sit steps out; finished requests give
    their blocks, block-table rows and state slots to new ones. -> the logits of every request."""
    lens = [len(r) for r in reqs]
    got = [[] for _ in reqs]
    at, k = [0] * len(reqs), [0] * len(reqs)
    waiting, live, rows = list(range(len(reqs))), {}, list(range(rows_total - 1, -1, -1))
    steps = 0
    while waiting or live:
        while waiting and rows:
            live[waiting.pop(0)] = rows.pop()
        batch, ended = [], []
        for r, row in live.items():
            if (steps + r) % 4 == 3 and len(live) > 1:
                continue
            c = min(cuts[r][min(k[r], len(cuts[r]) - 1)], lens[r] - at[r])
            batch.append((r, entry(row, reqs[r][at[r]:at[r] + c], at[r])))
            at[r] += c
            k[r] += 1
        if batch:
            lg = model.step([e for _, e in batch]).clone()
            o = 0
            for r, e in batch:
                got[r].append(lg[o:o + len(e.tokens)])
                o += len(e.tokens)
                if at[r] == lens[r]:
                    ended.append(r)
        for r in ended:
            model.free_seqs_resources([live[r]])
            rows.append(live.pop(r))
        steps += 1
    return [torch.cat(g) for g in got]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batches_and_reused_blocks_and_slots(tmp_path, default_case, dtype):
    cfg, W, _, _, _ = default_case
    model = make_model(tmp_path / "m", cfg, W, dtype, num_blocks=20, max_seqs=4)
    lens = [70, 5, 33, 1, 98, 17, 2]
    reqs = [tokens_for(cfg, n, 50 + i) for i, n in enumerate(lens)]
    wants = [O.forward(cfg, f64(W), t) for t in reqs]
    got = _serve(model, reqs, [[9, 1, 1, 50, 2], [2, 1], [33], [1], [66, 1], [3, 2], [1]], 4)
    assert model.gpu_block_manager.num_free_blocks == 20 and model.state.num_free_slots == 4
    if dtype == "float32":
        for r in range(len(reqs)):
            assert rel_err(got[r], wants[r]) < F32_TOL, f"request {r}"
    else:
        assert close(torch.cat(got), torch.cat(wants), dtype)


def varied_config():
    """Sizes that a symmetric configuration would hide: one kv head, heads = kv heads, heads not a power of two, no rotation,
    rotation of the whole head, no cap, no interpolation, windows of one page and of one token, no window, a layer without
    feed-forward first, top = 1 and top = experts, no shared expert, a width that is no multiple of 8, five streams, a loop of
    the first layer alone, no logit cap."""
    layers = [O.min_gru_layer(width=37, mlp=None),
              O.attention_layer(heads=3, kv_heads=1, dim=12, rot_dims=12, softcap=None, scale=0.4, mlp=O.moe(12, 6, 1, 0)),
              O.latent_layer(heads=5, dim=6, rot_dim=4, vdim=14, kv_rank=18, window=16, factor=None, mlp=O.moe(20, 3, 3, 28)),
              O.attention_layer(heads=2, kv_heads=2, dim=20, rot_dims=0, softcap=4.0, mlp=None),
              O.latent_layer(heads=2, dim=10, rot_dim=10, vdim=6, kv_rank=9, window=1, base=90.0, factor=16.0, original=30, fast=4.0,
                             slow=0.5, mlp=O.moe(8, 9, 2, 8)),
              O.latent_layer(heads=1, dim=8, rot_dim=2, vdim=8, kv_rank=8, window=None, mlp=O.moe(8, 2, 1, 8))]
    return O.make_config(layers=layers, width=44, vocab=37, groups=11, streams=5, loop=(0, 1, 3), logit_softcap=None, eps=1e-3)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_other_sizes(tmp_path, dtype):
    cfg = varied_config()
    W = O.random_weights(cfg, seed=5)
    toks = tokens_for(cfg, 75, 6)
    streams = []
    want = O.forward(cfg, f64(W), toks, streams)
    model = make_model(tmp_path / "m", cfg, W, dtype)
    model.layer_tap = []
    got = model.step([entry(0, toks, 0)])
    if dtype == "float32":
        for x, ref in zip(model.layer_tap, streams):
            assert (x.cpu().double() - ref).abs().max() < 3e-4 * max(1.0, float(ref.abs().max()))
    model.layer_tap = None
    assert close(got, want, dtype)
    assert close(run_in_portions(model, 1, toks, [4, 1, 2, 17, 1]), want, dtype)


def test_a_model_without_streams_loop_or_attention(tmp_path):
    """The plain residual, no loop; and recurrent layers alone (no keys in the pool)."""
    for layers in (None, [O.min_gru_layer(width=24), O.min_gru_layer(width=40, mlp=None)]):
        cfg = O.make_config(layers=layers, streams=None, loop=None, groups=1)
        W = O.random_weights(cfg, 6)
        toks = tokens_for(cfg, 60, 8)
        want = O.forward(cfg, f64(W), toks)
        model = make_model(tmp_path / f"m{layers is None}", cfg, W, "float32")
        assert close(run_in_portions(model, 0, toks, [40, 2, 1]), want, "float32")
    cfg = O.make_config(layers=[O.attention_layer(), O.latent_layer()], streams=1, loop=None)
    W = O.random_weights(cfg, 7)
    toks = tokens_for(cfg, 40, 9)
    model = make_model(tmp_path / "one", cfg, W, "float32")
    assert model.state is None          # no recurrent layer: no slots
    assert close(run_in_portions(model, 0, toks, [30, 2, 1]), O.forward(cfg, f64(W), toks), "float32")


def random_config(rng):
    def mlp():
        if rng.random() < 0.2:
            return None
        experts = rng.randint(1, 6)
        return O.moe(ff=rng.choice([8, 16, 20]), experts=experts, top=rng.randint(1, experts), shared=rng.choice([0, 8, 24]))
    layers = []
    for _ in range(rng.randint(2, 5)):
        kind = rng.choice(["attention", "latent", "gru"])
        if kind == "attention":
            G, d = rng.choice([1, 2, 3]), rng.choice([8, 12, 16, 40])
            layers.append(O.attention_layer(heads=G * rng.choice([1, 2, 3]), kv_heads=G, dim=d,
                                            rot_dims=rng.choice([0, 4, 8, d]), softcap=rng.choice([None, 3.0, 30.0]), mlp=mlp()))
        elif kind == "latent":
            layers.append(O.latent_layer(heads=rng.choice([1, 2, 5]), dim=rng.choice([8, 20]), rot_dim=rng.choice([2, 8, 16]),
                                         vdim=rng.choice([8, 18]), kv_rank=rng.choice([8, 24, 30]),
                                         window=rng.choice([None, 3, 16, 20, 50]), factor=rng.choice([None, 2.0, 8.0]), mlp=mlp()))
        else:
            layers.append(O.min_gru_layer(width=rng.choice([16, 35, 64]), mlp=mlp()))
    n = len(layers)
    start = rng.randint(0, n - 1)
    loop = (start, rng.randint(start + 1, n), rng.randint(1, 3)) if rng.random() < 0.7 else None
    return O.make_config(layers=layers, width=rng.choice([24, 40, 60]), vocab=rng.choice([17, 50]), groups=rng.choice([1, 2, 4]),
                         streams=rng.choice([None, 1, 2, 4]), loop=loop, logit_softcap=rng.choice([None, 5.0, 30.0]))


@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6])
def test_random_configurations_in_a_mixed_batch(tmp_path, seed):
    rng = random.Random(seed)
    cfg = random_config(rng)
    W = O.random_weights(cfg, seed=seed)
    model = make_model(tmp_path / "m", cfg, W, "float32", num_blocks=18, max_seqs=3)
    lens = [rng.randint(1, 90) for _ in range(5)]
    reqs = [tokens_for(cfg, n, seed * 10 + i) for i, n in enumerate(lens)]
    wants = [O.forward(cfg, f64(W), t) for t in reqs]
    cuts = [[rng.choice([1, 2, 3, 16, 17, 40, 66]) for _ in range(4)] + [1] for _ in reqs]
    got = _serve(model, reqs, cuts, 3)
    assert model.gpu_block_manager.num_free_blocks == 18
    for r in range(len(reqs)):
        assert rel_err(got[r], wants[r]) < F32_TOL, f"request {r} of {cfg}"


def test_matrix_core_paths_in_the_model(tmp_path):
    """Sizes that the matrix-core attention serves as they are and padded, in bfloat16: whole, in portions and decoded."""
    layers = [O.attention_layer(heads=8, kv_heads=4, dim=64, rot_dims=32, mlp=O.moe(32, 8, 2, 64)),
              O.latent_layer(heads=6, dim=32, rot_dim=16, vdim=48, kv_rank=112, window=50, mlp=O.moe(32, 8, 1, 64)),
              O.attention_layer(heads=3, kv_heads=1, dim=80, rot_dims=16, mlp=O.moe(48, 4, 2, 32)),
              O.min_gru_layer(width=160, mlp=O.moe(32, 8, 2, 64))]
    cfg = O.make_config(layers=layers, width=64, groups=2, streams=4, loop=(1, 3, 2))
    W = O.random_weights(cfg, seed=7)
    toks = tokens_for(cfg, 300, 2)
    want = O.forward(cfg, f64(W), toks)
    model = make_model(tmp_path / "m", cfg, W, "bfloat16")
    assert close(model.step([entry(0, toks, 0)]), want, "bfloat16")
    assert close(run_in_portions(model, 1, toks, [33, 2, 64, 1]), want, "bfloat16")


def test_first_tokens_of_a_sequence(tmp_path, default_case):
    """Sequences of one to four tokens, alone and decoded, in blocks and slots that longer sequences used before."""
    cfg, W, toks, want, _ = default_case
    model = make_model(tmp_path / "m", cfg, W, "float32", max_seqs=2)
    model.step([entry(0, toks, 0, want=[]), entry(1, toks[::-1], 0, want=[])])
    model.free_seqs_resources([0, 1])
    for n in (1, 2, 3, 4):
        assert rel_err(model.step([entry(0, toks[:n], 0)]), want[:n]) < F32_TOL
        assert rel_err(run_in_portions(model, 1, toks[:n], [1]), want[:n]) < F32_TOL
        model.free_seqs_resources([0, 1])


def test_long_decoding(tmp_path, default_case):
    cfg, W, _, _, _ = default_case
    toks = tokens_for(cfg, 330, 3)
    want = O.forward(cfg, f64(W), toks)
    model = make_model(tmp_path / "m", cfg, W, "float32", num_blocks=24)
    assert rel_err(run_in_portions(model, 0, toks, [10, 1]), want) < F32_TOL


def test_swap_out_and_in_keeps_the_sequence(tmp_path, default_case):
    cfg, W, toks, want, _ = default_case
    model = make_model(tmp_path / "m", cfg, W, "float32", num_blocks=12, cpu_blocks=8, max_seqs=2)
    first = model.step([entry(0, toks[:40], 0)])
    model.swap_out_seqs([0])
    assert model.gpu_block_manager.num_free_blocks == 12 and model.state.num_free_slots == 2
    model.step([entry(1, tokens_for(cfg, 100, 1), 0, want=[])])      # overwrites the freed blocks and the freed slot
    model.free_seqs_resources([1])
    model.step([entry(1, tokens_for(cfg, 30, 2), 0, want=[])])
    model.swap_in_seqs([0])
    rest = model.step([entry(0, toks[40:], 40)])
    assert rel_err(torch.cat((first, rest)), want) < F32_TOL


def test_greedy_generation_through_the_engine(tmp_path, default_case):
    """The framework's own entry point: Engine + scheduler + worker protocol, whole prompts then decoding, requests of
    unequal length finishing at different times."""
    from swiftllm_amd import EngineConfig
    from swiftllm_amd.server import Engine, RawRequest
    cfg, W, _, _, _ = default_case
    path = str(tmp_path / "m")
    O.write_checkpoint(path, cfg, W)
    ecfg = EngineConfig(model_path=path, use_dummy=False, block_size=16, gpu_mem_utilization=0.12, num_cpu_blocks=8,
                        max_seqs_in_block_table=4, max_blocks_per_seq=16, max_batch_size=4, max_tokens_in_batch=256,
                        dtype="float32", use_hip_graph=True)
    prompts = [tokens_for(cfg, n, 20 + n) for n in (5, 43, 18)]
    outs = (6, 12, 9)
    Wd = f64(W)

    def oracle(prompt, n):
        seq = list(prompt)
        for _ in range(n):
            lg = O.forward(cfg, Wd, seq)[-1]
            top2 = torch.topk(lg, 2).values
            assert float(top2[0] - top2[1]) > 1e-4, "the test's weights make a close call"
            seq.append(int(torch.argmax(lg)))
        return seq[len(prompt):]

    async def run():
        engine = Engine(ecfg)
        await engine.initialize()
        assert type(engine.model).__name__ == "RokevikModel"
        loops = asyncio.ensure_future(engine.start_all_event_loops())
        res = await asyncio.gather(*[engine.add_request_and_wait(RawRequest("", n, p)) for p, n in zip(prompts, outs)])
        loops.cancel()
        try:
            await loops
        except (asyncio.CancelledError, Exception):
            pass
        return [r[1] for r in res]

    got = asyncio.run(run())
    import gc
    gc.collect()                    # (the engine's pool goes back before the next test sizes its own)
    torch.cuda.empty_cache()
    for g, p, n in zip(got, prompts, outs):
        assert g == oracle(p, n)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner_replays_a_mixed_schedule(tmp_path, dtype):
    """bin/trace_run as a user starts it: five requests through four block-table rows and state slots and a pool of 20 blocks,
    portions beside decoded tokens, a request that sits steps out, finished requests whose blocks and slot the next one takes."""
    import json
    import os
    import subprocess
    import sys
    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = varied_config()
    W = O.random_weights(cfg, seed=13)
    path = O.write_checkpoint(str(tmp_path / "m"), cfg, W)
    lens = {"a": 70, "b": 5, "c": 40, "d": 1, "e": 33}
    reqs = {k: tokens_for(cfg, n, 90 + i) for i, (k, n) in enumerate(lens.items())}
    schedule = [[("a", 30), ("b", 2), ("c", 17)], [("a", 1), ("b", 1), ("d", 1)], [("a", 2), ("c", 1), ("b", 2)],
                [("e", 16), ("a", 20)], [("e", 1), ("c", 22)], [("a", 17), ("e", 16)]]
    at = {k: 0 for k in lens}
    lines, asked = [], []
    for n, step in enumerate(schedule):
        entries, end = [], []
        for k, c in step:
            want = list(range(c))[-3:]       # the last three places of every portion
            entries.append({"id": k, "tokens": reqs[k][at[k]:at[k] + c], "want": want})
            asked += [(n, k, at[k] + w) for w in want]
            at[k] += c
            if at[k] == lens[k]:
                end.append(k)
        lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
    assert at == lens
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", dtype, "--out",
                        str(out), "--max-tokens", "320"], input="\n".join(lines) + "\n", capture_output=True, text=True,
                       timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {n}" for n in range(len(schedule))]
    wants = {k: O.forward(cfg, f64(W), t) for k, t in reqs.items()}
    got, want = [], []
    for n in range(len(schedule)):
        rows = [(k, p) for m, k, p in asked if m == n]
        got.append(torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(len(rows), cfg["vocab"])))
        want.append(torch.stack([wants[k][p] for k, p in rows]))
        if dtype == "float32":
            assert close(got[-1], want[-1], dtype), f"step {n}"
    assert close(torch.cat(got), torch.cat(want), dtype)
