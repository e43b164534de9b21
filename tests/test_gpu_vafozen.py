"""Vafozen on the GPU against the plain implementation in tests/vafozen_oracle.py: every mechanism alone, whole prompts,
token-by-token decoding, portions down to two tokens, unequal batches, reused blocks and state slots, far keys, keys at page
borders and at both sides of a chunk's edge, the first tokens of a sequence, long decoding, odd sizes, hipGraph replays,
swapping, and greedy generation through the Engine and its scheduler. Configurations and weights are made here (small, random,
seeded)."""
import asyncio
import random

import pytest
import torch

import vafozen_oracle as O

pytestmark = pytest.mark.gpu

F32_TOL = 3e-5      # relative rms error of fp32 logits (true fp32 products, fp32 statistics)
BF16_TOL = 8e-2     # the same in bfloat16 (bf16 products and activations, fp32 stream, statistics and recurrences)
EPS = 1e-5


def f64(W):
    return {k: v.double() for k, v in W.items()}


def make_model(path, cfg, W, dtype="float32", num_blocks=48, max_seqs=4, cpu_blocks=0, graph=False, max_len=512, **kw):
    from swiftllm_amd import EngineConfig, build_model
    O.write_checkpoint(str(path), cfg, W)
    ecfg = EngineConfig(model_path=str(path), use_dummy=False, block_size=16, gpu_mem_utilization=0.9,
                        num_cpu_blocks=cpu_blocks, max_seqs_in_block_table=max_seqs, max_blocks_per_seq=-(-max_len // 16),
                        max_batch_size=max_seqs, max_tokens_in_batch=1024, dtype=dtype, use_hip_graph=graph, **kw)
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
    """fp32: every position within the tolerance; 16-bit: the median within half of it and all but a few positions within it."""
    e = row_err(got, want)
    if dtype in ("float32", torch.float32):
        return float(e.max()) < (tol or F32_TOL)
    tol = tol or BF16_TOL
    return float(e.median()) < tol / 2 and float((e < tol).double().mean()) >= 0.9


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


def cut(n, sizes):
    """[(start, count)] of a sequence of n tokens cut into portions of the given sizes (the last repeats)."""
    out, at, i = [], 0, 0
    while at < n:
        c = min(sizes[min(i, len(sizes) - 1)], n - at)
        out.append((at, c))
        at += c
        i += 1
    return out


class Pages:
    """A pool of pages full of finite garbage and a block table in which another sequence owns the first blocks."""

    def __init__(self, k_elems, v_elems, dtype, num_blocks=40, off=24, max_blocks=None):
        from swiftllm_amd.worker.block_manager import BlockManager
        from swiftllm_amd.worker.kernels.window_attn import PoolSlice
        self.mgr = BlockManager("GPU", num_blocks, 3, max_blocks or num_blocks, 16, "cuda")
        self.mgr.allocate_blocks_for_seqs([1], [37])
        self.slice = PoolSlice(off, off + k_elems * 16)
        elems = off + (k_elems + v_elems) * 16 + 16
        self.pool = torch.full((num_blocks, elems + -elems % 8), 3e4, dtype=dtype, device="cuda")

    def token(self, seq, pos, G, kd, vd):
        """-> (key rows [G, kd], value rows [G, vd]) of one position as the pool holds them"""
        page = self.pool[int(self.mgr.block_table[seq][pos // 16])].cpu().double()
        k0, v0, o = self.slice.k_offset, self.slice.v_offset, pos % 16
        return page[k0:k0 + G * kd * 16].view(G, 16, kd)[:, o], page[v0:v0 + G * vd * 16].view(G, vd, 16)[:, :, o]


class Step:
    """Plans hand-made steps of sequences 0 and 2 over a StateSlotManager whose slots hold NaN, and over Pages when given."""

    def __init__(self, state, pages=None):
        self.state, self.pages = state, pages
        state.allocate()
        state.pool.fill_(float("nan"))          # nothing may be read before it is written

    def context(self, parts, tiled=True):
        """parts: (sequence, start, count) of every portion of the step."""
        from swiftllm_amd.worker.batch_plan import StepEntry, plan_step
        from swiftllm_amd.worker.kernels.rms_stream import StateRef
        from swiftllm_amd.worker.layers.lorulix_layer import StepContext
        plan = plan_step([StepEntry(s, [0] * c, at) for s, at, c in parts])
        codes = self.state.begin_step([p[0] for p in parts], [p[1] for p in parts])
        plan.tok_state = torch.tensor([int(x) for p, x in zip(parts, codes) for _ in range(p[2])]).numpy()
        dev = {name: torch.from_numpy(getattr(plan, name).astype("int32")).cuda() for name in plan.SEGMENTS}
        st = StateRef(self.state.pool, dev["tok_pos"], dev["tok_start"], dev["tok_state"], dev["tok_seq"], dev["seq_row0"],
                      dev["seq_cnt"], (dev["tile_row0"], dev["tile_cnt"], dev["seq_tile0"]))
        table = None
        if self.pages is not None:
            for s, at, c in parts:
                self.pages.mgr.allocate_blocks_for_seqs([s], [at + c])
            table = self.pages.mgr.block_table
        return StepContext(self.pages.pool if self.pages else None, table, dev["tok_seq"], dev["tok_pos"],
                           (dev["tile_row0"], dev["tile_cnt"]) if tiled else None, st)

    def ref(self, parts):
        return self.context(parts).state


def state_manager():
    from swiftllm_amd.worker.state_slots import StateSlotManager
    m = StateSlotManager(3)
    m.add_region(5)         # (regions do not start at the slot's first float)
    return m


# ---- decays ------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("n,width,rank,channels", [(1, 64, 16, 48), (37, 320, 32, 80), (130, 96, 64, 256), (5, 40, 7, 30),
                                                   (33, 1024, 128, 1024), (3, 64, 16, 33), (18, 2048, 64, 2048)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
def test_low_rank_decays(n, width, rank, channels, dtype):
    """Both kinds, with and without the first matrix, with values that reach both flat ends."""
    from swiftllm_amd.worker.kernels.linear_scan import DECAY_EXP_EXP, DECAY_SIGMOID_POWER, low_rank_decay
    g = torch.Generator().manual_seed(n + rank)
    wide = torch.randn(n, width + 8, generator=g).to(dtype)
    x = wide[:, 8:]
    w1 = (torch.randn(rank, width, generator=g) / width ** 0.5).to(dtype)
    w2 = (2 * torch.randn(channels, rank, generator=g) / rank ** 0.5).to(dtype)
    b = 3 * torch.randn(channels, generator=g)
    b[0], b[1] = 200.0, -200.0
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    z = x.double() @ w1.double().T
    y = torch.tanh(z) @ w2.double().T + b.double()
    got = low_rank_decay(wide.cuda()[:, 8:], w1.cuda(), w2.cuda(), b.cuda(), DECAY_EXP_EXP, tanh=True)
    assert got.dtype == torch.float32 and (got.cpu().double() - torch.exp(-torch.exp(y))).abs().max() < tol
    assert bool((got[:, 0] == 0).all()) and bool((got[:, 1] == 1).all())
    for tau in (1.0, 16.0):
        y = z @ w2.double().T + b.double()
        want = torch.sigmoid(y).pow(1.0 / tau)
        got = low_rank_decay(wide.cuda()[:, 8:], w1.cuda(), w2.cuda(), b.cuda(), DECAY_SIGMOID_POWER, 1.0 / tau)
        assert (got.cpu().double() - want).abs().max() < tol
        rows = torch.cat((torch.zeros(n, 8), z.float()), dim=1).to(dtype)
        y = rows[:, 8:].double() @ w2.double().T + b.double()
        got = low_rank_decay(rows.cuda()[:, 8:], None, w2.cuda(), b.cuda(), DECAY_SIGMOID_POWER, 1.0 / tau)
        assert (got.cpu().double() - torch.sigmoid(y).pow(1.0 / tau)).abs().max() < tol


# ---- shifted mixes -----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width,mixes", [(64, 5), (37, 3), (2056, 5), (8, 1)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_token_shift_in_portions_of_two_sequences(width, mixes, dtype):
    from swiftllm_amd.worker.kernels.rms_stream import token_shift_mix
    g = torch.Generator().manual_seed(width)
    hs = [torch.randn(n, width, generator=g).to(dtype) for n in (23, 40)]
    mu = torch.rand(mixes, width, generator=g)
    mgr = state_manager()
    off = mgr.add_region(2 * width)
    step = Step(mgr)
    at, got = [0, 0], [[], []]
    for counts in [(1, 0), (2, 7), (0, 1), (1, 16), (17, 2), (2, 14)]:
        parts = [((0, 2)[i], at[i], c) for i, c in enumerate(counts) if c]
        rows = torch.cat([hs[i][at[i]:at[i] + c] for i, c in enumerate(counts) if c])
        y = token_shift_mix(rows.cuda(), mu.cuda(), step.ref(parts), off)
        o = 0
        for i, c in enumerate(counts):
            got[i].append(y[:, o:o + c].cpu())
            o += c
            at[i] += c
    for h, y in zip(hs, got):
        hd = h.double()
        prev = torch.cat((torch.zeros_like(hd[:1]), hd[:-1]))
        want = hd + (prev - hd) * mu.double()[:, None]
        err = (torch.cat(y, dim=1).double() - want).abs().max()
        assert err < (1e-6 if dtype == torch.float32 else 3e-2)


@pytest.mark.parametrize("m,k,n,groups", [(1, 128, 256, 4), (32, 256, 512, 4), (20, 64, 96, 3), (70, 128, 128, 2), (5, 1024, 4096, 4)])
@pytest.mark.parametrize("packed", [True, False])
def test_grouped_products(m, k, n, groups, packed):
    """Several inputs, each with its own rows of one matrix: the one-launch form of decode steps and the others."""
    from swiftllm_amd.worker.kernels.linear import linear_grouped, pack_weight, packable
    g = torch.Generator().manual_seed(m)
    for dtype in (torch.bfloat16, torch.float32):
        x = torch.randn(groups, m, k, generator=g).to(dtype)
        w = (torch.randn(n, k, generator=g) / k ** 0.5).to(dtype).cuda()
        if packed and dtype == torch.bfloat16 and packable(w):
            pack_weight(w)
        size = n // groups
        want = torch.cat([x[i].double() @ w[i * size:(i + 1) * size].cpu().double().T for i in range(groups)], dim=1)
        got = linear_grouped(x.cuda(), w, dtype == torch.bfloat16).cpu().double()
        assert (got - want).abs().max() < (1e-4 if dtype == torch.float32 else 3e-2)


# ---- recurrences -------------------------------------------------------------------------------------------------------------
REC_CASES = [  # H, heads of q / k, d, dv, bonus, decay per channel, factor on k, skip
    (3, 3, 12, 20, False, True, False, False), (4, 4, 64, 64, True, True, False, False), (2, 2, 128, 128, False, True, False, False),
    (6, 2, 20, 12, False, False, True, True), (1, 1, 5, 3, True, True, False, False), (2, 1, 200, 40, False, False, True, True),
    (2, 2, 320, 16, True, True, False, False), (3, 3, 33, 260, False, True, False, False), (5, 5, 16, 256, True, True, False, True)]


@pytest.mark.parametrize("H,G,d,dv,bonus,channel,scaled,skip", REC_CASES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_linear_recurrences(H, G, d, dv, bonus, channel, scaled, skip, dtype):
    """Whole, in portions and token by token, two sequences per step, slots that hold NaN; decays from almost none to total ones."""
    from swiftllm_amd.worker.kernels.linear_scan import linear_recurrence
    g = torch.Generator().manual_seed(d + dv)
    lens = (75, 34)
    data = []
    for n in lens:
        q, k, v = (torch.randn(n, s, generator=g).to(dtype) for s in (G * d, G * d, H * dv))
        decay = torch.rand(n, H * d if channel else H, generator=g) ** 0.2
        decay[torch.rand(decay.shape, generator=g) < 0.03] = 0.0
        decay[torch.rand(decay.shape, generator=g) < 0.2] = 1.0
        data.append((q, k, v, decay, 0.2 + torch.rand(n, H, generator=g)))
    u = torch.randn(H, d, generator=g) if bonus else None
    D = torch.randn(H, generator=g) if skip else None
    want = []
    for (q, k, v, decay, ks), n in zip(data, lens):
        rep = lambda x: x.double().view(n, G, d).repeat_interleave(H // G, dim=1)       # noqa: E731
        a = decay.double().view(n, H, -1).expand(n, H, d)
        kk = rep(k) * ks.double()[..., None] if scaled else rep(k)
        vv = v.double().view(n, H, dv)
        o = O.bonus_scan(0.3 * rep(q), kk, vv, a, u.double()) if bonus else O.linear_scan(0.3 * rep(q), kk, vv, a)
        want.append((o + (D.double()[:, None] * vv if skip else 0)).reshape(n, H * dv))
    norm_w, tol = 1 + 0.3 * torch.randn(H * dv, generator=g), 3e-5
    gates = [torch.randn(n, H * dv, generator=g).to(dtype) for n in lens]
    for steps in ([lens], [(17, 1), (1, 2), (40, 0), (2, 30), (15, 1)], [(1, 1)] * 34 + [(1, 0)] * 41):
        for finish in (False, True):
            mgr = state_manager()
            off = mgr.add_region(H * d * dv)
            step = Step(mgr)
            at, got = [0, 0], [[], []]
            for counts in steps:
                parts = [((0, 2)[i], at[i], c) for i, c in enumerate(counts) if c]
                pick = lambda j: torch.cat([data[i][j][at[i]:at[i] + c] for i, c in enumerate(counts) if c]).cuda()     # noqa: E731
                # (q | k | v are column slices of wider rows)
                rows = torch.cat((pick(0), pick(1), pick(2)), dim=1)
                q, k, v = rows[:, :G * d], rows[:, G * d:2 * G * d], rows[:, 2 * G * d:]
                kw, out = {}, None
                if finish:
                    gate = torch.cat([gates[i][at[i]:at[i] + c] for i, c in enumerate(counts) if c]).cuda()
                    out = torch.zeros(rows.shape[0], H * dv + 8, dtype=dtype, device="cuda")
                    kw["finish"] = (out[:, 8:], norm_w.cuda() if bonus else norm_w[:dv].cuda(), gate, EPS, 1.7)
                y = linear_recurrence(q, k, v, pick(3), step.ref(parts), off, H, d, dv, q_scale=0.3,
                                      bonus=u.cuda() if bonus else None, k_scale=pick(4).contiguous() if scaled else None,
                                      dskip=D.cuda() if skip else None, num_qk_heads=G, **kw)
                assert not finish or bool((out[:, :8] == 0).all())
                o = 0
                for i, c in enumerate(counts):
                    got[i].append(y[o:o + c].cpu().double())
                    o += c
                    at[i] += c
            for i, n in enumerate(lens):
                y, w_ = torch.cat(got[i]), want[i]
                if finish:
                    nw = norm_w.double().view(H, dv) if bonus else norm_w[:dv].double()
                    w_ = (1.7 * O.unit_rms(w_.view(n, H, dv), EPS) * nw).reshape(n, H * dv) * O.silu(gates[i].double())
                scale = float(w_.abs().max())
                assert (y - w_).abs().max() < (tol if dtype == torch.float32 or not finish else 1e-2) * scale, (steps[0], finish)


def test_a_state_that_keeps_the_first_token_and_one_that_forgets_at_once():
    from swiftllm_amd.worker.kernels.linear_scan import linear_recurrence
    n, H, d, dv = 300, 2, 32, 16
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(n, s, generator=g) for s in (H * d, H * d, H * dv))
    k[0] *= 1000.0
    decay = torch.full((n, H, d), 0.9999)
    decay[:, 1] = 0.0
    args = [x.double().view(n, H, -1) for x in (q, k, v)] + [decay.double()]
    want = O.linear_scan(*args).reshape(n, -1)
    lost = args[1].clone()
    lost[0] = 0
    other = O.linear_scan(args[0], lost, args[2], args[3]).reshape(n, -1)
    scale = float(want.abs().max())
    assert (other[-1, :dv] - want[-1, :dv]).abs().max() > 0.05 * scale and torch.equal(other[1:, dv:], want[1:, dv:])
    for sizes in ((1000,), (1,), (100, 1, 2, 33)):
        mgr = state_manager()
        off = mgr.add_region(H * d * dv)
        step, got = Step(mgr), []
        for at, c in cut(n, sizes):
            s = slice(at, at + c)
            got.append(linear_recurrence(q[s].cuda(), k[s].cuda(), v[s].cuda(), decay.view(n, -1)[s].contiguous().cuda(),
                                         step.ref([(0, at, c)]), off, H, d, dv).cpu().double())
        assert (torch.cat(got) - want).abs().max() < 3e-5 * scale, sizes


@pytest.mark.parametrize("heads,P,N,groups,conv,parts,n", [(3, 8, 12, 1, 3, 1, 70), (4, 24, 20, 2, 1, 2, 33), (2, 32, 64, 2, 4, 1, 90),
                                                           (6, 16, 128, 3, 2, 3, 21), (1, 64, 16, 1, 5, 4, 50), (2, 8, 400, 1, 2, 1, 37)])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_state_space_mixer_alone(heads, P, N, groups, conv, parts, n, dtype):
    """State sizes on both sides of what runs by tiles."""
    check_layer(O.mamba_layer(heads=heads, vdim=P, state=N, groups=groups, conv=conv, norm_groups=parts, ff=0), n, 40, dtype,
                cuts=((1000,), (5, 1, 2, 16, 3), (1,)))


# ---- convolved, normed, rotated rows -----------------------------------------------------------------------------------------
STORE_CASES = [  # H, G, d, dv, taps, norm, rot dims, half, key row, value row
    (4, 2, 64, 64, 4, False, 64, True, 64, 64), (6, 3, 40, 56, 3, False, 16, True, 64, 64), (3, 1, 10, 6, 2, False, 6, True, 10, 10),
    (5, 5, 24, 16, 0, True, 0, True, 32, 32), (2, 1, 128, 96, 0, True, 0, True, 128, 128), (4, 4, 16, 24, 5, True, 8, True, 32, 32),
    (3, 3, 48, 32, 1, False, 48, True, 48, 48), (7, 1, 12, 20, 3, True, 12, False, 15, 21), (2, 2, 200, 64, 4, False, 64, True, 288, 256)]


@pytest.mark.parametrize("H,G,d,dv,taps,norm,rd,half,kd,vd", STORE_CASES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_convolution_norm_rotation_and_store(H, G, d, dv, taps, norm, rd, half, kd, vd, dtype):
    """Pages read back around far positions and at the start; the convolution's inputs cross portions and carry no bias before the
    sequence's start."""
    from swiftllm_amd.model_config import RotaryConfig
    from swiftllm_amd.worker.kernels.rope_kv import qkv_conv_rope_and_store_kv, rotary_frequencies
    g = torch.Generator().manual_seed(d + H)
    n, C, extra = 45, (H + G) * d + G * dv, 5
    rows = torch.randn(n, C + extra + -(C + extra) % 8, generator=g).to(dtype)
    bias, conv = torch.randn(C, generator=g), torch.randn(C, taps, generator=g) / max(taps, 1) ** 0.5
    qw, kw_ = 1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)
    rot_cfg = {"dims": rd, "base": 777.0}
    rot = RotaryConfig(rot_cfg if rd else None, d, half=half)
    freq = rotary_frequencies(rot, torch.device("cuda"))
    mgr = state_manager()
    off = mgr.add_region(2 * max(taps - 1, 0) * C)
    pages = Pages(G * kd, G * vd, dtype)
    step, got = Step(mgr, pages), []
    for at, c in cut(n, (1, 2, 17, 1, 16, 3)):
        ctx = step.context([(2, at, c)])
        got.append(qkv_conv_rope_and_store_kv(rows[at:at + c].cuda(), bias.cuda(), conv.t().contiguous().cuda() if taps else None,
                                              qw.cuda() if norm else None, kw_.cuda() if norm else None, freq, rot, ctx.pool,
                                              pages.slice, ctx.block_table, ctx.state, off, H, G, d, dv, kd, vd, EPS, 0.7).cpu())
    u = rows[:, :C].double() + bias.double()
    if taps:
        u = O.causal_conv(u, conv.double())
    q, k, v = u[:, :H * d].view(n, H, d), u[:, H * d:(H + G) * d].view(n, G, d), 0.7 * u[:, (H + G) * d:].view(n, G, dv)
    if norm:
        q, k = O.unit_rms(q, EPS) * qw.double(), O.unit_rms(k, EPS) * kw_.double()

    def turn(x):
        if not rd:
            return x
        if half:
            return O.rotate_halves(x, rd, 777.0)
        perm = torch.tensor(list(range(0, rd, 2)) + list(range(1, rd, 2)) + list(range(rd, d)))     # neighbouring pairs
        y = torch.empty_like(x)
        y[..., perm] = O.rotate_halves(x[..., perm], rd, 777.0)
        return y
    q, k = turn(q), turn(k)
    tol = (2e-5 if dtype == torch.float32 else 2e-2) * max(1.0, float(q.abs().max()), float(v.abs().max()))
    gq = torch.cat(got).double().view(n, H, kd)
    assert (gq[..., :d] - q).abs().max() < tol and bool((gq[..., d:] == 0).all())
    for t in range(n):
        gk, gv = pages.token(2, t, G, kd, vd)
        assert (gk[:, :d] - k[t]).abs().max() < tol and bool((gk[:, d:] == 0).all()), t
        assert (gv[:, :dv] - v[t]).abs().max() < tol and bool((gv[:, dv:] == 0).all()), t


def test_rotation_far_from_the_start():
    """Angles are evaluated in double precision: positions around 30 000 are as exact as the first ones."""
    from swiftllm_amd.model_config import RotaryConfig
    from swiftllm_amd.worker.kernels.rope_kv import qkv_conv_rope_and_store_kv, rotary_frequencies
    H, G, d, dv, n, start = 2, 1, 16, 8, 9, 30011
    g = torch.Generator().manual_seed(1)
    rows = torch.randn(n, (H + G) * d + G * dv, generator=g)
    rot = RotaryConfig({"dims": 12, "base": 1e4}, d, half=True)
    pages = Pages(G * d, G * dv, torch.float32, num_blocks=2000, max_blocks=1990)
    mgr = state_manager()
    step = Step(mgr, pages)
    mgr.begin_step([2], [0])
    ctx = step.context([(2, start, n)])
    q = qkv_conv_rope_and_store_kv(rows.cuda(), None, None, None, None, rotary_frequencies(rot, torch.device("cuda")), rot, ctx.pool,
                                   pages.slice, ctx.block_table, ctx.state, 0, H, G, d, dv, d, dv, EPS)
    x = torch.zeros(start + n, H, d, dtype=torch.float64)
    x[start:] = rows[:, :H * d].double().view(n, H, d)
    assert (q.cpu().double().view(n, H, d) - O.rotate_halves(x, 12, 1e4)[start:]).abs().max() < 1e-5


# ---- a layer's mixers --------------------------------------------------------------------------------------------------------
class LayerBench:
    """One layer of the product with weights loaded by the product's loader, on a hand-made pool of garbage and state slots that hold
    NaN; `pad`: the pool's rows as the worker would choose them for the dtype."""

    def __init__(self, layer, W, dtype, width=64, num_blocks=48, pad=True, skinny=False):
        from swiftllm_amd.model_config import VafozenModelConfig
        from swiftllm_amd.worker.kernels.window_attn import served_row_sizes
        from swiftllm_amd.worker.layers.vafozen_layer import VafozenLayer
        from swiftllm_amd.worker.vafozen_weight import VafozenLayerWeight
        cfg = VafozenModelConfig(O.make_config(layers=[layer], width=width, eps=EPS))
        lcfg = cfg.layers[0]
        lw = VafozenLayerWeight(0)
        lw.load(lambda name, shape: W[name].clone(), cfg, lcfg, dtype, torch.device("cuda"))
        self.dtype, mgr, pages, sizes = dtype, state_manager(), None, None
        if lcfg.attention is not None:
            mx = lcfg.attention
            need = (mx.head_dim, mx.value_dim)
            sizes = served_row_sizes(*need, dtype) if pad else need
            pages = Pages(mx.num_kv_heads * sizes[0], mx.num_kv_heads * sizes[1], dtype, num_blocks)
        self.op = VafozenLayer(lcfg, lw, cfg.norm_eps, skinny, mgr, pages.slice if pages else None, sizes, 1024)
        self.step = Step(mgr, pages)
        self.bias = lw.y_bias.cpu().double() if lw.y_bias is not None else 0

    def run(self, h, portions, tiled=True, seq=2):
        """-> the layer's result for every token of one sequence, fed in the given portions (the last size repeats)."""
        out = []
        for at, c in cut(h.shape[0], portions):
            out.append(self.op.forward(h[at:at + c].to(self.dtype).cuda(), self.step.context([(seq, at, c)], tiled)).cpu().double())
        return torch.cat(out) + self.bias

    def run_together(self, hs, steps, tiled=True):
        """hs: the inputs of sequences 0 and 2; steps: per step the tokens each brings (0: sits out)."""
        at, got = [0] * len(hs), [[] for _ in hs]
        for counts in steps:
            parts = [((0, 2)[i], at[i], c) for i, c in enumerate(counts) if c]
            rows = torch.cat([hs[i][at[i]:at[i] + c] for i, c in enumerate(counts) if c])
            y = self.op.forward(rows.to(self.dtype).cuda(), self.step.context(parts, tiled))
            o = 0
            for i, c in enumerate(counts):
                got[i].append(y[o:o + c].cpu().double())
                o += c
                at[i] += c
        return [torch.cat(g) + self.bias for g in got]


def one_layer(layer, seed, width=64):
    return O.random_weights(O.make_config(layers=[layer], width=width), seed)


def oracle_layer(layer, W, h):
    Wd, hd = f64(W), h.double()
    y = O.MIXERS[layer["type"]](hd, Wd, "l0.mix.", layer["mixer"], EPS)
    return y + O.gated_unit(hd, Wd, "l0.mlp.") if layer["mlp"] else y


def layer_tol(dtype, want):
    return (1e-4 if dtype == torch.float32 else 4e-2) * max(1.0, float(want.abs().max()))


def check_layer(layer, n, width=64, dtype=torch.float32, cuts=((1000,), (5, 1, 2, 30, 2), (1,)), tiled=True, pad=True, seed=0):
    W = one_layer(layer, seed + n, width)
    if dtype != torch.float32:
        W = {k: v.to(dtype).float() for k, v in W.items()}
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(n)).to(dtype).float()
    want = oracle_layer(layer, W, h)
    for portions in cuts:
        got = LayerBench(layer, W, dtype, width, pad=pad).run(h, portions, tiled)
        assert (got - want).abs().max() < layer_tol(dtype, want), portions


@pytest.mark.parametrize("kw,n", [(dict(), 130), (dict(heads=3, kv_heads=3, dim=10, vdim=6, chunk=1, tau=1.0), 40),
                                  (dict(heads=6, kv_heads=1, dim=24, vdim=40, chunk=0, g_heads=1, g_dim=33, g_vdim=9), 70),
                                  (dict(heads=1, kv_heads=1, dim=8, vdim=8, chunk=16, g_heads=5, g_dim=4, g_vdim=28, rank=16, ff=0), 1),
                                  (dict(heads=8, kv_heads=4, dim=16, vdim=16, chunk=50, left_scale=1.0, right_scale=-0.4), 101)])
def test_distance_attention_beside_linear_attention(kw, n):
    check_layer(O.parallel_layer(**kw), n)


@pytest.mark.parametrize("kw,n", [(dict(heads=4, kv_heads=2, dim=64, vdim=64, chunk=40, g_heads=2, g_dim=64, g_vdim=32, rank=16), 130),
                                  (dict(heads=6, kv_heads=3, dim=40, vdim=56, chunk=33, rank=12), 90),
                                  (dict(heads=10, kv_heads=5, dim=112, vdim=96, chunk=0, g_heads=1, g_dim=128, g_vdim=128, ff=0), 60),
                                  (dict(heads=16, kv_heads=1, dim=32, vdim=32, chunk=17), 80)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
def test_distance_attention_on_the_matrix_cores(kw, n, dtype):
    layer = O.parallel_layer(**kw)
    check_layer(layer, n, 128, dtype, cuts=((17, 1, 2, 40), (1000,), (1,)))
    check_layer(layer, n, 128, dtype, cuts=((17, 1, 2, 40),), tiled=False, pad=False)


@pytest.mark.parametrize("kw,n", [(dict(), 130), (dict(heads=3, kv_heads=1, dim=10, vdim=6, conv=1, rot_dims=10, softcap=1.0), 60),
                                  (dict(heads=2, kv_heads=2, dim=24, vdim=16, conv=5, rot_dims=4, softcap=50.0, r_heads=1, r_dim=33), 70),
                                  (dict(heads=6, kv_heads=3, dim=8, vdim=24, conv=2, rot_dims=8, r_heads=5, r_dim=8, rank=16, ff=0), 1),
                                  (dict(heads=4, kv_heads=4, conv=6, left_scale=1.0, right_scale=1.0), 3)])
def test_convolved_attention_beside_time_mixing(kw, n):
    check_layer(O.parallel2_layer(**kw), n)


@pytest.mark.parametrize("kw,n", [(dict(heads=4, kv_heads=2, dim=64, vdim=64, rot_dims=32, r_heads=2, r_dim=64, rank=16), 130),
                                  (dict(heads=6, kv_heads=3, dim=40, vdim=56, rot_dims=40, conv=4, rank=20), 90),
                                  (dict(heads=5, kv_heads=1, dim=128, vdim=128, rot_dims=64, conv=2, r_heads=1, r_dim=128, ff=0), 60)])
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
def test_convolved_attention_on_the_matrix_cores(kw, n, dtype):
    layer = O.parallel2_layer(**kw)
    check_layer(layer, n, 128, dtype, cuts=((17, 1, 2, 40), (1000,), (1,)))
    check_layer(layer, n, 128, dtype, cuts=((17, 1, 2, 40),), tiled=False, pad=False)


@pytest.mark.parametrize("layer", [O.parallel_layer(), O.parallel2_layer(), O.mamba_layer()], ids=lambda l: l["type"])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_two_sequences_of_a_step_do_not_meet(layer, dtype):
    W = {k: v.to(dtype).float() for k, v in one_layer(layer, 21).items()}
    g = torch.Generator().manual_seed(2)
    hs = [torch.randn(n, 64, generator=g).to(dtype).float() for n in (130, 77)]
    got = LayerBench(layer, W, dtype).run_together(hs, [(70, 1), (1, 40), (0, 3), (1, 1), (1, 1), (2, 31), (55, 0)])
    for h, y in zip(hs, got):
        want = oracle_layer(layer, W, h)
        assert (y - want).abs().max() < layer_tol(dtype, want)


def _asking_weights(layer, W, h_ask, h_answer, gain):
    """Rewrite the left projections so that the asking direction's query is the answering direction's key."""
    k = W["l0.mix.left.k"]
    reps = layer["mixer"]["left"]["heads"] // layer["mixer"]["left"]["kv_heads"]
    d, G = layer["mixer"]["left"]["dim"], layer["mixer"]["left"]["kv_heads"]
    turned = (gain * k @ torch.outer(h_answer, h_ask) / (h_ask @ h_ask)).view(G, 1, d, -1).expand(G, reps, d, h_ask.numel())
    W["l0.mix.left.q"] = turned.reshape(G * reps * d, -1) + 0.02 * W["l0.mix.left.q"]
    W["l0.mix.left.q.b"] *= 0.01
    W["l0.mix.left.k.b"] *= 0.01
    W["l0.mix.left.v.b"] *= 0.01


@pytest.mark.parametrize("tiled,dtype", [(False, torch.float32), (True, torch.bfloat16)])
@pytest.mark.parametrize("n,target", [(400, 3), (400, 15), (400, 16), (400, 0)])
def test_a_far_key_among_hundreds_and_at_page_borders(tiled, dtype, n, target):
    """The query projection turns the askers' direction into the key of the answering direction, which only token `target` has: one
    score stands out among hundreds, for askers near and hundreds of positions away, in prompts and decoded."""
    layer = O.parallel2_layer(heads=2, kv_heads=1, dim=32, vdim=32, conv=2, rot_dims=4, base=1e6, scale=0.5, softcap=30.0, ff=0,
                              left_scale=4.0, right_scale=0.1)
    W = one_layer(layer, 7)
    g = torch.Generator().manual_seed(n)
    ask, answer = torch.randn(64, generator=g), torch.randn(64, generator=g)
    _asking_weights(layer, W, ask, answer, 1.0)
    for t in "qkv":     # the convolutions pass the current token and a little of the last one
        W[f"l0.mix.left.{t}.conv"] = torch.tensor([0.1, 1.0]).expand_as(W[f"l0.mix.left.{t}.conv"]).clone()
    h = 0.2 * torch.randn(n, 64, generator=g)
    h[target] = answer
    askers = [t for t in range(target + 2, n) if t % 2 == 0]
    h[askers] += ask
    W = {k: v.to(dtype).float() for k, v in W.items()}
    h = h.to(dtype).float()
    want = oracle_layer(layer, W, h)
    hidden = h.clone()
    hidden[target] = h[target + 1]
    other = oracle_layer(layer, W, hidden)
    assert (other[askers] - want[askers]).abs().max(dim=-1).values.median() > 4 * layer_tol(dtype, want)
    for portions in ((n - 30, 1), (97, 2, 1, 16), (n,)):
        got = LayerBench(layer, W, dtype).run(h, portions, tiled)
        assert (got - want).abs().max() < layer_tol(dtype, want), portions


@pytest.mark.parametrize("tiled,dtype", [(False, torch.float32), (True, torch.bfloat16)])
@pytest.mark.parametrize("chunk", [1, 2, 16, 17, 31, 45, 100])
def test_keys_just_inside_and_just_outside_the_chunk(tiled, dtype, chunk):
    """Marked tokens whose key answers every query, at both sides of every chunk's edge: seen to the end of their chunk and never
    after it, at every place of a page, in prompts, portions and decoding. Chunks one token longer or shifted by one would show."""
    n = 210
    layer = O.parallel_layer(heads=8, kv_heads=4, dim=32, vdim=32, chunk=chunk, scale=1.0, ff=0, left_scale=3.0, right_scale=0.1)
    W = one_layer(layer, 11)
    for t in "qk":
        W[f"l0.mix.left.{t}.norm"] = torch.ones(32)
    g = torch.Generator().manual_seed(chunk)
    u, m = torch.randn(64, generator=g), torch.randn(64, generator=g)
    h = u + 0.2 * torch.randn(n, 64, generator=g)           # every token asks
    edges = range(chunk, n, chunk)
    marks = [t for e in edges for t in (e - 1, e)] if chunk > 2 else [5, 6, 47, 48, 111, 150]
    marks = [t for i, t in enumerate(marks) if (i // 2) % 2 == 0]
    h[marks] += 2 * m                                         # (and the marked ones answer)
    _asking_weights(layer, W, u, m, 1.0)
    W = {k: v.to(dtype).float() for k, v in W.items()}
    h = h.to(dtype).float()
    want = oracle_layer(layer, W, h)
    for portions in ((n - 40, 1), (37, 2, 1, 16, 2), (n,)):
        got = LayerBench(layer, W, dtype).run(h, portions, tiled)
        assert (got - want).abs().max() < layer_tol(dtype, want), portions
    for other_chunk in (chunk + 1, chunk - 1, 0):
        if chunk == 1 and other_chunk == 0:
            continue
        left = dict(layer["mixer"]["left"], mask={"size": other_chunk} if other_chunk else None)
        wrong = dict(layer, mixer=dict(layer["mixer"], left=left))
        assert (oracle_layer(wrong, W, h) - want).abs().max() > 3 * layer_tol(dtype, want), other_chunk


@pytest.mark.parametrize("tiled,dtype", [(False, torch.float32), (True, torch.bfloat16)])
def test_distance_penalty_of_every_head(tiled, dtype):
    """Keys that all score the same: a head's weights fall off as exp(-slope distance) alone, from the steepest head to the flattest,
    far into a long chunk; a slope of another head or form would show."""
    n, H = 300, 4
    layer = O.parallel_layer(heads=H, kv_heads=1, dim=32, vdim=32, chunk=280, ff=0, left_scale=1.0, right_scale=0.0)
    W = one_layer(layer, 3)
    for t in "qk":
        W["l0.mix.left." + t] *= 0
    for t in "qkv":
        W["l0.mix.left." + t + ".b"] *= 0
    W["l0.mix.left.k.b"] += 1.0
    W["l0.mix.left.q.b"] += 1.0
    W = {k: v.to(dtype).float() for k, v in W.items()}
    h = torch.randn(n, 64, generator=torch.Generator().manual_seed(4)).to(dtype).float()
    h[::13] *= 5.0
    h = h.to(dtype).float()
    want = oracle_layer(layer, W, h)
    flat = O.head_slope
    try:
        O.head_slope = lambda hh, heads: flat(min(hh + 1, heads - 1), heads)
        assert (oracle_layer(layer, W, h) - want).abs().max() > 4 * layer_tol(dtype, want)
    finally:
        O.head_slope = flat
    for portions in ((n,), (n - 30, 1), (33, 2, 100, 1)):
        got = LayerBench(layer, W, dtype).run(h, portions, tiled)
        assert (got - want).abs().max() < layer_tol(dtype, want), portions


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_stream_step_sums_k_shares(dtype):
    from swiftllm_amd.worker.kernels.hyper_stream import StreamWeights, hyper_step
    from swiftllm_amd.worker.kernels.linear import SplitKPartials, linear_splitk
    g = torch.Generator().manual_seed(0)
    x, a = torch.randn(9, 1, 256, generator=g), torch.randn(9, 2048, generator=g).bfloat16()
    w, norm, bias = (torch.randn(256, 2048, generator=g) / 45).bfloat16(), torch.rand(256, generator=g), torch.randn(256, generator=g)
    y = linear_splitk(a.cuda(), w.cuda())
    if dtype == torch.float32 or not isinstance(y, SplitKPartials):
        y = (a.double() @ w.double().T).float().to(dtype).cuda()
    want = x[:, 0].double() + a.double() @ w.double().T + bias.double()
    sw, xd = StreamWeights.plain(torch.device("cuda")), x.cuda()
    h = hyper_step(xd, y, sw, y_bias=bias.cuda(), norm=norm.cuda(), eps=EPS)
    tol = 1e-5 if dtype == torch.float32 else 2e-2
    assert (xd.cpu()[:, 0].double() - want).abs().max() < tol
    assert (h.cpu().double() - O.unit_rms(want, EPS) * norm).abs().max() < max(tol, 1e-5)


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
    assert type(model).__name__ == "VafozenModel"
    model.layer_tap = []
    got = model.step([entry(0, toks, 0)])
    assert len(model.layer_tap) == len(streams) == len(cfg["layers"])
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


def matrix_core_config(width=128, vocab=96):
    """Sizes that the 16-bit matrix-core forms serve as they are and padded, projections the decode GEMMs can pack."""
    layers = [O.parallel_layer(heads=4, kv_heads=2, dim=64, vdim=64, chunk=50, g_heads=2, g_dim=64, g_vdim=64, rank=16, ff=256),
              O.parallel2_layer(heads=6, kv_heads=3, dim=40, vdim=56, conv=4, rot_dims=40, r_heads=2, r_dim=64, rank=32, ff=128),
              O.mamba_layer(heads=4, vdim=32, state=64, groups=2, conv=4, norm_groups=2, ff=128),
              O.parallel2_layer(heads=4, kv_heads=1, dim=128, vdim=128, conv=3, rot_dims=64, r_heads=1, r_dim=128, rank=20, ff=0)]
    return O.make_config(layers=layers, width=width, vocab=vocab)


def test_decode_graph_replays_in_bfloat16(tmp_path):
    """Matrix-core shapes: the captured step against eager steps of the same model, replay after replay."""
    cfg = matrix_core_config()
    W = O.random_weights(cfg, 17)
    toks = [tokens_for(cfg, 60, 5), tokens_for(cfg, 44, 6), tokens_for(cfg, 35, 7)]
    runs = []
    for graph in (True, False):
        model = make_model(tmp_path / f"m{graph}", cfg, W, "bfloat16", graph=graph)
        model.step([entry(i, t[:20], 0, want=[]) for i, t in enumerate(toks)])
        runs.append([model.step([entry(i, t[20 + k:21 + k], 20 + k) for i, t in enumerate(toks)]).clone() for k in range(15)])
        torch.cuda.synchronize()
    assert all(torch.equal(a, b) for a, b in zip(*runs))


@pytest.mark.parametrize("packed", [True, False])
def test_matrix_core_paths_in_the_model(tmp_path, packed):
    """bfloat16, with and without the packed weights of the decode GEMMs: whole, in portions and decoded."""
    cfg = matrix_core_config(256)
    W = O.random_weights(cfg, seed=7)
    toks = tokens_for(cfg, 300, 2)
    want = O.forward(cfg, f64(W), toks)
    model = make_model(tmp_path / "m", cfg, W, "bfloat16", pack_decode_weights=packed)
    assert close(model.step([entry(0, toks, 0)]), want, "bfloat16")
    assert close(run_in_portions(model, 1, toks, [33, 2, 64, 1]), want, "bfloat16")


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
    """Sizes that a symmetric configuration would hide: one kv head, heads = kv heads, heads not a power of two, values wider and
    narrower than keys, one tap, six taps, rotation of the whole head, no chunk, chunks of one token and of a page, tau 1, equal and
    negative scales, one norm part, one head, layers without feed-forward first, a width that is no multiple of 8."""
    layers = [O.mamba_layer(heads=3, vdim=10, state=7, groups=1, conv=1, norm_groups=1, ff=0),
              O.parallel2_layer(heads=3, kv_heads=1, dim=12, vdim=30, conv=1, rot_dims=12, base=50.0, softcap=2.0, r_heads=1, r_dim=21,
                                rank=3, left_scale=1.0, right_scale=1.0, ff=20),
              O.parallel_layer(heads=5, kv_heads=5, dim=18, vdim=7, chunk=1, g_heads=1, g_dim=10, g_vdim=40, tau=1.0, rank=1,
                               left_scale=-0.5, right_scale=0.25, ff=28),
              O.parallel2_layer(heads=2, kv_heads=2, dim=20, vdim=4, conv=6, rot_dims=2, softcap=40.0, r_heads=4, r_dim=6, rank=9, ff=0),
              O.parallel_layer(heads=1, kv_heads=1, dim=9, vdim=9, chunk=16, g_heads=4, g_dim=5, g_vdim=6, tau=32.0, ff=12),
              O.parallel_layer(heads=6, kv_heads=2, dim=8, vdim=16, chunk=0, ff=0),
              O.mamba_layer(heads=6, vdim=5, state=33, groups=3, conv=5, norm_groups=5, ff=9)]
    return O.make_config(layers=layers, width=44, vocab=37, eps=1e-3, scale=1.0)


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


def test_models_of_one_kind_of_layer(tmp_path):
    """Each kind alone, also a model without attention (no keys in the pool)."""
    for i, layers in enumerate(([O.mamba_layer(), O.mamba_layer(ff=0)], [O.parallel_layer()], [O.parallel2_layer()])):
        cfg = O.make_config(layers=layers)
        W = O.random_weights(cfg, 6)
        toks = tokens_for(cfg, 60, 8)
        model = make_model(tmp_path / f"m{i}", cfg, W, "float32")
        assert close(run_in_portions(model, 0, toks, [40, 2, 1]), O.forward(cfg, f64(W), toks), "float32")


def random_config(rng):
    layers = []
    for _ in range(rng.randint(2, 5)):
        kind, ff = rng.choice(["parallel", "parallel_2", "mamba2"]), rng.choice([0, 8, 20, 36])
        G = rng.choice([1, 2, 3])
        heads = dict(heads=G * rng.choice([1, 2, 3]), kv_heads=G, dim=rng.choice([8, 12, 16, 40]), vdim=rng.choice([8, 14, 24]),
                     left_scale=rng.choice([0.5, 1.0, 1.4]), right_scale=rng.choice([0.5, 1.0, 1.4]), rank=rng.choice([2, 7, 16]),
                     scale=rng.choice([0.1, 0.4]), ff=ff)
        if kind == "parallel":
            layers.append(O.parallel_layer(chunk=rng.choice([0, 3, 16, 20, 50]), g_heads=rng.choice([1, 3]), g_dim=rng.choice([8, 20]),
                                           g_vdim=rng.choice([4, 18]), tau=rng.choice([1.0, 5.0, 16.0]), **heads))
        elif kind == "parallel_2":
            layers.append(O.parallel2_layer(conv=rng.choice([1, 2, 4, 5]), rot_dims=rng.choice([2, 4, 8]), base=rng.choice([100.0, 1e6]),
                                            softcap=rng.choice([2.0, 30.0]), r_heads=rng.choice([1, 3]), r_dim=rng.choice([6, 17]), **heads))
        else:
            groups = rng.choice([1, 2])
            layers.append(O.mamba_layer(heads=groups * rng.choice([1, 2, 3]), vdim=12, state=rng.choice([8, 20, 31]), groups=groups,
                                        conv=rng.choice([1, 2, 4]), norm_groups=rng.choice([1, 2, 3]), ff=ff))
    return O.make_config(layers=layers, width=rng.choice([24, 40, 60]), vocab=rng.choice([17, 50]), scale=rng.choice([1.0, 4.0]))


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


def _generate(path, dtype, prompts, outs, name):
    """The framework's own entry point: Engine + scheduler + worker protocol with graph replay. -> the generated tokens."""
    from swiftllm_amd import EngineConfig
    from swiftllm_amd.server import Engine, RawRequest
    ecfg = EngineConfig(model_path=path, use_dummy=False, block_size=16, gpu_mem_utilization=0.12, num_cpu_blocks=8,
                        max_seqs_in_block_table=4, max_blocks_per_seq=16, max_batch_size=4, max_tokens_in_batch=256,
                        dtype=dtype, use_hip_graph=True)

    async def run():
        engine = Engine(ecfg)
        await engine.initialize()
        assert type(engine.model).__name__ == name
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
    return got


def test_greedy_generation_through_the_engine(tmp_path, default_case):
    """Whole prompts then decoding, requests of unequal length finishing at different times: the oracle's greedy tokens."""
    cfg, W, _, _, _ = default_case
    path = str(tmp_path / "m")
    O.write_checkpoint(path, cfg, W)
    prompts = [tokens_for(cfg, n, 20 + n) for n in (5, 43, 18)]
    outs = (6, 12, 9)
    Wd = f64(W)
    got = _generate(path, "float32", prompts, outs, "VafozenModel")
    for g, p, n in zip(got, prompts, outs):
        seq = list(p)
        for _ in range(n):
            lg = O.forward(cfg, Wd, seq)[-1]
            top2 = torch.topk(lg, 2).values
            assert float(top2[0] - top2[1]) > 1e-4, "the test's weights make a close call"
            seq.append(int(torch.argmax(lg)))
        assert g == seq[len(p):]


def test_greedy_generation_in_bfloat16(tmp_path):
    """The default serving path (bfloat16, packed decode weights, graph replay, the argmax kernel): every generated token is the
    oracle's choice for the same prefix, or ties with it within what bfloat16 can tell apart."""
    cfg = matrix_core_config(256, vocab=512)
    W = O.random_weights(cfg, 23)
    path = str(tmp_path / "m")
    O.write_checkpoint(path, cfg, W)
    prompts = [tokens_for(cfg, n, 20 + n) for n in (5, 43, 18)]
    outs = (6, 12, 9)
    exact = total = 0
    for g, p, n in zip(_generate(path, "bfloat16", prompts, outs, "VafozenModel"), prompts, outs):
        assert len(g) == n
        lg = O.forward(cfg, f64(W), p + g)[len(p) - 1:-1]
        spread = float(lg.std())
        for t in range(n):
            assert float(lg[t].max() - lg[t][g[t]]) < 4 * BF16_TOL * spread
            exact += int(torch.argmax(lg[t])) == g[t]
            total += 1
    assert exact >= 0.8 * total


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
    path = str(tmp_path / "m")
    O.write_checkpoint(path, cfg, W)
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
                        str(out), "--max-tokens", "320"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.split("\n") if x.startswith("done ")] == [f"done {n}" for n in range(len(schedule))]
    logits = {k: O.forward(cfg, f64(W), t) for k, t in reqs.items()}
    got = [np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"]) for n in range(len(schedule))]
    assert sum(len(g) for g in got) == len(asked)
    got = torch.from_numpy(np.concatenate(got))
    want = torch.stack([logits[k][p] for _, k, p in asked])
    assert close(got, want, dtype)
