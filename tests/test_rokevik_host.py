"""Host-side pieces of the Rokevik worker (no GPU): the configuration reader, the registry, the order of layer runs, rotary
frequencies, the plan's chunks, the block and slot layout, and the plain implementation's own mechanisms against closed forms."""
import json
import math

import numpy as np
import pytest
import torch

import rokevik_oracle as O
from swiftllm_amd import registry
from swiftllm_amd.model_config import RokevikModelConfig, RotaryConfig
from swiftllm_amd.worker.batch_plan import StepEntry, StepPlan, plan_step


def test_config_reads_every_layer():
    layers = [O.min_gru_layer(width=72, mlp=O.moe(ff=20, experts=7, top=3, shared=0)),
              O.attention_layer(heads=6, kv_heads=3, dim=24, rot_dims=12, base=77.0, scale=0.3, softcap=None, mlp=None),
              O.latent_layer(heads=5, dim=14, rot_dim=6, vdim=18, kv_rank=30, window=None, factor=None)]
    cfg = RokevikModelConfig(O.make_config(layers=layers, width=60, vocab=37, eps=1e-4, groups=4, streams=None, loop=None,
                                           logit_softcap=None))
    assert (cfg.hidden_size, cfg.vocab_size, cfg.norm_eps, cfg.norm_groups) == (60, 37, 1e-4, 4)
    assert (cfg.num_streams, cfg.logit_softcap, cfg.has_state) == (0, 0.0, True)
    assert cfg.max_position_embeddings == cfg.DEFAULT_MAX_POSITIONS
    gru, att, lat = (l.mixer for l in cfg.layers)
    assert gru.width == 72
    m = cfg.layers[0].mlp
    assert (m.ffn_inter_dim, m.num_experts, m.top_k, m.shared_ffn_inter_dim) == (20, 7, 3, 0)
    assert (att.q_size, att.k_size, att.v_size, att.o_size, att.softcap, att.scale) == (144, 72, 72, 144, 0.0, 0.3)
    assert (att.rot.dims, att.rot.base, att.rot.half, att.rot.multiplier) == (12, 77.0, True, 1.0)
    assert (lat.q_size, lat.dkv_size, lat.k_size, lat.v_size, lat.o_size, lat.window) == (100, 36, 36, 30, 90, 0)
    assert cfg.layers[1].mlp is None and [r.layer for r in cfg.layer_runs] == [0, 1, 2]
    full = RokevikModelConfig(O.make_config())
    assert (full.num_streams, full.logit_softcap, full.layers[1].mixer.softcap) == (3, 12.0, 20.0)
    assert full.layers[0].mixer.window == 24 and full.layers[0].mixer.rot.scaling == (4.0, 64.0, 16.0, 1.0)
    # every run of a looped layer has a cache of its own
    assert full.kv_elems_per_token() == (28 + 20) + 2 * (32 + 32) + (28 + 20)


def test_config_refuses_what_cannot_run():
    for layers, kw in (([O.attention_layer(heads=3, kv_heads=2)], {}),
                       ([O.attention_layer(dim=16, rot_dims=20)], {}),
                       ([O.attention_layer(dim=16, rot_dims=7)], {}),
                       ([O.attention_layer(mlp=O.moe(experts=3, top=4))], {}),
                       ([O.attention_layer()], {"groups": 5}),
                       ([O.attention_layer()], {"streams": 17}),
                       ([O.attention_layer()], {"loop": (0, 2, 2)})):
        with pytest.raises(ValueError):
            RokevikModelConfig(O.make_config(layers=layers, loop=kw.pop("loop", None), **kw))
    bad = O.make_config(layers=[O.attention_layer()], loop=None)
    bad["layers"][0]["mixer"]["vdim"] = 20         # the values are the keys
    with pytest.raises(ValueError):
        RokevikModelConfig(bad)
    bad = O.make_config(layers=[O.latent_layer()], loop=None)
    bad["layers"][0]["mixer"]["rot"]["dims"] = 4   # the rotated part is rotated whole
    with pytest.raises(ValueError):
        RokevikModelConfig(bad)
    for key, value in (("type", "delta"), ("mlp", {"kind": "dense", "ff": 8})):
        bad = O.make_config(loop=None)
        bad["layers"][0][key] = value
        with pytest.raises(ValueError):
            RokevikModelConfig(bad)


@pytest.mark.parametrize("loop,order", [(None, [0, 1, 2, 3]), ((0, 4, 1), [0, 1, 2, 3]), ((1, 3, 3), [0, 1, 2, 1, 2, 1, 2, 3]),
                                        ((3, 4, 2), [0, 1, 2, 3, 3]), ((0, 2, 2), [0, 1, 0, 1, 2, 3])])
def test_order_of_layer_runs(loop, order):
    cfg = O.make_config(loop=loop)
    runs = RokevikModelConfig(cfg).layer_runs
    assert [r.layer for r in runs] == order == O.layer_order(cfg)
    assert [r.index for r in runs] == list(range(len(order)))


def test_registry_knows_the_design(tmp_path):
    cfg = O.make_config()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert registry.architecture_of(cfg) == "Rokevik"
    assert isinstance(registry.load_model_config(str(tmp_path)), RokevikModelConfig)
    assert registry.MODELS["Rokevik"][1].endswith(":RokevikModel")
    from swiftllm_amd.csrc import build
    assert {"hyper_stream.hip", "min_gru.hip", "moe.hip", "rope_kv.hip"} <= set(build.MODEL_SOURCES["Rokevik"])
    assert set(build.MODEL_SOURCES["Rokevik"]) <= set(build.SOURCES)


def test_checkpoint_names_and_shapes_round_trip(tmp_path):
    from swiftllm_amd.worker.kekapel_weight import _checkpoint_getter
    cfg = O.make_config()
    W = O.random_weights(cfg, 0)
    O.write_checkpoint(str(tmp_path), cfg, W)
    get = _checkpoint_getter(str(tmp_path))
    for name, shape in O.tensor_shapes(cfg).items():
        assert torch.equal(get(name, shape).float(), W[name])


def test_the_loader_asks_for_every_tensor_of_the_checkpoint_and_no_other():
    from swiftllm_amd.worker.rokevik_weight import RokevikWeight
    for cfg in (O.make_config(), O.make_config(streams=None, loop=None)):
        W, seen = O.random_weights(cfg, 1), set()

        def get(name, shape):
            assert tuple(W[name].shape) == tuple(shape), name
            seen.add(name)
            return W[name]
        RokevikWeight(RokevikModelConfig(cfg), torch.float32).load(get, torch.device("cpu"))
        assert seen == set(W)


# ---- rotation ----------------------------------------------------------------------------------------------------------------
def test_frequencies_without_interpolation_are_powers_of_the_base():
    rot = RotaryConfig({"dims": 8, "base": 625.0}, 8, half=True)
    assert rot.frequencies() == pytest.approx([1.0, 0.2, 0.04, 0.008])
    assert rot.multiplier == 1.0


def test_interpolated_frequencies_by_hand():
    # base e, so that the index of a dimension that turns t times over `original` positions is dims / 2 * ln(original / (2 pi t))
    sc = {"factor": 4.0, "original": 2 * math.pi * math.e ** 1.25, "fast": 1.0, "slow": math.e ** -1.0}
    rot = RotaryConfig({"dims": 8, "base": math.e, "scaling": sc}, 8, half=True)
    # dim(fast) = 4 * 1.25 = 5 -> lo = 5; dim(slow) = 4 * 2.25 = 9 -> hi = min(9, 7) = 7: every pair is below the ramp
    assert rot.frequencies() == pytest.approx([math.e ** (-i / 4) for i in range(4)])
    assert rot.multiplier == pytest.approx(0.1 * math.log(4.0) + 1.0)
    sc = {"factor": 4.0, "original": 2 * math.pi * math.e ** 0.3, "fast": 1.0, "slow": math.e ** -0.4}
    rot = RotaryConfig({"dims": 8, "base": math.e, "scaling": sc}, 8, half=True)
    # dim(fast) = 1.2 -> 1, dim(slow) = 2.8 -> 3: pair 0 and 1 kept, pair 2 half way, pair 3 slowed down by the factor
    want = [1.0, math.e ** -0.25, math.e ** -0.5 * (0.5 / 4 + 0.5), math.e ** -0.75 / 4]
    assert rot.frequencies() == pytest.approx(want)
    assert O.rotary_frequencies({"dims": 8, "base": math.e, "scaling": sc})[0] == pytest.approx(want)
    # the lower end clips at 0, the upper at dims - 1; an empty ramp (lower above upper) keeps every pair
    sc = {"factor": 2.0, "original": 2 * math.pi, "fast": math.e, "slow": math.e ** -9.0}
    got = RotaryConfig({"dims": 8, "base": math.e, "scaling": sc}, 8, half=True).frequencies()
    assert got == pytest.approx([math.e ** (-i / 4) * (1 - 0.5 * i / 7) for i in range(4)])
    sc = {"factor": 2.0, "original": 2 * math.pi * math.e ** 5, "fast": 1.0, "slow": 1.0}
    got = RotaryConfig({"dims": 8, "base": math.e, "scaling": sc}, 8, half=True).frequencies()
    assert got == pytest.approx([math.e ** (-i / 4) for i in range(4)])


def test_half_rotation_by_hand():
    x = torch.arange(1.0, 7.0, dtype=torch.float64).view(1, 1, 6)
    rot = {"dims": 4, "base": 100.0}
    y = O.rotate_half(x, torch.tensor([3]), rot)[0, 0]
    a, b = 3.0, 3.0 * 100.0 ** -0.5
    assert y.tolist() == pytest.approx([1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b),
                                        3 * math.cos(a) + 1 * math.sin(a), 4 * math.cos(b) + 2 * math.sin(b), 5.0, 6.0])


# ---- the plain implementation against closed forms ---------------------------------------------------------------------------
def test_streams_by_hand():
    X = torch.tensor([[[1.0, 2.0]], [[10.0, 20.0]]])
    y = torch.tensor([[100.0, 200.0]])
    mix = torch.tensor([[2.0, 3.0], [5.0, 7.0]])        # [from, to]
    out = torch.tensor([0.5, 0.25])
    new = O.hyper_step(X, y, mix, out)
    assert new[0, 0].tolist() == [2 * 1 + 5 * 10 + 50, 2 * 2 + 5 * 20 + 100]
    assert new[1, 0].tolist() == [3 * 1 + 7 * 10 + 25, 3 * 2 + 7 * 20 + 50]


def test_norm_parts_have_their_own_scale():
    x = torch.tensor([[3.0, 3.0, 4.0, 4.0]])
    assert O.group_norm(x, torch.ones(4), 2, 0.0).tolist() == [[1.0, 1.0, 1.0, 1.0]]
    assert O.group_norm(x, torch.ones(4), 1, 0.0)[0, 0] == pytest.approx(3 / math.sqrt(12.5))
    assert O.group_norm(x, torch.ones(4), 2, 16.0)[0, 0] == pytest.approx(3 / 5)       # eps inside the root


def test_min_gru_by_hand():
    z = torch.tensor([[0.25], [0.5], [1.0]], dtype=torch.float64)
    u = torch.tensor([[1.5], [-1.0], [0.0]], dtype=torch.float64)
    S = O.min_gru_states(z, u)[:, 0].tolist()
    s1 = 0.25 * 2.0
    s2 = 0.5 * s1 + 0.5 / (1 + math.e)
    assert S == pytest.approx([s1, s2, 0.5])
    assert torch.allclose(O.min_gru_states(z[1:], u[1:], torch.tensor([s1], dtype=torch.float64))[:, 0],
                          torch.tensor(S[1:], dtype=torch.float64))


def test_experts_get_scaled_inputs_and_scores_are_not_renormalised():
    idx, w = O.route(torch.tensor([[0.0, 2.0, -1.0]]), 2)
    assert idx.tolist() == [[1, 0]] and w[0].tolist() == pytest.approx([1 / (1 + math.exp(-2.0)), 0.5])
    cfg = O.make_config(layers=[O.min_gru_layer(mlp=O.moe(ff=8, experts=2, top=2, shared=0))], loop=None)
    W = {k: v.double() for k, v in O.random_weights(cfg, 1).items()}
    h = torch.randn(3, 48, dtype=torch.float64, generator=torch.Generator().manual_seed(0))
    s = torch.sigmoid(h @ W["l0.mlp.router"].T)
    want = sum(O.expert(s[:, e:e + 1] * h, W, f"l0.mlp.e{e}.") for e in range(2))
    assert torch.allclose(O.moe_ff(h, W, "l0.mlp.", cfg["layers"][0]["mlp"]), want)


def test_window_and_softcap_of_the_plain_attention():
    m = O.causal(5, 2)
    assert m.tolist() == [[j in (i, i - 1) for j in range(5)] for i in range(5)]
    q = torch.tensor([[[1.0]], [[1.0]]], dtype=torch.float64)
    k = torch.tensor([[[3.0]], [[-1.0]]], dtype=torch.float64)
    v = torch.tensor([[[1.0]], [[0.0]]], dtype=torch.float64)
    o = O.softmax_heads(q, k, v, 0.5, O.causal(2), softcap=2.0, temp=torch.tensor([1.5], dtype=torch.float64))
    a, b = 2 * math.tanh(2.25 / 2), 2 * math.tanh(-0.75 / 2)
    assert float(o[1, 0, 0]) == pytest.approx(math.exp(a) / (math.exp(a) + math.exp(b)))
    assert float(o[0, 0, 0]) == 1.0


# ---- the step's plan and the layouts -----------------------------------------------------------------------------------------
def test_plan_cuts_portions_into_chunks():
    c = StepPlan.CHUNK
    lens = [1, c, c + 1, 3 * c, 2]
    plan = plan_step([StepEntry(i, [0] * n, 5 * i) for i, n in enumerate(lens)])
    assert plan.chunk_cnt.tolist() == [1, c, c, 1, c, c, c, 2]
    assert plan.chunk_row0.tolist() == (np.cumsum(plan.chunk_cnt) - plan.chunk_cnt).tolist()
    assert plan.seq_chunk0.tolist() == [0, 1, 2, 4, 7]
    buf = np.full(plan.packed_layout()[1], -1, dtype=np.int32)
    plan.pack_into(buf)
    at = {name: (off, n) for name, off, n in plan.packed_layout()[0]}
    off, n = at["seq_chunk0"]
    assert buf[off:off + n].tolist() == [0, 1, 2, 4, 7]


class _Layout:
    """The worker's block layout without a device or weights."""

    def __new__(cls, cfg, dtype):
        from swiftllm_amd.worker.rokevik_model import RokevikModel

        class Probe(RokevikModel):
            def __init__(self):
                self.model_config, self.dtype = RokevikModelConfig(cfg), dtype
                self.engine_config = type("E", (), {"block_size": 16})()
                self._layout_pool()
        return Probe()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_block_layout_has_a_slice_per_run(dtype):
    p = _Layout(O.make_config(loop=(0, 3, 3)), dtype)
    cfg, at = p.model_config, 0
    assert len(p.pool_slices) == sum(cfg.layers[r.layer].type != "mingru" for r in cfg.layer_runs) == 7
    for run in cfg.layer_runs:
        mx = cfg.layers[run.layer].mixer
        if mx.kind == "mingru":
            continue
        kd, vd = p.row_sizes[run.index]
        need = (mx.k_size, mx.v_size) if mx.kind == "latent_attention" else (mx.head_dim, mx.value_dim)
        assert kd >= need[0] and vd >= need[1]
        if dtype == torch.float32:
            assert (kd, vd) == need
        sl = p.pool_slices[run.index]
        assert sl.k_offset == at and sl.k_offset % 8 == 0 and sl.v_offset == at + mx.num_kv_heads * kd * 16
        at = sl.v_offset + mx.num_kv_heads * vd * 16
        at += -at % 8
    assert p.block_elems == at


def test_padded_row_sizes():
    from swiftllm_amd import _hip
    from swiftllm_amd.worker.kernels.window_attn import served_row_sizes
    lib = _hip.load()
    for dim, vdim in ((64, 64), (128, 128), (576, 512)):        # served as they are
        assert served_row_sizes(dim, vdim, torch.bfloat16) == (dim, vdim)
    for dim, vdim in ((16, 16), (40, 40), (80, 80), (112, 96), (200, 176), (33, 30)):
        kd, vd = served_row_sizes(dim, vdim, torch.bfloat16)
        assert kd >= dim and vd >= vdim and lib.swl_masked_attn_tiles_supported(4, 2, 2, kd, vd, 1)
        assert kd + vd <= 2.5 * (dim + vdim)
        assert served_row_sizes(dim, vdim, torch.float32) == (dim, vdim)
    assert served_row_sizes(4, 4, torch.bfloat16) == (4, 4)      # padding would cost too much: the plain kernel serves it
    assert served_row_sizes(1000, 900, torch.bfloat16) == (1000, 900)
