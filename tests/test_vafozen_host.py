"""Host-side pieces of the Vafozen worker (no GPU): the configuration reader, the registry, the weight loader and its fused matrices,
the plan's tiles, the block layout, the library's completeness check, and the plain implementation's own mechanisms against closed
forms."""
import json
import math
import subprocess

import pytest
import torch

import vafozen_oracle as O
from swiftllm_amd import registry
from swiftllm_amd.model_config import VafozenModelConfig
from swiftllm_amd.worker.batch_plan import StepEntry, StepPlan, plan_step


def test_config_reads_every_layer():
    layers = [O.mamba_layer(heads=6, vdim=10, state=14, groups=3, conv=5, norm_groups=4, ff=0),
              O.parallel_layer(heads=6, kv_heads=2, dim=20, vdim=28, chunk=37, scale=0.3, g_heads=5, g_dim=9, g_vdim=11, tau=7.0,
                               left_scale=0.25, right_scale=-2.0, ff=24),
              O.parallel2_layer(heads=4, kv_heads=4, dim=24, vdim=8, conv=6, rot_dims=10, base=77.0, scale=0.11, softcap=3.5,
                                r_heads=2, r_dim=13, left_scale=1.5, right_scale=0.5, ff=40)]
    cfg = VafozenModelConfig(O.make_config(layers=layers, width=60, vocab=37, eps=1e-4, scale=2.5))
    assert (cfg.hidden_size, cfg.vocab_size, cfg.norm_eps, cfg.embedding_scale) == (60, 37, 1e-4, 2.5)
    assert cfg.max_position_embeddings == cfg.DEFAULT_MAX_POSITIONS
    ssm, par, par2 = (l.mixer for l in cfg.layers)
    assert (ssm.inner, ssm.conv_channels, ssm.proj_size, ssm.state_elems) == (60, 60 + 2 * 42, 2 * 60 + 84 + 6, 6 * 14 * 10)
    assert (ssm.conv_taps, ssm.norm_groups) == (5, 4) and cfg.layers[0].mlp is None and cfg.layers[0].attention is None
    lf, rt = par.left, par.right
    assert (lf.q_size, lf.k_size, lf.v_size, lf.o_size, lf.chunk, lf.scale) == (120, 40, 56, 168, 37, 0.3)
    assert (lf.conv_taps, lf.softcap, lf.rot.dims) == (0, 0.0, 0)
    assert lf.slopes() == pytest.approx([2.0 ** (-8 * (h + 1) / 6) for h in range(6)])
    assert (rt.keys, rt.inner, rt.state_elems, rt.tau) == (45, 55, 5 * 9 * 11, 7.0)
    assert (par.left_scale, par.right_scale, cfg.layers[1].mlp.ffn_inter_dim) == (0.25, -2.0, 24)
    lf, rt = par2.left, par2.right
    assert (lf.conv_taps, lf.softcap, lf.chunk, lf.slopes()) == (6, 3.5, 0, None)
    assert (lf.rot.dims, lf.rot.base, lf.rot.half) == (10, 77.0, True)
    assert (rt.keys, rt.inner, rt.state_elems) == (26, 26, 2 * 13 * 13)
    assert cfg.kv_elems_per_token() == 40 + 56 + 96 + 32
    # a chunk, a convolution, a cap that config.json leaves out are off
    bare = O.make_config(layers=[O.parallel_layer(chunk=0), O.parallel2_layer()])
    del bare["layers"][1]["mixer"]["left"]["softcap"], bare["layers"][1]["mixer"]["left"]["conv"]
    a, b = (l.mixer.left for l in VafozenModelConfig(bare).layers)
    assert (a.chunk, b.softcap, b.conv_taps) == (0, 0.0, 0)


def test_config_refuses_what_cannot_run():
    for layer in (O.parallel_layer(heads=3, kv_heads=2), O.parallel_layer(tau=0.0), O.parallel_layer(tau=-1.0),
                  O.parallel2_layer(dim=16, rot_dims=20), O.parallel2_layer(dim=16, rot_dims=7), O.mamba_layer(heads=4, groups=3),
                  O.mamba_layer(heads=4, vdim=12, norm_groups=5)):
        with pytest.raises(ValueError):
            VafozenModelConfig(O.make_config(layers=[layer]))
    for key, value in (("type", "delta"), ("mlp", {"kind": "moe", "ff": 8})):
        bad = O.make_config()
        bad["layers"][0][key] = value
        with pytest.raises(ValueError):
            VafozenModelConfig(bad)
    with pytest.raises(AssertionError):
        VafozenModelConfig(dict(O.make_config(), architecture="Other"))


def test_registry_knows_the_design(tmp_path):
    cfg = O.make_config()
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert registry.architecture_of(cfg) == "Vafozen"
    assert isinstance(registry.load_model_config(str(tmp_path)), VafozenModelConfig)
    assert registry.MODELS["Vafozen"][1].endswith(":VafozenModel")
    from swiftllm_amd.csrc import build
    assert {"linear_scan.hip", "low_rank_decay.hip", "ssd.hip", "rope_kv.hip", "hyper_stream.hip"} <= set(build.MODEL_SOURCES["Vafozen"])
    assert set(build.MODEL_SOURCES["Vafozen"]) <= set(build.SOURCES)


def test_checkpoint_names_and_shapes_round_trip(tmp_path):
    from swiftllm_amd.worker.kekapel_weight import _checkpoint_getter
    cfg = O.make_config()
    W = O.random_weights(cfg, 0)
    O.write_checkpoint(str(tmp_path), cfg, W)
    get = _checkpoint_getter(str(tmp_path))
    for name, shape in O.tensor_shapes(cfg).items():
        assert torch.equal(get(name, shape).float(), W[name])


def _load(cfg, W, dtype=torch.float32):
    from swiftllm_amd.worker.vafozen_weight import VafozenWeight
    seen = set()

    def get(name, shape):
        have = tuple(W[name].shape)
        assert len(have) == len(shape) and all(b is None or a == b for a, b in zip(have, shape)), name
        seen.add(name)
        return W[name]
    weight = VafozenWeight(VafozenModelConfig(cfg), dtype)
    weight.load(get, torch.device("cpu"))
    return weight, seen


def test_the_loader_asks_for_every_tensor_of_the_checkpoint_and_no_other():
    for cfg in (O.make_config(), O.make_config(layers=[O.parallel2_layer(conv=1, ff=0), O.mamba_layer()])):
        W = O.random_weights(cfg, 1)
        assert _load(cfg, W)[1] == set(W)


@pytest.mark.parametrize("layer", [O.parallel_layer(g_vdim=7, ff=13), O.parallel2_layer(heads=3, kv_heads=1, vdim=5, ff=0),
                                   O.mamba_layer(heads=3, vdim=5, groups=1, norm_groups=1, ff=9)], ids=lambda l: l["type"])
def test_fused_matrices_hold_every_projection_once(layer):
    """The columns that a piece of the fused input product gets are that projection's, and the fused output product of the pieces is
    the sum of the projections; sizes that are no multiples of 8."""
    cfg = O.make_config(layers=[layer])
    W = O.random_weights(cfg, 2)
    lw = _load(cfg, W)[0].layers[0]
    h = torch.randn(3, cfg["width"], generator=torch.Generator().manual_seed(0))
    proj = h @ lw.proj.T
    left, right, mix, mlp = "l0.mix.left.", "l0.mix.right.", "l0.mix.", "l0.mlp."
    names = {"parallel": {"right_q": right + "q", "right_k": right + "k", "right_v": right + "v", "right_g": right + "g",
                          "decay": right + "a1", "ff_gate": mlp + "gate", "ff_up": mlp + "up"},
             "parallel_2": {"gate": left + "g"}, "mamba2": {"in": mix + "in", "ff_gate": mlp + "gate", "ff_up": mlp + "up"}}
    pieces = {k: W[v] for k, v in names[layer["type"]].items()}
    if layer["type"] != "mamba2":
        pieces["qkv"] = torch.cat([W[left + n] for n in "qkv"])
    assert set(pieces) == set(lw.cols)
    for name, w in pieces.items():
        assert lw.cols[name].start % 8 == 0 and torch.allclose(proj[:, lw.cols[name]], h @ w.T, atol=1e-5), name
    outs = {"left": left + "o", "right": right + "o", "mixer": mix + "o", "ff": mlp + "down"}
    row, want = torch.zeros(3, lw.row_size), 0
    for name, s in lw.ins.items():
        row[:, s] = torch.randn(3, s.stop - s.start, generator=torch.Generator().manual_seed(s.stop))
        want = want + row[:, s] @ W[outs[name]].T
        assert s.start % 8 == 0
    assert set(lw.ins) == {k for k, v in outs.items() if v in W}
    assert torch.allclose(row @ lw.out.T, want, atol=1e-5)
    assert lw.row_gaps == (sum(s.stop - s.start for s in lw.ins.values()) != lw.row_size)


def test_low_ranks_are_padded_with_zeros_in_16_bit_models():
    cfg = O.make_config(layers=[O.parallel_layer(rank=5), O.parallel2_layer(rank=20)])
    W = O.random_weights(cfg, 3)
    for dtype, want in ((torch.float32, (5, 20)), (torch.bfloat16, (16, 32))):
        a, b = _load(cfg, W, dtype)[0].layers
        assert (a.decay_2.shape[1], b.decay_2.shape[1]) == want
        assert (a.cols["decay"].stop - a.cols["decay"].start, b.decay_1.shape[0]) == want
        assert torch.equal(b.decay_2[:, :20].float(), W["l1.mix.right.w2"]) and not b.decay_2[:, 20:].any()
        assert torch.equal(b.decay_1[:20].float(), W["l1.mix.right.w1"]) and not b.decay_1[20:].any()


# ---- the plan and the layouts --------------------------------------------------------------------------------------------------
def test_plan_knows_every_portions_first_tile():
    T = StepPlan.TILE
    lens = [1, T, T + 1, 3 * T, 2]
    plan = plan_step([StepEntry(i, [0] * n, 5 * i) for i, n in enumerate(lens)])
    assert plan.seq_tile0.tolist() == [0, 1, 2, 4, 7]
    assert plan.tile_row0[plan.seq_tile0].tolist() == plan.seq_row0.tolist()
    for s, n in enumerate(lens):
        t0 = plan.seq_tile0[s]
        assert plan.tile_cnt[t0:t0 + -(-n // T)].sum() == n


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_block_layout_has_a_slice_per_attention(dtype):
    from swiftllm_amd.worker.vafozen_model import VafozenModel

    class Probe(VafozenModel):
        def __init__(self, cfg):
            self.model_config, self.dtype = VafozenModelConfig(cfg), dtype
            self.engine_config = type("E", (), {"block_size": 16})()
            self._layout_pool()
    p = Probe(O.make_config(layers=[O.parallel_layer(dim=10, vdim=7), O.mamba_layer(), O.parallel2_layer(dim=40, vdim=56)]))
    assert set(p.pool_slices) == {0, 2}
    at = 0
    for i in (0, 2):
        mx = p.model_config.layers[i].attention
        kd, vd = p.row_sizes[i]
        assert kd >= mx.head_dim and vd >= mx.value_dim and p.pool_slices[i].k_offset == at and at % 8 == 0
        assert p.pool_slices[i].v_offset == at + mx.num_kv_heads * kd * 16
        at = p.pool_slices[i].v_offset + mx.num_kv_heads * vd * 16
        at += -at % 8
    assert p.block_elems == at
    assert Probe(O.make_config(layers=[O.mamba_layer()])).block_elems == 8


def test_a_partial_or_outdated_library_is_noticed(tmp_path):
    from swiftllm_amd import _hip
    from swiftllm_amd.csrc import build
    assert set(build.entry_points(build.SOURCES)) == set(_hip.SIGNATURES) | set(_hip._SPECIAL)
    if _hip.is_available():
        assert build.serves(build.SOURCES)
    assert not build.serves(build.MODEL_SOURCES["Vafozen"], str(tmp_path / "none.so"))
    names = build.entry_points(["swap_blocks.hip", "linear_scan.hip"])
    for case, (version, have) in enumerate(((_hip.ABI_VERSION, names), (_hip.ABI_VERSION - 1, names), (_hip.ABI_VERSION, names[:-1]))):
        src, lib = tmp_path / f"l{case}.c", tmp_path / f"l{case}.so"
        src.write_text("".join(f"int {n}(void) {{ return {version}; }}\n" for n in have))
        subprocess.run(["gcc", "-shared", "-fPIC", str(src), "-o", str(lib)], check=True)
        assert build.serves(["swap_blocks.hip", "linear_scan.hip"], str(lib)) == (case == 0)


# ---- the plain implementation against closed forms -----------------------------------------------------------------------------
def test_convolution_by_hand():
    u, w = torch.tensor([[1.0], [10.0], [100.0]]), torch.tensor([[2.0, 3.0, 5.0]])
    assert O.causal_conv(u, w)[:, 0].tolist() == [5.0, 3 + 50.0, 2 + 30 + 500.0]       # the last tap is the current token's


def test_rotation_by_halves_by_hand():
    x = torch.arange(1.0, 7.0, dtype=torch.float64).view(1, 1, 6).repeat(4, 1, 1)
    a, b = 3.0, 3.0 * 100.0 ** -0.5
    assert O.rotate_halves(x, 4, 100.0)[3, 0].tolist() == pytest.approx(
        [1 * math.cos(a) - 3 * math.sin(a), 2 * math.cos(b) - 4 * math.sin(b), 3 * math.cos(a) + 1 * math.sin(a),
         4 * math.cos(b) + 2 * math.sin(b), 5.0, 6.0])


def test_scans_by_hand():
    q, k, v = (torch.tensor(x, dtype=torch.float64).view(3, 1, 1) for x in ([1.0, 2.0, 3.0], [5.0, 7.0, 11.0], [1.0, 10.0, 100.0]))
    a = torch.tensor([0.3, 0.5, 0.25], dtype=torch.float64).view(3, 1, 1)
    s = [5.0, 0.5 * 5 + 70, 0.25 * (0.5 * 5 + 70) + 1100]
    assert O.linear_scan(q, k, v, a).view(-1).tolist() == pytest.approx([1 * s[0], 2 * s[1], 3 * s[2]])
    # with the bonus the read-out comes first: the state of the tokens before, the current one times u
    u = torch.tensor([[0.1]], dtype=torch.float64)
    assert O.bonus_scan(q, k, v, a, u).view(-1).tolist() == pytest.approx([1 * 0.5, 2 * (5.0 + 7.0), 3 * (s[1] + 110.0)])


def test_chunks_and_slopes_by_hand():
    assert O.causal_mask(5, 2).tolist() == [[j <= i and j // 2 == i // 2 for j in range(5)] for i in range(5)]
    assert O.causal_mask(4).tolist() == [[j <= i for j in range(4)] for i in range(4)]
    assert [O.head_slope(h, 4) for h in range(4)] == [0.25, 0.0625, 0.015625, 0.00390625]


def test_norm_is_stored_around_zero():
    x = torch.tensor([[3.0, 4.0]])
    assert O.layer_norm1p(x, torch.tensor([0.0, 1.0]), 12.5)[0].tolist() == pytest.approx([3 / 5.0, 2 * 4 / 5.0])


def test_both_halves_read_the_same_norm():
    """x + mixer(h) + ff(h), not a feed-forward of the updated stream."""
    cfg = O.make_config(layers=[O.mamba_layer()])
    W = {k: v.double() for k, v in O.random_weights(cfg, 1).items()}
    toks, taps = [3, 1, 4, 1, 5], []
    O.forward(cfg, W, toks, taps)
    x = W["embed"][toks] * cfg["embedding"]["scale"]
    h = O.layer_norm1p(x, W["l0.norm1"], cfg["norm"]["eps"])
    want = x + O.state_space(h, W, "l0.mix.", cfg["layers"][0]["mixer"], cfg["norm"]["eps"]) + O.gated_unit(h, W, "l0.mlp.")
    assert torch.allclose(taps[0], want)
