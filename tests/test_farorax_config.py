"""Farorax on the CPU: its configuration, its specs, its tensors, what its runs ask of the cache manager,
the stretched frequencies, and the plain implementation held to a few closed forms."""
import copy
import math

import numpy as np
import pytest
import torch

from tests.farorax_helpers import CONFIGS, FARORAX_A, FARORAX_B, FARORAX_C, FARORAX_D, FARORAX_E, make_folder, read_folder
from tests.plain import farorax as plain


def parsed(raw):
    from pylon_amd.config.registry import resolve

    arch = resolve(raw)
    return arch, arch.parse_config(raw)


def test_config_json_selects_the_architecture_and_round_trips():
    for raw in CONFIGS.values():
        arch, cfg = parsed(raw)
        assert arch.name == "Farorax"
        assert arch.parse_config(arch.config_to_json(cfg)) == cfg
    _, cfg = parsed(FARORAX_A)
    assert cfg.runs() == ((0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None))
    assert cfg.residual_mult == 0.7 and cfg.logit_softcap == 15.0 and cfg.layers[2].mlp is None
    assert cfg.layers[1].mixer.rot.scaling == (4.0, 1.0, 4.0, 24.0) and cfg.layers[3].mixer.rot.scaling is None
    assert cfg.layers[1].mlp.groups == 3 and cfg.layers[1].mlp.keep == 2 and cfg.layers[1].mlp.shared_ff == 12
    _, cfg = parsed(FARORAX_B)
    assert [i for i, _ in cfg.runs()] == [0, 1, 2, 3, 2, 3, 2, 3] and [t for _, t in cfg.runs()][2::2] == [0, 1, 2]
    _, cfg = parsed(FARORAX_D)
    assert cfg.loop is None and cfg.logit_softcap is None and cfg.layers[1].mixer.rot is None and cfg.layers[4].mixer.mask_size is None
    null = dict(copy.deepcopy(FARORAX_D), loop=None, logit_softcap=None)
    assert parsed(null)[1] == cfg
    bare = copy.deepcopy(FARORAX_D)
    del bare["residual_mult"]
    assert parsed(bare)[1] == cfg


def test_layers_become_specs_of_parts_that_other_designs_can_use():
    from pylon_amd.config.specs import (AttentionSpec, GatedFeedForwardSpec, LightningAttentionSpec, MixtureFeedForwardSpec,
                                        PassEntrySpec, RotaryBandScalingSpec)

    arch, cfg = parsed(FARORAX_A)
    spec = arch.model_spec(cfg)
    assert [(e.layer, e.begins_pass) for e in spec.schedule] == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert spec.pass_entry == PassEntrySpec(dim=40, times=2) and not spec.tie_word_embeddings
    assert spec.logit_parts[0].cap == 15.0
    assert all(layer.arrangement == "pre_norm" and layer.residual_factor == 0.7 for layer in spec.layers)
    attention = spec.layers[1].mixer
    assert isinstance(attention, AttentionSpec) and attention.sink and attention.window == 7 and attention.chunk is None
    assert attention.value_dim == 14 and attention.position.interleaved and attention.position.rotary_dim == 6
    assert attention.position.scaling == RotaryBandScalingSpec(4.0, 1.0, 4.0, 24.0)
    lightning = spec.layers[0].mixer
    assert isinstance(lightning, LightningAttentionSpec) and (lightning.n_heads, lightning.head_dim, lightning.v_head_dim) == (3, 12, 20)
    assert lightning.norm_eps == 2e-5 and len(lightning.decay) == 3
    assert isinstance(spec.layers[0].feed_forward, GatedFeedForwardSpec) and spec.layers[0].feed_forward.activation == "gelu_tanh"
    moe = spec.layers[1].feed_forward
    assert isinstance(moe, MixtureFeedForwardSpec) and moe.scoring == "sigmoid" and moe.renormalize and moe.group_score == "top2"
    assert (moe.groups, moe.groups_kept, moe.shared_size, moe.shared_gate) == (3, 2, 12, False)
    assert spec.layers[2].feed_forward is None and spec.layers[2].feed_forward_norm is None
    arch, cfg = parsed(FARORAX_D)
    spec = arch.model_spec(cfg)
    assert spec.pass_entry is None and spec.logit_parts == () and spec.layers[1].mixer.position.kind == "none"


def _changed(path, value):
    def change(raw):
        node = raw
        for key in path[:-1]:
            node = node[key]
        if value is KeyError:
            del node[path[-1]]
        else:
            node[path[-1]] = value
    return change


@pytest.mark.parametrize("change, message", [
    (_changed(("layers", 0, "type"), "retention"), "unknown layer type"),
    (_changed(("layers", 0, "mixer", "decay"), [0.5, 0.5]), "decay must hold 3"),
    (_changed(("layers", 0, "mixer", "decay"), [0.5, 0.5, 1.5]), "from 0 to 1"),
    (_changed(("layers", 1, "mixer", "kv_heads"), 3), "divisible"),
    (_changed(("layers", 1, "mixer", "rot", "dims"), 5), "must be even"),
    (_changed(("layers", 1, "mixer", "rot", "dims"), 12), "at most the head's"),
    (_changed(("layers", 1, "mixer", "rot", "scaling", "low"), KeyError), "lacks required keys"),
    (_changed(("layers", 1, "mixer", "rot", "scaling", "low"), 4.0), "less than high"),
    (_changed(("layers", 1, "mixer", "mask", "size"), 0), "positive integer"),
    (_changed(("layers", 1, "mlp", "router", "groups", "count"), 4), "equal groups"),
    (_changed(("layers", 1, "mlp", "router", "groups", "keep"), 4), "are kept"),
    (_changed(("layers", 1, "mlp", "router", "top"), 5), "exceeds the 4 experts"),
    (_changed(("layers", 0, "mlp", "kind"), "plain"), "unknown feed-forward kind"),
    (_changed(("layers", 0, "mlp", "ff"), KeyError), "lacks required keys"),
    (_changed(("loop", "stop"), 5), "not a stretch"),
    (_changed(("loop", "times"), 0), "positive integer"),
    (_changed(("logit_softcap",), -1.0), "positive"),
    (_changed(("norm",), KeyError), "lacks required keys"),
    (_changed(("layers",), []), "no layers"),
])
def test_bad_configurations_are_refused(change, message):
    raw = copy.deepcopy(FARORAX_A)
    change(raw)
    with pytest.raises(ValueError, match=message):
        parsed(raw)


def test_parts_refuse_what_their_kernels_do_not_cover():
    from dataclasses import replace

    from pylon_amd.config.specs import (GatedFeedForwardSpec, LayerSpec, LightningAttentionSpec, MixtureFeedForwardSpec,
                                        NormSpec, PassEntrySpec)
    from pylon_amd.parts import build_part

    kw = dict(dtype=torch.float32, device="cpu")
    linear = LightningAttentionSpec(hidden_size=32, n_heads=2, head_dim=8, v_head_dim=8, decay=(0.5, 0.9), norm_eps=1e-6)
    build_part("mixer", linear, **kw)
    for change in (dict(decay=(0.5,)), dict(v_head_dim=300), dict(head_dim=2000)):
        with pytest.raises(ValueError):
            build_part("mixer", replace(linear, **change), **kw)
    moe = MixtureFeedForwardSpec(hidden_size=32, n_experts=8, top=2, expert_size=16, shared_gate=False, router_bias=False,
                                 scoring="sigmoid", groups=4, groups_kept=2, group_score="top2", renormalize=True)
    build_part("feed_forward", moe, **kw)
    for change, message in ((dict(groups=3), "equal groups"), (dict(top=5), "do not hold"), (dict(group_score="mean"), "score of a group"),
                            (dict(scoring="top_softmax"), "belong to"), (dict(n_identity=2), "identity"),
                            (dict(shared_size=8, shared_gate=True), "plain ways")):
        with pytest.raises(ValueError, match=message):
            build_part("feed_forward", replace(moe, **change), **kw)
    gated = GatedFeedForwardSpec(hidden_size=8, intermediate_size=8, activation="gelu_tanh")
    build_part("feed_forward", gated, **kw)
    for change in (dict(activation="gelu"), dict(bias=True)):
        with pytest.raises(ValueError):
            build_part("feed_forward", replace(gated, **change), **kw)
    norm = NormSpec(kind="rmsnorm", dim=32, eps=1e-6)
    layer = LayerSpec(mixer=linear, feed_forward=None, mixer_norm=norm, feed_forward_norm=None, residual_factor=0.5)
    build_part("block", layer, **kw)
    for change in (dict(depth_mix=(1, 3)), dict(arrangement="hyper_connections"), dict(arrangement="sandwich_norm", mixer_post_norm=norm)):
        with pytest.raises(ValueError, match="factor"):
            build_part("block", replace(layer, **change), **kw)
    with pytest.raises(ValueError):
        build_part("pass", PassEntrySpec(dim=8, times=0), **kw)


def test_a_schedule_whose_passes_have_no_entry_part_is_refused():
    from dataclasses import replace

    from pylon_amd.engine.model import Model

    arch, cfg = parsed(FARORAX_A)
    spec = arch.model_spec(cfg)
    with pytest.raises(ValueError, match="pass_entry"):
        Model(replace(spec, pass_entry=None), dtype=torch.float32, device="cpu")
    far = tuple(replace(e, begins_pass=2 if e.begins_pass == 1 else e.begins_pass) for e in spec.schedule)
    with pytest.raises(ValueError, match="numbered"):
        Model(replace(spec, schedule=far), dtype=torch.float32, device="cpu")


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_written_folder_loads_into_every_parameter(tmp_path, name):
    from pylon_amd.config.registry import load_model_config
    from pylon_amd.engine.model import Model
    from pylon_amd.weights.loader import load_weights

    folder = make_folder(tmp_path, name)
    arch, cfg = load_model_config(folder)
    model = Model(arch.model_spec(cfg), dtype=torch.float32, device="cpu")
    for _path, owner, pname in model.named_params():
        owner.params[pname].fill_(float("nan"))
    assert load_weights(model, arch, cfg, folder, strict=True) == []
    for path, owner, pname in model.named_params():
        assert not torch.isnan(owner.params[pname]).any(), path
    _cfg, weights = read_folder(folder)
    if name == "A":
        same = lambda tensor, name: np.array_equal(tensor.numpy(), weights[name].astype(np.float32))  # noqa: E731
        linear = model.blocks[0].mixer
        assert linear.params["qkvg"].shape == (36 + 36 + 60 + 60, 40)
        assert same(linear.params["qkvg"][36: 72], "l0.mix.k") and same(linear.params["qkvg"][linear.gate_off:], "l0.mix.g")
        assert same(linear.params["norm"], "l0.mix.norm")
        attention = model.blocks[1].mixer
        assert same(attention.params["qkv"][40: 60], "l1.mix.k") and same(attention.params["sink"], "l1.mix.sink")
        moe = model.blocks[1].feed_forward
        assert same(moe.params["gate_up"][2 * 32 + 16: 2 * 32 + 32], "l1.mlp.e2.up")
        assert same(moe.params["shared_gate_up"][:12], "l1.mlp.shared.gate") and same(moe.params["down"][40: 80], "l1.mlp.e1.down")
        assert same(model.pass_entry.params["join"], "loop.in") and same(model.pass_entry.params["step"], "loop.step")
        assert "l2.norm2" not in weights and model.blocks[2].feed_forward is None


def test_a_folder_that_lacks_a_tensor_or_holds_one_too_many_is_refused(tmp_path):
    from safetensors.torch import load_file, save_file

    from pylon_amd.config.registry import load_model_config
    from pylon_amd.engine.model import Model
    from pylon_amd.weights.loader import WeightsError, load_weights

    folder = make_folder(tmp_path, "A")
    arch, cfg = load_model_config(folder)
    tensors = load_file(str(folder / "model.safetensors"))
    tensors["l0.mix.sink"] = tensors.pop("l1.mix.sink")
    save_file(tensors, str(folder / "model.safetensors"))
    model = Model(arch.model_spec(cfg), dtype=torch.float32, device="cpu")
    with pytest.raises(WeightsError) as error:
        load_weights(model, arch, cfg, folder, strict=True)
    assert "l0.mix.sink" in str(error.value) and "l1.mix.sink" in str(error.value)


def test_every_run_asks_for_keys_and_values_or_a_state_of_its_own():
    from pylon_amd.cache.manager import CacheManager
    from pylon_amd.engine.model import Model
    from pylon_amd.parts.base import KVRequirement, StateRequirement

    arch, cfg = parsed(FARORAX_A)
    needs = Model(arch.model_spec(cfg), dtype=torch.float32, device="cpu").cache_requirements()
    first, looped = StateRequirement((3, 12, 20), torch.float32), StateRequirement((2, 20, 6), torch.float32)
    window = KVRequirement(2, 10, 7, v_head_dim=14)
    assert needs == [first, window, looped, window, looped, KVRequirement(3, 12, 5, v_head_dim=8)]
    manager = CacheManager(needs, dtype=torch.float32, page_size=16, num_pages=6, max_requests=2, device="cpu")
    seq = manager.open("a")
    assert manager.view(2).state.data_ptr() != manager.view(4).state.data_ptr()
    assert manager.view(1).k.data_ptr() != manager.view(3).k.data_ptr()
    for tensor in manager.slots.tensors.values():
        tensor.fill_(7.0)
    manager.close(seq)
    again = manager.open("b")  # a slot that is handed out again starts from zeros
    for key, tensor in manager.slots.tensors.items():
        assert float(tensor[again.slot].abs().max()) == 0.0, key


def test_stretches_of_chunks_fill_the_units():
    from pylon_amd.kernels import ops

    span = lambda rows, heads, n: ops.retention_chunk_span(rows, heads, n, units=256)  # noqa: E731
    assert [span(1, 10, 2048), span(1, 16, 2048), span(1, 32, 2048), span(1, 10, 8192), span(1, 10, 512)] == [3, 4, 4, 6, 1]
    for heads in (1, 3, 10, 40, 100):
        for n in (130, 2048, 20000):
            s = span(1, heads, n)
            assert 1 <= s <= -(-n // 32)
            assert heads * -(-(-(-n // 32)) // s) <= 3 * 256
    assert ops.retention_chunk_parallel(1, 10, 128, 128, 2048, units=256) and not ops.retention_chunk_parallel(1, 10, 128, 128, 96, units=256)


# ---- the stretched frequencies ---------------------------------------------------------------------

@pytest.mark.parametrize("base, dims, scaling", [(500.0, 16, (4.0, 1.0, 4.0, 24)), (1.0e4, 64, (8.0, 1.0, 4.0, 256)),
                                                  (3.0e5, 32, (2.0, 1.5, 8.0, 64)), (777.0, 2, (3.0, 2.0, 6.0, 20))])
def test_frequencies_stretched_by_wavelength(base, dims, scaling):
    from pylon_amd.config.specs import PositionSpec, RotaryBandScalingSpec
    from pylon_amd.parts import build_part

    spec = PositionSpec(kind="rope", theta=base, rotary_dim=dims, interleaved=True, scaling=RotaryBandScalingSpec(*scaling))
    part = build_part("position", spec, dtype=torch.float32, device="cpu")
    rot = {"base": base, "dims": dims, "scaling": dict(zip(("factor", "low", "high", "original"), scaling))}
    want = plain.frequencies(rot)
    got, count = part.rotary()
    assert count == dims and part.rot_scale == 1.0 and part.interleaved
    assert np.allclose(got.double().numpy(), want, rtol=1e-7, atol=0.0)
    unscaled = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    ratio = want / unscaled
    if dims >= 32:  # all three kinds of pairs are there
        assert (ratio == 1.0).any() and np.isclose(ratio, 1.0 / scaling[0]).any() and ((ratio < 0.999) & (ratio > 1.001 / scaling[0])).any()


def test_frequencies_at_the_two_edges_of_the_band():
    """Just outside ``original / high`` a frequency stays, just outside ``original / low`` it is divided; the
    blend meets both without a jump."""
    from pylon_amd.config.specs import PositionSpec, RotaryBandScalingSpec
    from pylon_amd.parts.position import band_frequencies

    for turns, want in ((5.001, 1.0), (4.999, 1.0), (2.001, 0.25), (1.999, 0.25), (3.5, 0.625)):
        original = turns * 2.0 * math.pi  # the first pair turns at 1
        spec = PositionSpec(kind="rope", theta=100.0, rotary_dim=2, interleaved=True,
                            scaling=RotaryBandScalingSpec(4.0, 2.0, 5.0, original))
        assert abs(float(band_frequencies(spec)[0]) - want) < 1e-3
    with pytest.raises(ValueError):
        band_frequencies(PositionSpec(kind="rope", theta=100.0, rotary_dim=2, scaling=RotaryBandScalingSpec(4.0, 5.0, 2.0, 9)))


# ---- the plain implementation against closed forms --------------------------------------------------

def test_plain_activations_and_norm():
    assert abs(plain.gelu_tanh(np.array(1.0)) - 0.5 * (1 + math.tanh(math.sqrt(2 / math.pi) * 1.044715))) < 1e-15
    assert plain.gelu_tanh(np.array(0.0)) == 0.0 and abs(plain.silu(np.array(2.0)) - 2 / (1 + math.exp(-2))) < 1e-15
    assert np.allclose(plain.norm(np.array([[3.0, 4.0]]), np.array([1.0, 2.0]), 0.0), np.array([[3.0, 8.0]]) / math.sqrt(12.5))


def test_plain_rotation_pairs_neighbours_and_leaves_the_rest():
    x = np.arange(2 * 1 * 6, dtype=np.float64).reshape(2, 1, 6) + 1.0
    got = plain.rotate_pairs(x, {"base": 100.0, "dims": 4})
    assert np.array_equal(got[0], x[0]) and np.array_equal(got[1, 0, 4:], x[1, 0, 4:])
    a, (u, v) = 100.0 ** -0.5, x[1, 0, 2:4]
    assert np.allclose(got[1, 0, 2:4], [u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a)])


def test_plain_window_and_sink():
    seen = plain.window_mask(7, 3)
    assert seen[5].tolist() == [False, False, False, True, True, True, False] and seen[1].tolist()[:3] == [True, True, False]
    assert plain.window_mask(4, 1).astype(int).tolist() == np.eye(4, dtype=int).tolist() and plain.window_mask(4, None)[3].all()
    # one key of score 0 and a sink of ln 3: the key keeps a quarter of the weight
    assert np.allclose(plain.softmax_with_sink(np.zeros((1, 1)), np.ones((1, 1), bool), math.log(3.0)), 0.25)


def test_plain_state_fades_by_head_and_reads_its_own_write():
    q, k = np.ones((3, 2, 1)), np.ones((3, 2, 1))
    v = np.array([2.0, 3.0, 4.0]).reshape(3, 1, 1).repeat(2, axis=1)
    out = plain.decayed_state(q, k, v, [0.5, 0.0])
    assert np.allclose(out[:, 0, 0], [2.0, 4.0, 6.0]) and np.allclose(out[:, 1, 0], [2.0, 3.0, 4.0])


def test_plain_routing_chooses_from_the_best_groups_by_their_two_best():
    # group 0 holds the largest score but a poor second; group 1's two together are larger
    z = np.log(np.array([[0.9, 0.1, 0.6, 0.55]]) / (1 - np.array([[0.9, 0.1, 0.6, 0.55]])))
    margins = []
    experts, weights = plain.route(np.ones((1, 1)), {"router": z.T}, "", {"experts": 4, "top": 2, "groups": {"count": 2, "keep": 1}}, margins)
    assert experts.tolist() == [[2, 3]] and np.allclose(weights, [[0.6 / 1.15, 0.55 / 1.15]]) and np.isclose(margins[0][0], 0.15)
    experts, weights = plain.route(np.ones((1, 1)), {"router": z.T}, "", {"experts": 4, "top": 3})
    assert experts.tolist() == [[0, 2, 3]] and np.isclose(weights.sum(), 1.0)


def test_plain_order_of_runs_and_pass_entry():
    assert plain.layer_runs(FARORAX_B) == [(0, None), (1, None), (2, 0), (3, None), (2, 1), (3, None), (2, 2), (3, None)]
    assert plain.layer_runs(FARORAX_C) == [(0, 0), (1, None), (0, 1), (1, None)]
    assert plain.layer_runs(FARORAX_E) == [(0, 0), (1, None)]  # one pass has its entry too
    w = {"loop.in": np.array([[1.0, 0.0, 10.0, 0.0], [0.0, 1.0, 0.0, 10.0]]), "loop.step": np.array([[0.0, 0.0], [5.0, 7.0]])}
    assert plain.enter_pass(np.array([[1.0, 2.0]]), np.array([[3.0, 4.0]]), w, 1).tolist() == [[36.0, 49.0]]


def test_plain_forward_in_two_cuts_agrees_on_the_common_positions(tmp_path):
    for name in ("A", "E"):
        cfg, weights = read_folder(make_folder(tmp_path, name))
        toks = list(range(3, 40))
        whole, kept = plain.forward(cfg, weights, toks, keep_layers=True)
        assert np.allclose(plain.forward(cfg, weights, toks[:21]), whole[:21], atol=1e-9)
        assert kept.shape == (len(plain.layer_runs(cfg)), len(toks), cfg["width"])
