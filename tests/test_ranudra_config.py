"""Ranudra on the CPU: its configuration, its specs, its tensors, what its runs ask of the
cache manager, and the plain implementation held to a few closed forms."""
import copy
import math

import numpy as np
import pytest
import torch

from tests.plain import ranudra as plain
from tests.ranudra_helpers import CONFIGS, RANUDRA_A, RANUDRA_B, RANUDRA_D, make_folder, read_folder


def test_config_json_selects_the_architecture_and_round_trips():
    from pylon_amd.config.registry import resolve

    for raw in CONFIGS.values():
        arch = resolve(raw)
        assert arch.name == "Ranudra"
        cfg = arch.parse_config(raw)
        assert arch.parse_config(arch.config_to_json(cfg)) == cfg
    cfg = resolve(RANUDRA_A).parse_config(RANUDRA_A)
    assert cfg.streams == 3 and cfg.embedding_scale == 5.0 and cfg.layers[1].ff is None and cfg.layers[0].ff == 28
    assert cfg.runs() == (0, 1, 2, 1, 2, 3)
    assert cfg.layers[2].mixer.rot.scaling == (4.0, 16.0, 4.0, 1.0) and cfg.layers[0].mixer.rot.scaling is None
    assert cfg.layers[1].mixer.tau == 4.0 and cfg.layers[1].mixer.decay_rank == 5
    assert resolve(RANUDRA_B).parse_config(RANUDRA_B).runs() == (0, 1, 2, 3, 2, 3, 2, 3)
    cfg = resolve(RANUDRA_D).parse_config(RANUDRA_D)
    assert cfg.loop is None and cfg.runs() == (0, 1, 2, 3) and cfg.layers[2].mixer.rot is None
    null = dict(copy.deepcopy(RANUDRA_D), loop=None)
    assert resolve(null).parse_config(null) == cfg


def test_layers_become_specs_of_parts_that_other_designs_can_use():
    from pylon_amd.config.registry import resolve
    from pylon_amd.config.specs import GatedLinearAttentionSpec, LatentAttentionSpec, PlainFeedForwardSpec

    arch = resolve(RANUDRA_A)
    spec = arch.model_spec(arch.parse_config(RANUDRA_A))
    assert [(e.layer, e.cache, e.add_embedding) for e in spec.schedule] == [(i, None, False) for i in (0, 1, 2, 1, 2, 3)]
    assert spec.streams == 3 and spec.embedding_scale == 5.0 and spec.tie_word_embeddings and spec.final_norm.kind == "layernorm"
    assert all(layer.arrangement == "hyper_connections" and layer.streams == 3 for layer in spec.layers)
    second, linear, first = (spec.layers[i].mixer for i in (0, 1, 2))
    assert isinstance(first, LatentAttentionSpec) and isinstance(second, LatentAttentionSpec)
    assert (first.q_rank, first.kv_rank, first.head_dim, first.rot_dim, first.v_head_dim, first.window, first.scale) == \
        (None, 18, 10, 6, 14, 7, 0.4)
    assert first.gate_over == "head" and first.gate_size == 5 and not first.sink and first.position.interleaved
    assert first.position.scaling.original == 16 and second.position.scaling is None
    assert second.gate_over == "element" and second.gate_size == 3 * 4 and second.sink and second.window == 13
    assert isinstance(linear, GatedLinearAttentionSpec)
    assert (linear.n_heads, linear.head_dim, linear.v_head_dim, linear.tau, linear.decay_rank, linear.norm_eps) == \
        (3, 12, 20, 4.0, 5, 2e-5)
    assert isinstance(spec.layers[0].feed_forward, PlainFeedForwardSpec) and spec.layers[0].feed_forward.activation == "relu2"
    assert spec.layers[1].feed_forward is None and spec.layers[1].feed_forward_norm is None
    arch = resolve(RANUDRA_D)
    assert arch.model_spec(arch.parse_config(RANUDRA_D)).layers[2].mixer.position is None


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
    (_changed(("layers", 0, "type"), "attention"), "unknown layer type"),
    (_changed(("layers", 0, "mixer", "rot_dim"), 9), "must be even"),
    (_changed(("layers", 0, "mixer", "rot", "dims"), 8), "the whole rotated part"),
    (_changed(("layers", 2, "mixer", "rot", "scaling", "slow"), KeyError), "lacks required keys"),
    (_changed(("layers", 0, "mixer", "kv_rank"), KeyError), "lacks required keys"),
    (_changed(("layers", 0, "mixer", "mask", "size"), 0), "positive integer"),
    (_changed(("layers", 1, "mixer", "tau"), 0.0), "positive"),
    (_changed(("layers", 1, "mixer", "tau"), KeyError), "lacks required keys"),
    (_changed(("layers", 0, "mlp", "kind"), "moe"), "unknown feed-forward kind"),
    (_changed(("loop", "stop"), 5), "not a stretch"),
    (_changed(("loop", "times"), 0), "positive integer"),
    (_changed(("streams",), KeyError), "lacks required keys"),
    (_changed(("embedding",), KeyError), "lacks required keys"),
    (_changed(("norm",), KeyError), "lacks required keys"),
    (_changed(("layers",), []), "no layers"),
])
def test_bad_configurations_are_refused(change, message):
    from pylon_amd.config.registry import resolve

    raw = copy.deepcopy(RANUDRA_A)
    change(raw)
    with pytest.raises(ValueError, match=message):
        resolve(raw).parse_config(raw)


def test_parts_refuse_what_their_kernels_do_not_cover():
    from dataclasses import replace

    from pylon_amd.config.specs import (GatedLinearAttentionSpec, LatentAttentionSpec, LayerSpec, NormSpec,
                                        PlainFeedForwardSpec, PositionSpec)
    from pylon_amd.parts import build_part

    kw = dict(dtype=torch.float32, device="cpu")
    base = LatentAttentionSpec(hidden_size=32, n_heads=2, head_dim=8, v_head_dim=8, q_rank=None, kv_rank=16, scale=0.3,
                               norm_eps=1e-6, rot_dim=4, position=PositionSpec(kind="rope", rotary_dim=4, interleaved=True))
    build_part("mixer", base, **kw)
    for change, message in ((dict(kv_rank=520), "up to 512"), (dict(rot_dim=5), "even"), (dict(q_rank=12), "straight from the input"),
                            (dict(window=3, chunk=3), "not both"), (dict(gate_over="row"), "gate_over"), (dict(rot_dim=6), "whole part")):
        with pytest.raises(ValueError, match=message):
            build_part("mixer", replace(base, **change), **kw)
    linear = GatedLinearAttentionSpec(hidden_size=32, n_heads=2, head_dim=8, v_head_dim=8, decay_rank=4, tau=2.0, norm_eps=1e-6)
    build_part("mixer", linear, **kw)
    for change in (dict(tau=0.0), dict(decay_rank=0), dict(v_head_dim=2000)):
        with pytest.raises(ValueError):
            build_part("mixer", replace(linear, **change), **kw)
    with pytest.raises(ValueError, match="relu2"):
        build_part("feed_forward", PlainFeedForwardSpec(hidden_size=8, intermediate_size=8, activation="gelu"), **kw)
    norm = NormSpec(kind="layernorm", dim=32, eps=1e-6)
    layer = LayerSpec(mixer=linear, feed_forward=None, mixer_norm=norm, feed_forward_norm=None,
                      arrangement="hyper_connections", streams=2)
    build_part("block", layer, **kw)
    for change in (dict(streams=17), dict(sublayer_scale=True)):
        with pytest.raises(ValueError):
            build_part("block", replace(layer, **change), **kw)


def test_a_model_whose_layers_disagree_about_the_streams_copies_is_refused():
    from dataclasses import replace

    from pylon_amd.config.registry import resolve
    from pylon_amd.engine.model import Model

    arch = resolve(RANUDRA_A)
    spec = arch.model_spec(arch.parse_config(RANUDRA_A))
    with pytest.raises(ValueError, match="copies"):
        Model(replace(spec, streams=2), dtype=torch.float32, device="cpu")
    again = tuple(replace(e, add_embedding=i == 2) for i, e in enumerate(spec.schedule))
    with pytest.raises(ValueError, match="one copy"):
        Model(replace(spec, schedule=again), dtype=torch.float32, device="cpu")


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
        second = model.blocks[0].mixer
        assert second.params["down"].shape == (3 * 16 + 22 + 12, 40)
        assert same(second.params["down"][:48], "l0.mix.q") and same(second.params["down"][48: 70], "l0.mix.dkv")
        assert same(second.params["down"][70:], "l0.mix.g") and same(second.params["sink"], "l0.mix.sink")
        assert same(second.params["c_norm"], "l0.mix.dkv.norm") and same(second.params["uv"], "l0.mix.uv")
        first = model.blocks[2].mixer
        assert first.params["down"].shape == (5 * 16 + 24 + 5, 40) and "sink" not in first.params
        linear = model.blocks[1].mixer
        assert linear.params["proj"].shape == (36 + 36 + 60 + 60 + 5, 40)
        assert same(linear.params["proj"][36: 72], "l1.mix.k") and same(linear.params["proj"][132: 192], "l1.mix.g")
        assert same(linear.params["proj"][192:], "l1.mix.a1") and same(linear.params["a2"], "l1.mix.a2")
        assert same(linear.params["a2_bias"], "l1.mix.a2.b") and same(linear.params["norm"], "l1.mix.norm")
        assert same(model.blocks[0].params["mixer_mix"], "l0.hc1.mix") and same(model.blocks[0].params["feed_forward_write"], "l0.hc2.out")
        assert same(model.blocks[2].params["feed_forward_read"], "l2.hc2.in")
        assert model.blocks[1].feed_forward is None and "feed_forward_mix" not in model.blocks[1].params
        assert "l1.norm2" not in weights and "l1.hc2.mix" not in weights


def test_the_size_between_the_decays_two_maps_comes_from_the_tensors(tmp_path):
    import json

    from pylon_amd.config.registry import load_model_config

    folder = make_folder(tmp_path, "A")
    raw = json.loads((folder / "config.json").read_text())
    for layer in raw["layers"]:
        layer["mixer"].pop("decay_rank", None)
    (folder / "config.json").write_text(json.dumps(raw))
    arch, cfg = load_model_config(folder)
    assert [layer.mixer.decay_rank for layer in cfg.layers if layer.type == "gla"] == [5, 3]
    assert arch.model_spec(cfg).layers[3].mixer.decay_rank == 3


def test_a_folder_that_lacks_a_tensor_or_holds_one_too_many_is_refused(tmp_path):
    from safetensors.torch import load_file, save_file

    from pylon_amd.config.registry import load_model_config
    from pylon_amd.engine.model import Model
    from pylon_amd.weights.loader import WeightsError, load_weights

    folder = make_folder(tmp_path, "A")
    arch, cfg = load_model_config(folder)
    tensors = load_file(str(folder / "model.safetensors"))
    sink = tensors.pop("l0.mix.sink")
    tensors["l2.mix.sink"] = sink
    save_file(tensors, str(folder / "model.safetensors"))
    model = Model(arch.model_spec(cfg), dtype=torch.float32, device="cpu")
    with pytest.raises(WeightsError) as error:
        load_weights(model, arch, cfg, folder, strict=True)
    assert "l0.mix.sink" in str(error.value) and "l2.mix.sink" in str(error.value)


def test_every_run_asks_for_a_row_per_token_or_a_state_of_its_own():
    from pylon_amd.cache.manager import CacheManager
    from pylon_amd.config.registry import resolve
    from pylon_amd.engine.model import Model
    from pylon_amd.parts.base import KVRequirement, StateRequirement

    arch = resolve(RANUDRA_A)
    model = Model(arch.model_spec(arch.parse_config(RANUDRA_A)), dtype=torch.float32, device="cpu")
    needs = model.cache_requirements()
    row, wide = KVRequirement(1, 24, 7, values=False), KVRequirement(1, 22, 13, values=False)
    state, small = StateRequirement((3, 12, 20), torch.float32), StateRequirement((2, 20, 6), torch.float32)
    assert needs == [wide, state, row, state, row, small]  # the looped layers' passes keep their own
    manager = CacheManager(needs, dtype=torch.float32, page_size=16, num_pages=6, max_requests=2, device="cpu")
    seq = manager.open("a")
    assert manager.view(1).state.data_ptr() != manager.view(3).state.data_ptr()
    # a slot that is handed out again starts from zeros
    for tensor in manager.slots.tensors.values():
        tensor.fill_(7.0)
    manager.close(seq)
    again = manager.open("b")
    for key, tensor in manager.slots.tensors.items():
        assert float(tensor[again.slot].abs().max()) == 0.0, key


def test_the_row_kernels_rule_and_launch_shapes():
    from pylon_amd.kernels import ops

    ok = lambda width, rank, page=64, dtype=torch.bfloat16: ops.latent_attention_ok(dtype, width=width, rank=rank, page_size=page)  # noqa: E731
    assert ok(96, 64) and ok(320, 256, 256) and ok(576, 512) and ok(8, 8) and ok(200, 160)
    assert not ok(96, 64, 32) and not ok(100, 64) and not ok(96, 64, dtype=torch.float32) and not ok(584, 512)
    assert ops.latent_rows(32, 256) == 64 and ops.latent_rows(64, 512) == 64 and ops.latent_rows(65, 256) == 128
    assert ops.latent_rows(65, 512) is None and ops.latent_rows(129, 64) is None
    assert ops.latent_cuts(8, 32, 1024, units=256) == 8 and ops.latent_cuts(8, 32, 200, units=256) == 1
    assert ops.latent_cuts(1, 6, 100000, units=256) == 64 and ops.latent_cuts(300, 6, 100000, units=256) == 1
    assert ops.gla_chunked_ok(torch.bfloat16, dim=64, vdim=20) and not ops.gla_chunked_ok(torch.bfloat16, dim=48, vdim=32)
    assert not ops.gla_chunked_ok(torch.float32, dim=64, vdim=64) and ops.gla_ok(256, 256) and not ops.gla_ok(1024, 128)
    assert ops.gla_chunk_parallel(1, 10, 128, 128, 2048, units=256) and not ops.gla_chunk_parallel(40, 10, 128, 128, 2048, units=256)
    assert not ops.gla_chunk_parallel(1, 10, 128, 128, 100, units=256)


# ---- the plain implementation against closed forms --------------------------------------------------

def test_plain_layer_norm_takes_the_mean_off_first():
    x = np.array([[1.0, 3.0], [101.0, 103.0]])
    got = plain.layer_norm(x, np.array([2.0, 1.0]), 0.0)
    assert np.allclose(got, [[-2.0, 1.0], [-2.0, 1.0]])
    assert np.allclose(plain.rms_norm(np.array([[3.0, 4.0]]), 1.0, 0.0), np.array([[3.0, 4.0]]) / math.sqrt(12.5))


def test_plain_copies_of_the_stream_change_all_at_once_from_the_old_ones():
    xs = np.array([[[1.0, 10.0]], [[2.0, 20.0]]])  # two copies, one token
    w = {"in": np.array([1.0, 0.5]), "out": np.array([3.0, -1.0]), "mix": np.array([[0.0, 1.0], [1.0, 2.0]])}
    seen = []
    got = plain.hyper_step(xs, lambda u: (seen.append(u.copy()), u * 0 + 100.0)[1], w, "")
    assert np.allclose(seen[0], [[2.0, 20.0]])                      # 1 x_1 + 0.5 x_2
    assert np.allclose(got[0], [[2.0 + 300.0, 20.0 + 300.0]])       # from x_2 alone: mix[1, 0] = 1
    assert np.allclose(got[1], [[1.0 + 4.0 - 100.0, 10.0 + 40.0 - 100.0]])  # mix[0, 1] x_1 + mix[1, 1] x_2


def test_plain_rotation_pairs_neighbours_and_starts_at_any_position():
    x = np.arange(3 * 4, dtype=np.float64).reshape(3, 4) + 1.0
    rot = {"base": 100.0, "dims": 4}
    got = plain.rotate(x, rot)
    assert np.array_equal(got[0], x[0])
    a = 1.0 * 100.0 ** -0.5  # position 1, the second pair
    u, v = x[1, 2], x[1, 3]
    assert np.allclose(got[1, 2:], [u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a)])
    assert np.allclose(plain.rotate(x[1:], rot, first=1), got[1:])
    heads = plain.rotate(np.repeat(x[:, None, :], 2, axis=1), rot)
    assert np.allclose(heads[:, 1], got)
    scaled = dict(rot, scaling={"factor": 4.0, "original": 2 * math.pi * 16, "fast": 1000.0, "slow": 500.0})
    # every pair makes fewer turns than `slow`: the ramp ends before the first pair, whose index it still leaves
    # as it is (lo is at least 0), and the second is stretched
    f, mult = plain.rotary_frequencies(scaled)
    assert np.allclose(f, [1.0, 0.1 / 4.0])
    assert abs(mult - (0.1 * math.log(4.0) + 1.0)) < 1e-12
    assert np.allclose(plain.rotate(x, scaled)[0], x[0] * mult)  # the factor stays at position 0


def test_plain_window_holds_its_size_of_keys_the_query_included():
    seen = plain.visible(7, 3)
    assert seen[5].tolist() == [False, False, False, True, True, True, False]
    assert seen[1].tolist() == [True, True, False, False, False, False, False]
    assert plain.visible(4, 1).astype(int).tolist() == np.eye(4, dtype=int).tolist() and plain.visible(4, None)[3].all()


def test_plain_softmax_with_a_sink():
    q, k, v = np.zeros((1, 1, 2)), np.ones((1, 1, 2)), np.full((1, 1, 3), 5.0)
    # one key of score 0 and a sink of ln 3: the key keeps a quarter of the weight
    out = plain.softmax_attention(q, k, v, 1.0, plain.visible(1, None), np.array([math.log(3.0)]))
    assert np.allclose(out, 1.25)


def test_plain_keys_are_made_of_the_latent_and_one_shared_part():
    rng = np.random.default_rng(0)
    m = {"heads": 2, "dim": 3, "rot_dim": 2, "vdim": 4, "kv_rank": 5, "rot": {"base": 10.0, "dims": 2}}
    w = {"dkv": rng.normal(size=(7, 6)), "dkv.norm": rng.normal(size=5), "uk": rng.normal(size=(6, 5)), "uv": rng.normal(size=(8, 5))}
    h = rng.normal(size=(3, 6))
    k, v = plain.latent_keys_values(h, m, w, "", 1e-6)
    assert k.shape == (3, 2, 5) and v.shape == (3, 2, 4)
    assert np.array_equal(k[:, 0, 3:], k[:, 1, 3:]) and not np.allclose(k[:, 0, :3], k[:, 1, :3])
    c = plain.rms_norm(h @ w["dkv"][:5].T, w["dkv.norm"], 1e-6)
    assert np.allclose(k[2, 1, :3], w["uk"][3:] @ c[2]) and np.allclose(v[1, 0], w["uv"][:4] @ c[1])
    assert np.allclose(k[0, 0, 3:], h[0] @ w["dkv"][5:].T)  # not normed; position 0 turns nothing


def test_plain_gated_linear_attention_forgets_by_channel_and_reads_its_own_write():
    # one head, two key channels, one value: channel 0 keeps everything, channel 1 half of it
    q = np.array([[[1.0, 1.0]], [[1.0, 0.0]], [[0.0, 1.0]]])
    k = np.array([[[1.0, 1.0]], [[0.0, 0.0]], [[0.0, 1.0]]])
    v = np.array([[[3.0]], [[5.0]], [[7.0]]])
    decay = np.tile(np.array([1.0, 0.5]), (3, 1, 1))
    out = plain.gated_linear_attention(q, k, v, decay)
    assert np.allclose(out[:, 0, 0], [6.0, 3.0, 3.0 * 0.25 + 7.0])


def test_plain_squared_relu_and_the_order_of_a_loop():
    w = {"up": np.array([[1.0], [-1.0]]), "down": np.array([[1.0, 10.0]])}
    assert np.allclose(plain.feed_forward(np.array([[3.0], [-2.0]]), w, ""), [[9.0], [40.0]])
    assert plain.run_order(RANUDRA_A) == [0, 1, 2, 1, 2, 3] and plain.run_order(RANUDRA_D) == [0, 1, 2, 3]


def test_plain_forward_in_two_cuts_agrees_on_the_common_positions(tmp_path):
    for name in ("A", "E"):
        cfg, weights = read_folder(make_folder(tmp_path, name))
        toks = list(range(3, 40))
        whole = plain.forward(cfg, weights, toks)
        assert np.allclose(plain.forward(cfg, weights, toks[:21]), whole[:21], atol=1e-9)
        streams = []
        plain.forward(cfg, weights, toks, streams=streams)
        assert len(streams) == len(plain.run_order(cfg)) and streams[0].shape == (len(toks), cfg["width"])
