"""Farorax on the GPU against the plain implementation: every mechanism's kernel alone, then whole models
cut every way (whole prompts, token by token, portions down to two tokens, mixed batches over pages and
slots that are used again), long decoding, and greedy generation through the engine."""
import numpy as np
import pytest
import torch

from tests.farorax_helpers import CONFIGS, make_folder, read_folder, tokens
from tests.helpers import rows_within
from tests.plain import farorax as plain

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32_BOUND = 2e-4    # of a row's largest |logit|
BF16_BOUND = 1e-1
ROUTER_MARGIN = 0.02  # lead of a choice, in scores, below which a bfloat16 model may choose otherwise


@pytest.fixture(scope="module")
def ops():
    if not torch.cuda.is_available():
        pytest.skip("needs a GPU")
    from pylon_amd.kernels import ops as module

    return module


@pytest.fixture(scope="module")
def tmp(tmp_path_factory):
    if not torch.cuda.is_available():
        pytest.skip("needs a GPU")
    return tmp_path_factory.mktemp("farorax")


def i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def dev(array, dtype=torch.float32):
    return torch.tensor(np.asarray(array), dtype=dtype, device=DEV)


def close(got, want, bound, what=""):
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want)
    assert got.shape == want.shape, (what, got.shape, want.shape)
    err = np.abs(got - want).max() / max(np.abs(want).max(), 1e-30)
    assert err <= bound, f"{what}: off by {err:.2e} of the largest value"


def rounded(array, dtype):
    """What a tensor of ``dtype`` holds of these numbers, as float64."""
    return torch.tensor(np.asarray(array)).to(dtype).double().numpy()


# ---- lightning attention -------------------------------------------------------------------------------

LIGHTNING_SHAPES = [(3, 32, 32), (2, 12, 20), (3, 64, 128), (2, 128, 128), (1, 256, 64), (2, 128, 32), (1, 100, 24), (5, 1, 1),
                    (2, 48, 200), (1, 32, 256), (4, 96, 80), (1, 224, 7), (2, 160, 16), (7, 192, 48)]


def run_lightning(ops, proj, state, decay, rows, slots, heads, dim, vdim):
    """One step: ``rows`` of token counts, the chunked form where it fits (as the mixer chooses)."""
    starts = np.concatenate([[0], np.cumsum(rows)])
    chunked = max(rows) >= 4 and ops.retention_chunked_ok(proj.dtype, dim=dim, vdim=vdim, rot_dims=0)
    return ops.retention_recurrent(proj, state, decay, None, i32([0] * len(proj)), i32(starts), i32(slots), rows=len(rows),
                                   heads=heads, dim=dim, vdim=vdim, rot_dims=0, eps=1e-6, k_scale=1.0, chunked=chunked,
                                   max_count=max(rows), form="lightning").cpu().numpy()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, dim, vdim", LIGHTNING_SHAPES)
def test_lightning_in_portions_of_two_requests_over_reused_slots(ops, heads, dim, vdim, dtype):
    """Two requests of 301 and 23 tokens in portions of changing size, single tokens among them, in slots
    that held other numbers before; decays from nothing to one."""
    rng = np.random.default_rng(heads * 1000 + dim + vdim)
    lengths = {"x": 301, "y": 23}
    decay = np.linspace(0.0, 1.0, heads) if heads > 2 else np.array([0.97, 0.9995])[:heads]
    decay = decay.astype(np.float32).astype(np.float64)
    qk, vv = heads * dim, heads * vdim
    data = {rid: rounded(rng.normal(size=(n, 2 * qk + 2 * vv)), dtype) for rid, n in lengths.items()}
    want, bound = {}, (2e-5 if dtype == torch.float32 else 8e-3)
    for rid, x in data.items():
        q, k, v = (rounded(plain.silu(part), dtype).reshape(len(x), heads, -1)
                   for part in (x[:, :qk], x[:, qk: 2 * qk], x[:, 2 * qk: 2 * qk + vv]))
        want[rid] = plain.decayed_state(q, k, v, decay)
    state = torch.full((3, heads, dim, vdim), 9.0, device=DEV)
    slots = {"x": 2, "y": 0}
    for slot in slots.values():
        state[slot].zero_()  # as the cache manager does when a slot is handed out
    pos, got = {"x": 0, "y": 0}, {"x": [], "y": []}
    plan = [{"x": 2}, {"x": 1, "y": 1}, {"x": 31, "y": 2}, {"y": 1}, {"x": 3, "y": 19}, {"x": 65}, {"x": 1}, {"x": 190}, {"x": 8}]
    for step in plan:
        proj = np.concatenate([data[rid][pos[rid]: pos[rid] + n] for rid, n in step.items()])
        out = run_lightning(ops, dev(proj, dtype), state, dev(decay), list(step.values()), [slots[r] for r in step], heads, dim, vdim)
        cursor = 0
        for rid, n in step.items():
            got[rid].append(out[cursor: cursor + n])
            cursor += n
            pos[rid] += n
    assert pos == lengths
    for rid in data:
        close(np.concatenate(got[rid]).reshape(want[rid].shape), want[rid], bound, f"{rid} in portions")
    assert float(state[1].min()) == 9.0 == float(state[1].max())  # a slot that no row names is left alone
    # whole: with few heads the row's stretches of chunks run side by side
    again = torch.zeros_like(state)
    out = run_lightning(ops, dev(data["x"], dtype), again, dev(decay), [301], [1], heads, dim, vdim)
    close(out.reshape(want["x"].shape), want["x"], bound, "whole")
    close(again[1].cpu().numpy(), state[2].cpu().numpy(), 2e-5 if dtype == torch.float32 else 1e-4, "the state left behind")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_lightning_keeps_what_it_wrote_far_back(ops, dtype):
    """One key stands out at position 5 of 700; only the last query asks for it, through a state that went
    through portions, single tokens and stretches of several chunks."""
    rng = np.random.default_rng(3)
    heads, dim, vdim, n = 2, 64, 32, 700
    decay = np.array([0.999, 1.0]).astype(np.float32).astype(np.float64)
    x = rng.normal(size=(n, heads, 2 * dim + vdim)) * 0.1
    x[:, :, :dim // 2] = -20.0               # silu of it is nothing: queries and keys look at the other half ...
    x[:, :, dim: dim + dim // 2] = -20.0
    x[5, :, dim: dim + dim // 2] = 3.0       # ... but this key has the first half too
    x[-1, :, : dim // 2] = 3.0               # and so does the last query
    x[5, :, 2 * dim:] = 2.0 + rng.normal(size=(heads, vdim))
    flat = np.concatenate([x[:, :, :dim].reshape(n, -1), x[:, :, dim: 2 * dim].reshape(n, -1), x[:, :, 2 * dim:].reshape(n, -1),
                           np.zeros((n, heads * vdim))], axis=1)
    flat = rounded(flat, dtype)
    q, k, v = (rounded(plain.silu(flat[:, a: b]), dtype).reshape(n, heads, -1)
               for a, b in ((0, 128), (128, 256), (256, 320)))
    want = plain.decayed_state(q, k, v, decay)
    without = k.copy()
    without[5] = 0.0
    assert np.abs(plain.decayed_state(q, without, v, decay)[-1] - want[-1]).max() > 0.5 * np.abs(want[-1]).max()
    state = torch.zeros((2, heads, dim, vdim), device=DEV)
    out, pos = [], 0
    for size in (3, 40, 1, 600, 7, 1, 1, 46, 1):
        out.append(run_lightning(ops, dev(flat[pos: pos + size], dtype), state, dev(decay), [size], [1], heads, dim, vdim))
        pos += size
    assert pos == n
    got = np.concatenate(out).reshape(want.shape)
    assert np.abs(got[-1] - want[-1]).max() <= (1e-4 if dtype == torch.float32 else 5e-3) * np.abs(want[-1]).max()
    close(got, want, 1e-4 if dtype == torch.float32 else 5e-3)


@pytest.mark.parametrize("span", [1, 2, 3, 5, 40])
def test_stretches_of_any_number_of_chunks_give_the_same(ops, monkeypatch, span):
    rng = np.random.default_rng(span)
    heads, dim, vdim, n = 3, 64, 48, 420
    proj = dev(rng.normal(size=(n, 2 * heads * (dim + vdim))), torch.bfloat16)
    decay = dev([0.9, 0.99, 1.0])
    results = {}
    for form in ("lightning", "retention"):
        for way in ("one workgroup a head", "stretches"):
            state = dev(np.random.default_rng(9).normal(size=(2, heads, dim, vdim)))
            monkeypatch.setattr(ops, "retention_chunk_parallel", lambda *a, w=way, **k: w == "stretches")
            monkeypatch.setattr(ops, "retention_chunk_span", lambda *a, **k: span)
            out = ops.retention_recurrent(proj, state, decay, None, i32([0] * n), i32([0, 300, n]), i32([1, 0]), rows=2, heads=heads,
                                          dim=dim, vdim=vdim, rot_dims=0, eps=1e-6, k_scale=1.0, chunked=True, max_count=300,
                                          form=form)
            results[way] = (out.float().cpu().numpy(), state.cpu().numpy())
        bound = 1e-4 if form == "lightning" else 1e-2
        close(results["stretches"][0], results["one workgroup a head"][0], bound, form)
        close(results["stretches"][1], results["one workgroup a head"][1], 1e-4, form)


@pytest.mark.parametrize("dim", [5, 64, 100, 384, 1280, 4096, 4100, 8192, 16000, 20000])
def test_a_norm_over_all_heads_with_gates(ops, dim):
    rng = np.random.default_rng(dim)
    n = 3
    x = rng.normal(size=(n, dim)) * np.array([[1e-3], [1.0], [40.0]])
    w, eps = 1.0 + 0.3 * rng.normal(size=dim), 1e-5
    for dtype, bound in ((torch.float32, 5e-6), (torch.bfloat16, 5e-3)):
        for lead in (0, 8, 3):  # the gate's place in a wider row
            wide = rounded(rng.normal(size=(n, lead + dim)) * 2, dtype)
            gate = wide[:, lead:]
            for act, value in (("sigmoid", plain.sigmoid(gate)), ("silu", plain.silu(gate))):
                got = ops.norm_gate(dev(x), dev(w), dev(wide, dtype)[:, lead:], eps, act=act).float().cpu().numpy()
                for row in range(n):
                    close(got[row], (plain.norm(x, w, eps) * value)[row], bound, f"{act}, lead {lead}, row {row}")


# ---- feed-forwards -------------------------------------------------------------------------------------

@pytest.mark.parametrize("rows", [1, 5, 16, 17, 64, 65, 128, 200])
@pytest.mark.parametrize("width, ff", [(64, 88), (256, 512), (100, 44), (2560, 384)])
def test_a_product_gated_through_gelu(ops, rows, width, ff):
    rng = np.random.default_rng(rows + width)
    for dtype, bound in ((torch.float32, 1e-5), (torch.bfloat16, 1.2e-2)):
        x, w = rounded(rng.normal(size=(rows, width)), dtype), rounded(rng.normal(size=(2 * ff, width)) * width ** -0.5, dtype)
        for act, fn in (("gelu_tanh", plain.gelu_tanh), ("silu", plain.silu)):
            got = ops.linear_glu(dev(x, dtype), dev(w, dtype), out_dtype=dtype, act=act).float().cpu().numpy()
            close(got, fn(x @ w[:ff].T) * (x @ w[ff:].T), bound, f"{dtype} {act}")


def test_gelu_far_out_and_at_zero(ops):
    z = np.array([[-1e4, -40.0, -3.0, -0.5, 0.0, 1e-3, 0.5, 3.0, 40.0, 1e4]])
    got = ops.silu_gate(dev(np.concatenate([z, np.ones_like(z)], axis=1)), act="gelu_tanh").cpu().numpy()
    assert np.isfinite(got).all()
    assert np.allclose(got, plain.gelu_tanh(z), rtol=2e-6, atol=1e-7)
    # it is neither silu nor the other form of gelu
    assert abs(float(got[0, 7]) - float(plain.silu(np.array(3.0)))) > 1e-2


@pytest.mark.parametrize("experts, top, groups", [(6, 2, (3, 2)), (8, 3, (4, 2)), (12, 4, (2, 1)), (5, 3, (5, 4)), (9, 9, (3, 3)),
                                                  (64, 8, (8, 3)), (512, 16, (16, 4)), (7, 1, None), (16, 6, None), (1, 1, None)])
def test_routing_from_the_best_groups(ops, experts, top, groups):
    rng = np.random.default_rng(experts + top)
    n = 37
    z = np.array([rng.permutation(np.linspace(-4.0, 4.0, experts)) for _ in range(n)]) + rng.normal(size=(n, experts)) * 0.01
    z = z.astype(np.float32).astype(np.float64)
    router = {"experts": experts, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    margins = []
    want_e, want_w = plain.route(np.eye(n), {"router": z.T}, "", router, margins)
    got_e, got_w, identity = ops.route_scored(dev(z), None, n_experts=experts, top=top, groups=groups[0] if groups else 1,
                                              keep=groups[1] if groups else 1, scoring="sigmoid", group_score="top2",
                                              renormalize=True)
    assert identity is None
    clear = margins[0] > 1e-6
    assert clear.sum() > n // 2
    assert np.array_equal(got_e.cpu().numpy()[clear], want_e[clear])
    close(got_w.cpu().numpy()[clear], want_w[clear], 2e-6)
    assert np.allclose(got_w.sum(dim=1).cpu().numpy(), 1.0, atol=1e-5)
    if groups and experts == 12:
        # the sum of the two best and the best alone choose differently somewhere in this case
        other, _, _ = ops.route_scored(dev(z), None, n_experts=experts, top=top, groups=2, keep=1, scoring="sigmoid", renormalize=True)
        assert not np.array_equal(other.cpu().numpy(), got_e.cpu().numpy())


def test_scores_of_nothing_still_give_finite_weights(ops):
    got_e, got_w, _ = ops.route_scored(dev(np.full((2, 4), -200.0)), None, n_experts=4, top=2, groups=2, keep=1, scoring="sigmoid",
                                       group_score="top2", renormalize=True)
    assert torch.isfinite(got_w).all() and got_e.cpu().numpy().tolist() == [[0, 1], [0, 1]]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width, experts, top, ff, groups, shared", [
    (40, 6, 2, 16, (3, 2), 12), (64, 8, 3, 24, (4, 2), None), (128, 4, 1, 64, None, 32), (96, 12, 4, 40, (2, 1), 56),
    (100, 5, 3, 20, (5, 4), 12)])
def test_mixture_against_the_plain_one(ops, dtype, width, experts, top, ff, groups, shared):
    from pylon_amd.config.specs import MixtureFeedForwardSpec
    from pylon_amd.parts import build_part

    rng = np.random.default_rng(width)
    w = {"router": rng.normal(size=(experts, width)) * 2.0 * width ** -0.5}
    for name, size in [(f"e{e}", ff) for e in range(experts)] + ([("shared", shared)] if shared else []):
        w[f"{name}.gate"], w[f"{name}.up"] = (rng.normal(size=(size, width)) * width ** -0.5 for _ in range(2))
        w[f"{name}.down"] = rng.normal(size=(width, size)) * size ** -0.5
    w = {name: rounded(value, dtype) for name, value in w.items()}
    spec = MixtureFeedForwardSpec(hidden_size=width, n_experts=experts, top=top, expert_size=ff, shared_size=shared,
                                  shared_gate=False, router_bias=False, scoring="sigmoid", groups=groups[0] if groups else 1,
                                  groups_kept=groups[1] if groups else 1, group_score="top2", renormalize=True)
    part = build_part("feed_forward", spec, dtype=dtype, device=DEV)
    part.params["router"].copy_(dev(w["router"], dtype))
    part.params["gate_up"].copy_(dev(np.concatenate([w[f"e{e}.{x}"] for e in range(experts) for x in ("gate", "up")]), dtype))
    part.params["down"].copy_(dev(np.concatenate([w[f"e{e}.down"] for e in range(experts)]), dtype))
    if shared:
        part.params["shared_gate_up"].copy_(dev(np.concatenate([w["shared.gate"], w["shared.up"]]), dtype))
        part.params["shared_down"].copy_(dev(w["shared.down"], dtype))
    mlp = {"router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}
    if groups:
        mlp["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    for n in (1, 9, 33, 150):
        h = rounded(rng.normal(size=(n, width)), dtype)
        margins = []
        want = plain.mixture(h, w, "", mlp, margins)
        clear = margins[0] > 1e-4
        got = part.forward(dev(h, dtype), None).cpu().numpy()
        close(got[clear], want[clear], 1e-5 if dtype == torch.float32 else 2e-2, f"{n} tokens")


# ---- the residual stream -------------------------------------------------------------------------------

@pytest.mark.parametrize("rows, dim", [(1, 40), (5, 256), (700, 100), (600, 33), (3, 2560), (2, 5124)])
def test_a_factor_on_what_joins_the_stream(ops, rows, dim):
    rng = np.random.default_rng(rows + dim)
    resid, gain, eps, factor = rng.normal(size=(rows, dim)), 1.0 + 0.3 * rng.normal(size=dim), 1e-5, 0.3
    scale, bias = rng.normal(size=dim), rng.normal(size=dim)
    for parts, dtype in ((1, torch.float32), (1, torch.bfloat16), (2, torch.float32), (4, torch.float32), (7, torch.float32)):
        d = rounded(rng.normal(size=(parts, rows, dim)), dtype)
        delta = dev(d if parts > 1 else d[0], dtype)
        x = resid + factor * d.sum(axis=0)
        held = dev(resid)
        got = ops.add_rmsnorm(held, delta, dev(gain), eps, torch.float32, factor=factor)
        close(held.cpu().numpy(), x, 1e-6, "the stream")
        close(got.cpu().numpy(), plain.norm(x, gain, eps), 2e-5, "its norm")
        held, pick = dev(resid), [rows - 1, 0]
        got = ops.add_rmsnorm(held, delta, dev(gain), eps, torch.float32, factor=factor, row_idx=i32(pick))
        close(got.cpu().numpy(), plain.norm(x, gain, eps)[pick], 2e-5, "picked rows")
        close(held.cpu().numpy(), resid, 1e-7, "untouched")
        got = ops.add_normed_rmsnorm(held, delta, dev(gain), eps, torch.float32, delta_scale=dev(scale), delta_bias=dev(bias),
                                     factor=factor)
        x = resid + factor * scale * (d.sum(axis=0) + bias)
        close(held.cpu().numpy(), x, 2e-6, "with scale and bias")
        close(got.cpu().numpy(), plain.norm(x, gain, eps), 3e-5, "its norm with scale and bias")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows, dim", [(1, 40), (5, 64), (40, 100), (130, 256), (3, 301)])
def test_the_entry_of_a_pass(ops, dtype, rows, dim):
    from pylon_amd.config.specs import PassEntrySpec
    from pylon_amd.parts import Scaled, build_part

    rng = np.random.default_rng(rows + dim)
    part = build_part("pass", PassEntrySpec(dim=dim, times=3), dtype=dtype, device=DEV)
    w = {"loop.in": rounded(rng.normal(size=(dim, 2 * dim)) * dim ** -0.5, dtype), "loop.step": rng.normal(size=(3, dim))}
    part.params["join"].copy_(dev(w["loop.in"], dtype))
    part.params["step"].copy_(dev(w["loop.step"]))
    x0 = rounded(rng.normal(size=(rows, dim)), dtype)
    resid = rng.normal(size=(rows, dim))
    d = rounded(rng.normal(size=(3, rows, dim)), torch.bfloat16)
    scale, bias = rng.normal(size=dim), rng.normal(size=dim)
    cases = [("nothing pending", None, resid), ("bfloat16", dev(d[0], torch.bfloat16), resid + d[0]),
             ("partial sums", dev(d), resid + d.sum(axis=0)),
             ("a factor", Scaled(dev(d[1]), factor=0.3), resid + 0.3 * d[1]),
             ("a factor on partial sums", Scaled(dev(d), factor=-0.7), resid - 0.7 * d.sum(axis=0)),
             ("scale and bias", Scaled(dev(d[2]), dev(scale), dev(bias), 0.5), resid + 0.5 * scale * (d[2] + bias))]
    for t, (what, delta, x) in enumerate(cases):
        held = dev(resid)
        out, pending = part.forward(held, delta, dev(x0), t % 3, None)
        assert pending is None and out.dtype == torch.float32
        close(out.cpu().numpy(), plain.enter_pass(x, x0, w, t % 3), 2e-5 if dtype == torch.float32 else 1e-2, what)


# ---- attention -----------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("tokens_n, heads, groups, dim, vdim, rot_dims, transposed", [
    (5, 6, 2, 64, 48, 32, True), (300, 6, 2, 64, 48, 64, True), (300, 3, 3, 32, 64, 0, False), (9, 4, 2, 10, 14, 6, False),
    (70, 4, 1, 128, 128, 128, True), (600, 2, 1, 24, 8, 16, True), (8, 32, 8, 128, 128, 64, True), (3, 5, 5, 12, 10, 12, True)])
def test_unnormed_q_and_k_turn_by_neighbours_and_values_go_into_their_pages(ops, dtype, tokens_n, heads, groups, dim, vdim,
                                                                          rot_dims, transposed):
    rng = np.random.default_rng(dim + vdim + tokens_n)
    page, pool = 32, -(-tokens_n // 32) + 3
    qs, ks, vs = heads * dim, groups * dim, groups * vdim
    x = rounded(rng.normal(size=(tokens_n, qs + ks + vs)), dtype)
    rot = {"base": 1000.0, "dims": rot_dims, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 64}} if rot_dims else None
    first = 11
    pad = np.zeros((first, 1, 1))
    def turned(part, count):
        full = np.concatenate([np.repeat(np.repeat(pad, count, axis=1), dim, axis=2), part.reshape(tokens_n, count, dim)])
        return plain.rotate_pairs(full, rot)[first:]
    freq = dev(plain.frequencies(rot)) if rot_dims else None
    slots = rng.permutation(pool * page)[:tokens_n]
    k_cache = torch.full((pool, page, groups, dim), 7.0, dtype=dtype, device=DEV)
    v_cache = torch.full((pool, groups, vdim, page) if transposed else (pool, page, groups, vdim), 7.0, dtype=dtype, device=DEV)
    q = torch.empty((tokens_n, heads, dim), dtype=dtype, device=DEV)
    ops.qkv_prepare_wide(dev(x, dtype), q, k_cache, v_cache, n_heads=heads, n_kv_heads=groups, head_dim=dim, v_dim=vdim,
                         q_weight=None, k_weight=None, eps=1e-6, inv_freq=freq, rot_dim=rot_dims, interleaved=True,
                         positions=i32(range(first, first + tokens_n)), slot_map=i32(slots), store_kv=True, v_transposed=transposed)
    bound = 2e-5 if dtype == torch.float32 else 5e-3
    close(q.float().cpu().numpy(), turned(x[:, :qs], heads), bound, "q")
    k_all = k_cache.view(-1, groups, dim).float().cpu().numpy()
    close(k_all[slots], turned(x[:, qs: qs + ks], groups), bound, "k")
    v_all = (v_cache.permute(0, 3, 1, 2) if transposed else v_cache).reshape(-1, groups, vdim).float().cpu().numpy()
    assert np.array_equal(v_all[slots], x[:, qs + ks:].reshape(tokens_n, groups, vdim))
    untouched = np.setdiff1d(np.arange(pool * page), slots)
    assert (k_all[untouched] == 7.0).all() and (v_all[untouched] == 7.0).all()


def planted_case(rng, n, heads, groups, dim, vdim, planted):
    """Keys among which the planted positions stand out along a direction that every query has a large
    share of."""
    direction = rng.normal(size=dim)
    direction /= np.linalg.norm(direction)
    q = rng.normal(size=(n, heads, dim)) + 4.0 * direction
    k = rng.normal(size=(n, groups, dim)) * 0.5
    for j in planted:
        k[j] += 6.0 * direction
    return q, k, rng.normal(size=(n, groups, vdim))


@pytest.mark.parametrize("size", [37, 64, 129, 1, 300, None])
@pytest.mark.parametrize("dtype, heads, groups, dim, vdim, page", [
    (torch.float32, 4, 2, 12, 20, 16), (torch.float32, 2, 1, 64, 64, 64), (torch.bfloat16, 6, 2, 64, 64, 64),
    (torch.bfloat16, 3, 3, 32, 48, 32), (torch.bfloat16, 10, 2, 128, 128, 64)])
def test_attention_with_a_sink_at_the_edges_of_windows_and_pages(ops, size, dtype, heads, groups, dim, vdim, page):
    """A 300-token request whose planted keys lie at position 0, at a page's last and first slot, just inside
    and just outside the window of many queries, and far back; pages scattered over a pool whose other
    slots hold NaN; whole, and as a portion over a cached first part."""
    rng = np.random.default_rng(23 + (size or 0))
    n = 300
    planted = sorted({0, page - 1, page, 2 * page, 150, 151})
    q, k, v = planted_case(rng, n, heads, groups, dim, vdim, planted)
    q, k, v = rounded(q, dtype), rounded(k, dtype), rounded(v, dtype)
    scale, sink = 0.3, rng.normal(size=heads) * 3.0 + 4.0
    def attend(visible, sink):
        out = np.zeros((n, heads, vdim))
        for head in range(heads):
            g = head // (heads // groups)
            out[:, head] = plain.softmax_with_sink(q[:, head] @ k[:, g].T * scale, visible, sink[head]) @ v[:, g]
        return out
    want = attend(plain.window_mask(n, size), sink)
    pages = -(-n // page)
    pool = pages + 5
    order = rng.permutation(pool)[:pages]
    k_cache = torch.full((pool, page, groups, dim), float("nan"), dtype=dtype, device=DEV)
    v_cache = torch.full((pool, page, groups, vdim), float("nan"), dtype=dtype, device=DEV)
    slots = torch.tensor([order[j // page] * page + j % page for j in range(n)], device=DEV)
    k_cache.view(-1, groups, dim)[slots] = dev(k, dtype)
    v_cache.view(-1, groups, vdim)[slots] = dev(v, dtype)
    table = i32(order).view(1, -1)
    bound = 2e-5 if dtype == torch.float32 else 2e-2
    for first in (0, 143):
        out = ops.paged_attention(dev(q[first:], dtype), k_cache, v_cache, table, i32([0] * (n - first)), i32(range(first, n)),
                                  page_size=page, window=size, scale=scale, sink_logit=dev(sink))
        close(out.float().cpu().numpy(), want[first:], bound, f"from {first}")
    if dtype == torch.bfloat16:
        v_t = v_cache.view(pool, page, groups, vdim).permute(0, 2, 3, 1).contiguous()
        for first in (0, 143):
            tiles = i32(x for a in range(first, n, 32) for x in (a - first, min(32, n - a), 0, a)).view(-1, 4)
            out = ops.attention_sink(dev(q[first:], dtype), k_cache, v_t, table, tiles, None, page_size=page, scale=scale,
                                     bias=None, sink=True, window=size, sink_logit=dev(sink))
            close(out.float().cpu().numpy(), want[first:], bound, f"matrix cores from {first}")
        for cuts in (1, 2, 8):
            out = ops.attention_sink(dev(q, dtype), k_cache, v_t, table.expand(n, -1).contiguous(), None, i32(range(n)),
                                     page_size=page, scale=scale, bias=None, sink=True, cuts=cuts, window=size,
                                     sink_logit=dev(sink))
            close(out.float().cpu().numpy(), want, bound, f"single tokens, {cuts} cuts")
    # the sink and the window's exact size matter in this case
    assert np.abs(attend(plain.window_mask(n, size), np.full(heads, -1e3)) - want).max() > 0.05
    if size is not None and size < n:
        assert np.abs(attend(plain.window_mask(n, size + 1), sink) - want).max() > 0.05
        if size > 1:
            assert np.abs(attend(plain.window_mask(n, size - 1), sink) - want).max() > 0.05


# ---- whole models --------------------------------------------------------------------------------------

def clear_tokens(cfg, weights, count, seed, margin=2 * ROUTER_MARGIN):
    """A request drawn token by token so that no router of the plain model has a close call at any position
    (a position's routing depends on the tokens up to it only)."""
    rng = np.random.default_rng(seed)
    out = []
    for _ in range(count):
        for _attempt in range(30):
            candidate = out + [int(rng.integers(0, cfg["vocab"]))]
            margins = []
            plain.forward(cfg, weights, candidate, margins=margins)
            if not margins or min(m[-1] for m in margins) >= margin:
                break
        out = candidate
    return out


class Case:
    def __init__(self, tmp, name, dtype, lengths, seed=3, config=None, pick=None):
        self.folder = make_folder(tmp, name, dtype=dtype, seed=seed, config=config)
        self.cfg, self.weights = read_folder(self.folder)
        # bfloat16 requests of up to a hundred tokens are drawn so that the positions' routing is clear
        pick = (dtype != "float32" and max(lengths) <= 100) if pick is None else pick
        draw = (lambda n, s: clear_tokens(self.cfg, self.weights, n, s)) if pick else (lambda n, s: tokens(self.cfg["vocab"], n, s))
        self.requests = {f"r{i}": draw(n, 50 + i) for i, n in enumerate(lengths)}
        self.want, self.clear = {}, {}
        for rid, toks in self.requests.items():
            margins = []
            self.want[rid] = plain.forward(self.cfg, self.weights, toks, margins=margins)
            closest = np.min(margins, axis=0) if margins else np.full(len(toks), np.inf)
            if dtype == "float32":
                self.clear[rid] = closest >= 1e-5
            else:
                # In bfloat16 a choice between two nearly equal scores is an accident of rounding, and a
                # flipped choice reaches every later token through the state and the attention: only the
                # positions before the first unclear choice are held to the plain model.
                unclear = np.flatnonzero(closest < ROUTER_MARGIN)
                self.clear[rid] = np.arange(len(toks)) < (unclear[0] if len(unclear) else len(toks))
        self.dtype = dtype
        self.bound = F32_BOUND if dtype == "float32" else BF16_BOUND

    def runner(self, page_size=16, num_pages=40, max_requests=3):
        from pylon_amd.engine import Runner

        return Runner.from_folder(self.folder, dtype=self.dtype, page_size=page_size, num_pages=num_pages,
                                  max_requests=max_requests)

    def check(self, rid, got, label):
        clear = self.clear[rid][: len(got)]
        assert np.isfinite(got).all()
        if not clear.any():
            return
        got, want = got[clear], self.want[rid][: len(got)][clear]
        if self.dtype == "float32":
            ok, worst, frac = rows_within(got, want, self.bound)
            assert ok, f"{label}: request {rid}, position {np.flatnonzero(clear)[worst]} is off by {frac:.2e} of its largest logit"
            return
        # bfloat16: a choice that looked clear in the plain model may still fall the other way behind layers
        # of rounding; one position in twenty-five may be further off, none by more than six times
        off = np.abs(got - want).max(axis=1) / np.abs(want).max(axis=1)
        assert off.max() <= 6 * self.bound, f"{label}: request {rid}, position {np.flatnonzero(clear)[off.argmax()]} is off by {off.max():.2e}"
        assert (off > self.bound).sum() <= max(1, len(off) // 25), \
            f"{label}: request {rid}: {(off > self.bound).sum()} of {len(off)} positions are off by more than {self.bound}"

    def compared(self):
        return sum(int(c.sum()) for c in self.clear.values())


def run_plan(runner, case, plan):
    """``plan``: steps ``{request: tokens to feed}``; 0 closes a request.  Returns logits per request."""
    from pylon_amd.engine import StepEntry

    live, pos = {}, {rid: 0 for rid in case.requests}
    got = {rid: [] for rid in case.requests}
    for step in plan:
        entries = []
        for rid, size in step.items():
            if size == 0:
                runner.close(live.pop(rid))
                continue
            if rid not in live:
                live[rid] = runner.open(rid)
            chunk = case.requests[rid][pos[rid]: pos[rid] + size]
            entries.append((rid, StepEntry(live[rid], chunk, list(range(len(chunk))))))
            pos[rid] += len(chunk)
        if entries:
            logits = runner.step([e for _, e in entries]).cpu().numpy()
            cursor = 0
            for rid, e in entries:
                got[rid].append(logits[cursor: cursor + len(e.tokens)])
                cursor += len(e.tokens)
        runner.manager.check()
    for seq in live.values():
        runner.close(seq)
    return {rid: np.concatenate(parts) for rid, parts in got.items() if parts}, pos


@pytest.mark.parametrize("name, page", [("A", 16), ("B", 64), ("C", 16), ("D", 32), ("E", 16)])
def test_the_stream_after_every_layer_run(tmp, name, page):
    """The residual stream after every run of a layer, in float32, for a whole prompt and in two portions."""
    from pylon_amd.engine import StepEntry
    from pylon_amd.parts import summed

    case = Case(tmp, name, "float32", (45,))
    runner = case.runner(page_size=page, num_pages=8)
    kept = []

    def watch(block):
        def wrapped(*args, inner=block.forward):
            resid, delta = inner(*args)
            kept.append((resid + summed(delta)).cpu().numpy())
            return resid, delta
        block.forward = wrapped

    for block in runner.model.blocks:
        watch(block)
    toks = case.requests["r0"]
    _, want = plain.forward(case.cfg, case.weights, toks, keep_layers=True)
    seq = runner.open("a")
    runner.step([StepEntry(seq, toks, list(range(len(toks))))])
    runner.close(seq)
    assert len(kept) == len(want)
    for run, (got, ref) in enumerate(zip(kept, want)):
        assert np.abs(got - ref).max() <= 1e-4 * np.abs(ref).max(), f"run {run}"
    kept.clear()
    seq = runner.open("b")
    runner.step([StepEntry(seq, toks[:19], list(range(19)))])
    runner.step([StepEntry(seq, toks[19:], list(range(len(toks) - 19)))])
    for run, ref in enumerate(want):
        got = np.concatenate([kept[run], kept[len(want) + run]])
        assert np.abs(got - ref).max() <= 1e-4 * np.abs(ref).max(), f"run {run}, two portions"


@pytest.mark.parametrize("name, dtype, page", [("A", "float32", 16), ("B", "float32", 16), ("C", "float32", 16),
                                                ("D", "float32", 32), ("E", "float32", 16), ("A", "bfloat16", 16),
                                                ("B", "bfloat16", 64), ("B", "bfloat16", 32), ("C", "bfloat16", 64),
                                                ("D", "bfloat16", 64), ("E", "bfloat16", 32)])
def test_whole_token_by_token_and_in_portions(tmp, name, dtype, page):
    case = Case(tmp, name, dtype, (71, 38))
    assert case.compared() >= 60
    runner = case.runner(page_size=page, num_pages=640 // page)
    whole, _ = run_plan(runner, case, [{"r0": 71}, {"r0": 0, "r1": 38}])
    for rid, got in whole.items():
        case.check(rid, got, "whole")
    single, _ = run_plan(runner, case, [{"r1": 1} for _ in range(38)])
    case.check("r1", single["r1"], "token by token")
    cut, _ = run_plan(runner, case, [{"r0": n} for n in (2, 3, 2, 17, 1, 1, 30, 2, 13)])
    case.check("r0", cut["r0"], "portions")
    if dtype == "float32":  # how a request is cut moves nothing but the order of a product's sums
        assert np.abs(cut["r0"] - whole["r0"]).max() <= 2e-5 * np.abs(whole["r0"]).max()
        assert np.abs(single["r1"] - whole["r1"]).max() <= 2e-5 * np.abs(whole["r1"]).max()


@pytest.mark.parametrize("name, dtype, page", [("A", "float32", 16), ("B", "float32", 16), ("D", "float32", 16), ("E", "float32", 16),
                                                ("C", "bfloat16", 16), ("B", "bfloat16", 32), ("D", "bfloat16", 64)])
def test_mixed_batches_over_pages_and_slots_that_are_used_again(tmp, name, dtype, page):
    case = Case(tmp, name, dtype, (60, 45, 33, 20))
    pages = {16: 9, 32: 6, 64: 4}[page]  # never room for all four requests at once
    runner = case.runner(page_size=page, num_pages=pages, max_requests=3)
    plan = [{"r0": 20}, {"r0": 1, "r1": 30}, {"r0": 2, "r1": 1, "r2": 5}, {"r0": 1, "r1": 1, "r2": 1},
            {"r0": 20, "r1": 13, "r2": 2}, {"r1": 0, "r0": 1, "r2": 1}, {"r3": 17, "r0": 15, "r2": 24},
            {"r2": 0, "r0": 0, "r3": 1}, {"r3": 2}]
    got, pos = run_plan(runner, case, plan)
    assert pos == {"r0": 60, "r1": 45, "r2": 33, "r3": 20}
    for rid, logits in got.items():
        case.check(rid, logits, "mixed")
    alone, _ = run_plan(runner, case, [{"r3": 20}])
    if dtype == "float32":
        assert np.abs(alone["r3"] - got["r3"]).max() <= 2e-5 * np.abs(alone["r3"]).max()
    assert runner.manager.free_pages == pages and runner.manager.slots.free_slots == 3


@pytest.mark.parametrize("name, dtype", [("B", "float32"), ("B", "bfloat16"), ("A", "float32")])
def test_long_decoding_after_a_prompt(tmp, name, dtype):
    """420 tokens, 320 of them one by one: every pass's state goes through hundreds of single steps, windows of
    50 and 100 positions (or 7 and 5) move over decoded tokens, and the pages they have left go back."""
    case = Case(tmp, name, dtype, (420,))
    runner = case.runner(page_size=64, num_pages=7, max_requests=2)
    got, _ = run_plan(runner, case, [{"r0": 100}] + [{"r0": 1}] * 320)
    case.check("r0", got["r0"], "long decoding")
    assert runner.manager.free_pages == 7


def test_requests_do_not_see_what_a_freed_slot_or_page_held(tmp):
    """The same request, alone in a fresh runner and after others have used every page and slot."""
    case = Case(tmp, "A", "float32", (50, 64, 64))
    fresh, _ = run_plan(case.runner(num_pages=8, max_requests=2), case, [{"r0": 50}])
    runner = case.runner(num_pages=8, max_requests=2)
    for tensor in runner.manager.slots.tensors.values():
        tensor.fill_(float("nan"))
    for group in runner.manager.groups:
        for cache in list(group.k.values()) + [v for v in group.v.values() if v is not None]:
            cache.fill_(float("nan"))
    used, _ = run_plan(runner, case, [{"r1": 64, "r2": 64}, {"r1": 0, "r2": 0}, {"r0": 25}, {"r0": 25}])
    assert np.abs(used["r0"] - fresh["r0"]).max() <= 2e-5 * np.abs(fresh["r0"]).max()


def test_the_first_tokens_of_a_sequence_start_from_nothing(tmp):
    """Position 0 sees itself and the sink alone and its states start empty: its logits are those of a one-token
    request, whatever ran in its slot before."""
    case = Case(tmp, "D", "float32", (9, 30))
    runner = case.runner(num_pages=8, max_requests=1)
    first, _ = run_plan(runner, case, [{"r1": 30}, {"r1": 0}, {"r0": 1}])
    want = plain.forward(case.cfg, case.weights, case.requests["r0"][:1])
    assert np.abs(first["r0"] - want).max() <= F32_BOUND * np.abs(want).max()
    two, _ = run_plan(runner, case, [{"r0": 2}])
    assert np.abs(two["r0"] - case.want["r0"][:2]).max() <= F32_BOUND * np.abs(want).max()


def test_a_long_request_whole_and_with_its_tail_decoded(tmp):
    """700 tokens over eleven pages of 64: attention without a window looks back over all of them, the states
    have gone through all of them."""
    case = Case(tmp, "D", "float32", (700,))
    runner = case.runner(page_size=64, num_pages=12, max_requests=1)
    whole, _ = run_plan(runner, case, [{"r0": 700}])
    case.check("r0", whole["r0"], "whole")
    tail, _ = run_plan(runner, case, [{"r0": 650}] + [{"r0": 1}] * 50)
    case.check("r0", tail["r0"], "tail decoded")


@pytest.mark.parametrize("name, dtype, graphs, page", [("A", "float32", False, 16), ("B", "float32", True, 16),
                                                         ("C", "bfloat16", True, 64), ("B", "bfloat16", True, 32),
                                                         ("D", "bfloat16", True, 64), ("E", "float32", True, 16)])
def test_greedy_generation_through_the_engine(tmp, name, dtype, graphs, page):
    from pylon_amd.engine.engine import Engine
    from pylon_amd.sampling import Sampling

    folder = make_folder(tmp, name, dtype=dtype, seed=8)
    cfg, weights = read_folder(folder)
    prompts = [tokens(cfg["vocab"], n, 70 + n) for n in (3, 19, 41)]
    engine = Engine.from_folder(folder, dtype=dtype, page_size=page, num_pages=384 // page, max_batch_size=3,
                                prefill_chunk_size=16, cuda_graphs=graphs)
    try:
        results = engine.generate(prompts, Sampling(max_new_tokens=12, temperature=0.0))
    finally:
        engine.close()
    slack = 1e-4 if dtype == "float32" else 5e-2
    for prompt, result in zip(prompts, results):
        assert len(result.output_ids) == 12
        sequence = list(prompt)
        for produced in result.output_ids:
            margins = []
            row = plain.forward(cfg, weights, sequence, margins=margins)[-1]
            if dtype != "float32" and margins and np.min(margins) < ROUTER_MARGIN:
                break  # a router's close call somewhere before: from here on rounding decides
            assert produced == int(row.argmax()) or row.max() - row[produced] <= slack * np.abs(row).max(), \
                (prompt[:3], result.output_ids)
            sequence.append(produced)


def test_decode_graphs_replayed_beside_eager_steps(tmp):
    """A captured decode step, replayed over many tokens, gives what the eager step gives: the pass entries,
    the lightning states and the norm with gates write where the graph expects them."""
    from pylon_amd.engine.engine import Engine
    from pylon_amd.sampling import Sampling

    folder = make_folder(tmp, "B", dtype="bfloat16", seed=12)
    prompts = [tokens(CONFIGS["B"]["vocab"], n, n) for n in (5, 30)]
    outputs = []
    for graphs in (False, True):
        engine = Engine.from_folder(folder, dtype="bfloat16", page_size=64, num_pages=8, max_batch_size=2,
                                    prefill_chunk_size=64, cuda_graphs=graphs)
        try:
            outputs.append([r.output_ids for r in engine.generate(prompts, Sampling(max_new_tokens=60, temperature=0.0))])
        finally:
            engine.close()
    assert outputs[0] == outputs[1]


@pytest.mark.parametrize("name, dtype", [("B", "float32"), ("D", "float32"), ("B", "bfloat16")])
def test_the_replay_program_as_a_user_runs_it(tmp, tmp_path, name, dtype):
    """``bin/trace_run`` as a subprocess over pages of 64 and four slots: up to four live requests, portions of
    some beside single tokens of others, pages and slots used again; the logits files against the plain model."""
    import json
    import os
    import subprocess
    import sys
    from pathlib import Path

    from tests import traces

    root = Path(__file__).resolve().parent.parent
    case = Case(tmp, name, dtype, (5, 90, 64, 33, 70, 1), seed=11)
    steps = traces.mixed(case.requests, seed=7)
    out = tmp_path / "out"
    proc = subprocess.Popen(
        [sys.executable, str(root / "bin" / "trace_run"), "--model", str(case.folder), "--dtype", dtype,
         "--out", str(out), "--max-tokens", str(traces.peak_tokens(steps))],
        stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True, cwd=str(tmp_path),
        env=dict(os.environ, PYTHONUNBUFFERED="1"))
    try:
        for step in steps:
            proc.stdin.write(json.dumps(step) + "\n")
            proc.stdin.flush()
            assert proc.stdout.readline().strip() == f"done {step['step']}"
        proc.stdin.close()
        assert proc.wait(timeout=60) == 0
    finally:
        if proc.poll() is None:
            proc.kill()
    vocab = case.cfg["vocab"]
    outputs = {}
    for step in steps:
        wanted = sum(len(e["want"]) for e in step["entries"])
        if wanted:
            outputs[step["step"]] = np.fromfile(out / f"{step['step']}.f32", dtype="<f4").reshape(wanted, vocab)
    got = traces.collect(steps, outputs, vocab)
    for rid in case.requests:
        assert len(got[rid]) == len(case.requests[rid])
        case.check(rid, np.asarray(got[rid]), "replayed")


def draw_config(seed: int):
    """A configuration drawn over what config.json allows: layers in any order, heads and sizes in steps of 8
    and a few odd ones, windows that are no multiple of anything, with and without stretched frequencies,
    groups, shared experts, loops and feed-forwards."""
    rng = np.random.default_rng(8100 + seed)
    width = int(rng.choice([48, 64, 96, 136, 160, 256]))
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        if rng.random() < 0.5:
            kv_heads = int(rng.integers(1, 4))
            dim = int(rng.choice([8, 16, 24, 32, 40, 64, 96, 128, 12]))
            m = {"heads": kv_heads * int(rng.choice([1, 2, 3, 4, 8])), "kv_heads": kv_heads, "dim": dim,
                 "vdim": int(rng.choice([4, 8, 20, 32, 48, 64, 80, 128, 10])), "scale": float(rng.uniform(0.05, 0.4)),
                 "mask": {"size": int(rng.choice([int(rng.integers(3, 200)), 32, 64, 128, 1000]))}}
            dims = int(rng.choice([d for d in (2, 4, 8, 16, 32, 64, 128, dim) if d <= dim and d % 2 == 0]))
            m["rot"] = {"base": float(rng.choice([100.0, 1.0e4, 5.0e5, 1.0e6])), "dims": dims}
            if rng.random() < 0.8:
                m["rot"]["scaling"] = {"factor": float(rng.choice([2.0, 8.0, 32.0])), "low": float(rng.choice([1.0, 2.0])),
                                       "high": float(rng.choice([4.0, 6.0])), "original": int(rng.choice([16, 64, 2048]))}
            kind = "attention"
        else:
            heads = int(rng.integers(1, 7))
            m = {"heads": heads, "dim": int(rng.choice([8, 20, 32, 64, 96, 128])), "vdim": int(rng.choice([8, 12, 32, 64, 128])),
                 "decay": (1.0 - 10.0 ** rng.uniform(-3.5, -0.3, size=heads)).tolist()}
            kind = "lightning"
        mlp = None
        if rng.random() < 0.5:
            mlp = {"kind": "dense", "ff": 8 * int(rng.integers(1, 30))}
        elif rng.random() < 0.8:
            count = int(rng.integers(1, 5))
            experts, keep = count * int(rng.integers(1, 5)), int(rng.integers(1, count + 1))
            mlp = {"kind": "moe", "expert": {"ff": 8 * int(rng.integers(1, 12))},
                   "router": {"experts": experts, "top": int(rng.integers(1, min(experts // count * keep, 4) + 1)),
                              "groups": {"count": count, "keep": keep}}}
            if rng.random() < 0.7:
                mlp["shared"] = {"ff": 8 * int(rng.integers(1, 12))}
        layers.append({"type": kind, "mixer": m, "mlp": mlp})
    config = {"architecture": "Farorax", "vocab": int(rng.integers(90, 700)), "width": width,
              "norm": {"eps": float(10 ** rng.uniform(-7, -4))}, "layers": layers, "residual_mult": float(rng.uniform(0.2, 1.2))}
    if rng.random() < 0.8:
        start = int(rng.integers(0, len(layers)))
        config["loop"] = {"start": start, "stop": int(rng.integers(start + 1, len(layers) + 1)), "times": int(rng.integers(1, 4))}
    if rng.random() < 0.8:
        config["logit_softcap"] = float(rng.choice([5.0, 20.0, 50.0]))
    return config, (int(rng.integers(1, 40)), int(rng.integers(60, 200)), int(rng.integers(200, 330)))


@pytest.mark.parametrize("seed, dtype", [(seed, "float32") for seed in range(10)] + [(seed, "bfloat16") for seed in range(4)])
def test_a_configuration_drawn_at_random_matches_the_plain_model(tmp, seed, dtype):
    """Pages of 64 and four slots: each request whole, the longest with its tail token by token, then all three
    side by side in portions over a pool too small for them to have pages to spare."""
    config, lengths = draw_config(seed)
    if dtype != "float32":
        # shorter requests, drawn token by token so that the positions' routing is clear
        lengths = (lengths[0], min(lengths[1], 70), min(lengths[2], 90))
    case = Case(tmp, f"drawn{seed}", dtype, lengths, seed=seed, config=config, pick=dtype != "float32")
    if case.compared() < 40:
        pytest.skip("too few positions with clear routing in this draw")
    pages = sum(-(-n // 64) for n in lengths)
    runner = case.runner(page_size=64, num_pages=pages, max_requests=4)
    whole, _ = run_plan(runner, case, [{"r0": lengths[0]}, {"r0": 0, "r1": lengths[1]}, {"r1": 0, "r2": lengths[2]}])
    for rid, got in whole.items():
        case.check(rid, got, f"whole (seed {seed})")
    tail, _ = run_plan(runner, case, [{"r2": lengths[2] - 70}] + [{"r2": 1}] * 70 if lengths[2] > 70 else [{"r2": 1}] * lengths[2])
    assert len(tail["r2"]) == lengths[2]
    case.check("r2", tail["r2"], f"decoded tail (seed {seed})")
    plan, left = [], dict(zip(("r0", "r1", "r2"), lengths))
    sizes = iter(np.random.default_rng(seed).choice([1, 2, 3, 7, 31, 64, 65, 100], size=200).tolist())
    while any(left.values()):
        step = {}
        for rid in left:
            if left[rid]:
                step[rid] = min(left[rid], next(sizes))
                left[rid] -= step[rid]
        plan.append(step)
    mixed, _ = run_plan(runner, case, plan)
    for rid, got in mixed.items():
        case.check(rid, got, f"portions side by side (seed {seed})")
        if dtype == "float32":
            assert np.abs(got - whole[rid]).max() <= 2e-5 * np.abs(whole[rid]).max(), (seed, rid)
    assert runner.manager.free_pages == pages
