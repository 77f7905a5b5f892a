"""Ranudra on the GPU against the plain implementation: every mechanism's kernel alone, then
whole models cut every way (whole prompts, token by token, portions down to two tokens, mixed
batches over pages and slots that are used again), long decoding, and greedy generation
through the engine."""
import numpy as np
import pytest
import torch

from tests.helpers import rows_within
from tests.plain import ranudra as plain
from tests.ranudra_helpers import CONFIGS, make_folder, read_folder, tokens

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
F32_BOUND = 2e-4   # of a row's largest |logit|
BF16_BOUND = 1e-1


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
    return tmp_path_factory.mktemp("ranudra")


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


# ---- the residual stream's copies and the layer norm ---------------------------------------------------

@pytest.mark.parametrize("copies", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("dim", [40, 256, 100, 2560, 5124, 33])
def test_copies_of_the_stream_are_mixed_read_and_normed_in_one_kernel(ops, copies, dim):
    rng = np.random.default_rng(copies * 10000 + dim)
    n = 5
    x = rng.normal(size=(copies, n, dim)) + 0.7
    mix, write, read = rng.normal(size=(copies, copies)), rng.normal(size=copies), rng.normal(size=copies)
    w = 1.0 + 0.3 * rng.normal(size=dim)
    eps = 1e-5
    for parts, dtype in ((1, torch.float32), (1, torch.bfloat16), (2, torch.float32), (7, torch.float32)):
        d = rounded(rng.normal(size=(parts, n, dim)), dtype)
        delta = dev(d if parts > 1 else d[0], dtype)
        y = d.sum(axis=0)
        renewed = np.einsum("st,snd->tnd", mix, x) + write[:, None, None] * y
        u = np.einsum("s,snd->nd", read, renewed)
        for centre, norm in ((True, plain.layer_norm), (False, plain.rms_norm)):
            for out_dtype, bound in ((torch.float32, 2e-5), (torch.bfloat16, 5e-3)):
                resid = dev(x if copies > 1 else x[0])
                got = ops.stream_norm(resid, delta, dev(w), eps, out_dtype, centre=centre, mix=dev(mix), write=dev(write),
                                      read=dev(read))
                close(got.float().cpu().numpy(), norm(u, w, eps), bound, f"{parts} parts, centre {centre}")
                close(resid.cpu().numpy().reshape(x.shape), renewed, 1e-5, "the copies")
        # some rows only: the copies stay as they were; without coefficients the sum of the copies is read
        resid = dev(x if copies > 1 else x[0])
        got = ops.stream_norm(resid, delta, dev(w), eps, torch.float32, centre=True, mix=dev(mix), write=dev(write),
                              row_idx=i32([4, 1, 1]))
        close(got.cpu().numpy(), plain.layer_norm(renewed.sum(axis=0), w, eps)[[4, 1, 1]], 3e-5, "picked rows")
        close(resid.cpu().numpy().reshape(x.shape), x, 1e-6, "untouched")
        # an ordinary residual sum
        got = ops.stream_norm(resid, delta, dev(w), eps, torch.float32, centre=True, read=dev(read))
        close(resid.cpu().numpy().reshape(x.shape), x + y, 1e-5, "plain sum")
        close(got.cpu().numpy(), plain.layer_norm(np.einsum("s,snd->nd", read, x + y), w, eps), 3e-5, "plain sum's norm")
    resid = dev(x if copies > 1 else x[0])
    got = ops.stream_norm(resid, None, dev(w), eps, torch.float32, centre=True, read=dev(read))
    close(got.cpu().numpy(), plain.layer_norm(np.einsum("s,snd->nd", read, x), w, eps), 2e-5, "nothing to add")


def test_the_layer_norm_of_a_row_far_from_zero_keeps_its_deviations(ops):
    """The variance comes from the deviations, not from a difference of two large numbers."""
    rng = np.random.default_rng(0)
    x = rng.normal(size=(3, 512)).astype(np.float32).astype(np.float64) * 0.01 + 300.0
    x = x.astype(np.float32).astype(np.float64)
    got = ops.stream_norm(dev(x), None, dev(np.ones(512)), 1e-6, torch.float32, centre=True)
    close(got.cpu().numpy(), plain.layer_norm(x, 1.0, 1e-6), 5e-3)


def test_the_embedded_tokens_in_several_copies(ops):
    rng = np.random.default_rng(1)
    for dtype in (torch.float32, torch.bfloat16):
        table = rounded(rng.normal(size=(50, 36)), dtype)
        ids = rng.integers(0, 50, 7)
        for copies in (1, 2, 5):
            got = ops.embed(i32(ids), dev(table, dtype), scale=16.0, copies=copies).cpu().numpy().reshape(copies, 7, 36)
            for c in range(copies):
                close(got[c], table[ids] * 16.0, 1e-7)


@pytest.mark.parametrize("count", [1, 7, 64, 1000])
def test_squared_relu(ops, count):
    rng = np.random.default_rng(count)
    for a in (torch.float32, torch.bfloat16):
        for b in (torch.float32, torch.bfloat16):
            x = rounded(rng.normal(size=(3, count)), a)
            got = ops.relu2(dev(x, a), out_dtype=b).float().cpu().numpy()
            close(got, np.maximum(x, 0.0) ** 2, 1e-6 if b == torch.float32 else 5e-3)


@pytest.mark.parametrize("rows", [1, 5, 16, 17, 64, 65, 128, 200])
@pytest.mark.parametrize("width, ff", [(64, 88), (256, 512), (100, 44), (2560, 384)])
def test_a_product_with_squared_relu(ops, rows, width, ff):
    rng = np.random.default_rng(rows + width)
    for dtype, bound in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        x, w = rounded(rng.normal(size=(rows, width)), dtype), rounded(rng.normal(size=(ff, width)) * width ** -0.5, dtype)
        got = ops.linear_relu2(dev(x, dtype), dev(w, dtype), out_dtype=dtype).float().cpu().numpy()
        close(got, np.maximum(x @ w.T, 0.0) ** 2, bound, str(dtype))


# ---- gated linear attention --------------------------------------------------------------------------

def plain_gla_outputs(q, k, v, gate, low, a2, bias, norm_w, heads, dim, vdim, tau, eps):
    n = q.shape[0]
    decay = (plain.sigmoid(low @ a2.T + bias) ** (1.0 / tau)).reshape(n, heads, dim)
    o = plain.gated_linear_attention(q.reshape(n, heads, dim) * dim ** -0.5, k.reshape(n, heads, dim),
                                     v.reshape(n, heads, vdim), decay)
    return plain.rms_norm(o, norm_w, eps).reshape(n, -1) * plain.silu(gate)


GLA_SHAPES = [(3, 32, 32), (2, 12, 20), (3, 64, 128), (2, 128, 128), (1, 256, 64), (2, 128, 32), (1, 100, 24), (5, 1, 1),
              (2, 48, 200), (1, 32, 256), (1, 64, 16), (2, 96, 80)]


@pytest.mark.parametrize("strong", [False, True])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, dim, vdim", GLA_SHAPES)
def test_gated_linear_attention_in_portions_of_two_requests_over_reused_slots(ops, heads, dim, vdim, dtype, strong):
    """Two requests of 201 and 23 tokens in portions of changing size, single tokens among them, in
    slots that held other numbers before; decays close to one (a state lost between two portions is
    missed), or so strong that a channel is gone after a token or two."""
    rng = np.random.default_rng(heads * 1000 + dim + vdim)
    lengths = {"x": 201, "y": 23}
    qk, vv, rank, tau = heads * dim, heads * vdim, 8 if strong else 5, 3.0  # rows of the projection that are whole 16-byte pieces, or not
    data = {rid: {name: rounded(rng.normal(size=(n, size)), dtype) for name, size in
                  (("q", qk), ("k", qk), ("v", vv), ("gate", vv), ("low", rank))} for rid, n in lengths.items()}
    a2 = rng.normal(size=(qk, rank)).astype(np.float32).astype(np.float64) * (20.0 if strong else 1.0)
    bias = (rng.normal(size=qk) * 2 + (0.0 if strong else 5.0)).astype(np.float32).astype(np.float64)
    if strong:
        tau = 0.7
    norm_w = 1.0 + 0.3 * rng.normal(size=vdim)
    eps = 1e-5
    want = {rid: plain_gla_outputs(d["q"], d["k"], d["v"], d["gate"], d["low"], a2, bias, norm_w, heads, dim, vdim, tau, eps)
            for rid, d in data.items()}
    state = torch.full((3, heads, dim, vdim), 9.0, device=DEV)
    slots = {"x": 2, "y": 0}
    for slot in slots.values():
        state[slot].zero_()  # what the manager does when it hands a slot out
    plan = [{"x": 5}, {"x": 1, "y": 2}, {"y": 1}, {"x": 18, "y": 1}, {"x": 1}, {"y": 19, "x": 16}, {"x": 2}, {"x": 130}, {"x": 28}]
    pos = {rid: 0 for rid in lengths}
    got = {rid: [] for rid in lengths}
    for number, step in enumerate(plan):
        rows, parts, starts = [], [], [0]
        for rid, count in step.items():
            d, p = data[rid], pos[rid]
            parts.append(np.concatenate([d[name][p: p + count] for name in ("q", "k", "v", "gate", "low")], axis=1))
            rows.append(rid)
            starts.append(starts[-1] + count)
            pos[rid] += count
        out = ops.gla(dev(np.concatenate(parts), dtype), state, dev(a2), dev(bias), dev(norm_w), i32(starts),
                      i32(slots[r] for r in rows), rows=len(rows), heads=heads, dim=dim, vdim=vdim, rank=rank, tau=tau,
                      eps=eps, q_scale=dim ** -0.5, max_count=max(step.values()))
        out = out.float().cpu().numpy()
        for i, rid in enumerate(rows):
            got[rid].append(out[starts[i]: starts[i + 1]])
    assert pos == lengths
    assert float(state[1].min()) == 9.0  # nobody's slot
    for rid in lengths:
        close(np.concatenate(got[rid]), want[rid], 1e-4 if dtype == torch.float32 else 1e-2, rid)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows, count", [(1, 400), (7, 90), (40, 33), (2, 1500)])
def test_gated_linear_attention_over_many_and_long_rows(ops, rows, count, dtype):
    """However the kernel shares a step's rows and their pieces between workgroups."""
    rng = np.random.default_rng(rows)
    heads, dim, vdim, rank, tau, eps = 2, 64, 48, 8, 6.0, 1e-6
    qk, vv = heads * dim, heads * vdim
    a2, bias = dev(rng.normal(size=(qk, rank))), dev(rng.normal(size=qk) + 3.0)
    norm_w = dev(1 + 0.2 * rng.normal(size=vdim))
    n = rows * count
    proj = dev(rng.normal(size=(n, 2 * qk + 2 * vv + rank)), dtype)
    state = torch.zeros((rows + 2, heads, dim, vdim), device=DEV)
    state[:rows].copy_(dev(rng.normal(size=(rows, heads, dim, vdim))))
    before = state.clone()
    slots = list(rng.permutation(rows))
    args = dict(heads=heads, dim=dim, vdim=vdim, rank=rank, tau=tau, eps=eps, q_scale=dim ** -0.5)
    got = ops.gla(proj, state, a2, bias, norm_w, i32(range(0, n + 1, count)), i32(slots), rows=rows, max_count=count, **args)
    # the same rows one at a time through the token-by-token kernel in float32
    again = before.clone()
    want = ops.gla_recurrent(proj.float(), again, a2, bias, norm_w, i32(range(0, n + 1, count)), i32(slots), rows=rows, **args)
    close(got.float().cpu().numpy(), want.cpu().numpy(), 1e-5 if dtype == torch.float32 else 1e-2)
    close(state.cpu().numpy(), again.cpu().numpy(), 1e-4)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gated_linear_attention_keeps_what_it_wrote_far_back(ops, dtype):
    """With decays of one on the channel of token 3's key (and decays of almost zero on another), the
    state answers that key with token 3's value 300 tokens later, in a prompt and token by token."""
    n, dim, vdim, rank = 320, 64, 16, 1
    rng = np.random.default_rng(3)
    keys = np.zeros((n, dim))
    keys[np.arange(n), np.arange(n) % (dim - 2) + 2] = 1.0  # never channels 0 and 1 ...
    keys[3] = 0.0
    keys[3, :2] = 1.0                                        # ... except token 3
    values = rounded(rng.normal(size=(n, vdim)), dtype)
    queries = np.zeros((n, dim))
    queries[-1, :2] = 1.0                                    # reads both: channel 1 has been forgotten
    proj = np.concatenate([queries, keys, values, np.full((n, vdim), 30.0), np.ones((n, rank))], axis=1)
    bias = np.full(dim, 80.0)
    bias[1] = -5.0
    want = values[3] / np.sqrt((values[3] ** 2).mean() + 1e-6) * 30.0
    args = dict(rows=1, heads=1, dim=dim, vdim=vdim, rank=rank, tau=1.0, eps=1e-6, q_scale=1.0)
    a2, norm_w = dev(np.zeros((dim, rank))), dev(np.ones(vdim))
    state = torch.zeros((1, 1, dim, vdim), device=DEV)
    out = ops.gla(dev(proj, dtype), state, a2, dev(bias), norm_w, i32([0, n]), i32([0]), max_count=n, **args)
    bound = 1e-4 if dtype == torch.float32 else 5e-3
    close(out[-1].float().cpu().numpy(), want, bound, "whole")
    state.zero_()
    for t in range(n):
        out = ops.gla(dev(proj[t: t + 1], dtype), state, a2, dev(bias), norm_w, i32([0, 1]), i32([0]), max_count=1, **args)
    close(out[-1].float().cpu().numpy(), want, bound, "token by token")


# ---- latent attention ----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, dim, rot, rank, vdim, scaled", [(3, 10, 6, 18, 14, True), (6, 24, 32, 64, 40, True),
                                                                  (7, 16, 64, 120, 72, False), (1, 8, 2, 8, 4, False)])
def test_rows_and_queries_of_latent_attention(ops, heads, dim, rot, rank, vdim, scaled, dtype):
    """The latent normed and the shared key part rotated into scattered slots, the queries' rotated
    parts turned and their other parts carried into the latent's space (few tokens and many)."""
    from pylon_amd.config.specs import PositionSpec, RotaryScalingSpec
    from pylon_amd.parts.position import RotaryPosition

    rng = np.random.default_rng(dim + rank)
    raw = {"base": 5000.0, "dims": rot}
    if scaled:
        raw["scaling"] = {"factor": 4.0, "original": 300, "fast": 16.0, "slow": 1.0}
    part = RotaryPosition(PositionSpec(kind="rope", theta=raw["base"], rotary_dim=rot, interleaved=True,
                                       scaling=RotaryScalingSpec(**raw["scaling"]) if scaled else None), dtype=dtype, device=DEV)
    for n, first in ((9, 0), (70, 1000)):
        q_size, extra = heads * (dim + rot), 3
        proj = rounded(rng.normal(size=(n, q_size + rank + rot + extra)), dtype)
        c_w, uk = 1 + 0.3 * rng.normal(size=rank), rounded(rng.normal(size=(heads, dim, rank)) * dim ** -0.5, dtype)
        slots = rng.permutation(96)[:n]
        cache = torch.full((6, 16, 1, rank + rot), 7.0, dtype=dtype, device=DEV)
        q_out = torch.full((n, heads, rank + rot), 5.0, dtype=dtype, device=DEV)
        moved = dev(proj, dtype)
        ops.latent_rotate(moved, q_out, cache, i32(slots), q_off=0, n_heads=heads, head_dim=dim, rot_dim=rot, c_off=q_size,
                          kv_rank=rank, c_weight=dev(c_w), eps=1e-5, inv_freq=part.inv_freq, rot_scale=part.rot_scale,
                          interleaved=True, positions=i32(range(first, first + n)))
        q = proj[:, :q_size].reshape(n, heads, dim + rot)
        unrotated = moved[:, :q_size].view(n, heads, dim + rot)[..., :dim]
        ops.head_project(unrotated, dev(uk, dtype), out=q_out[..., :rank],
                         by_output=dev(uk, dtype).transpose(1, 2).contiguous() if n == 9 else None)
        want_q = np.concatenate([np.einsum("thd,hdr->thr", q[..., :dim], uk), plain.rotate(q[..., dim:], raw, first)], axis=2)
        want_row = np.concatenate([plain.rms_norm(proj[:, q_size: q_size + rank], c_w, 1e-5),
                                   plain.rotate(proj[:, q_size + rank: q_size + rank + rot], raw, first)], axis=1)
        bound = 3e-4 if dtype == torch.float32 else 1e-2
        close(q_out.float().cpu().numpy(), want_q, bound, "queries")
        flat = cache.view(96, rank + rot).float().cpu().numpy()
        close(flat[slots], want_row, bound, "rows")
        others = np.setdiff1d(np.arange(96), slots)
        assert (flat[others] == 7.0).all()
        # without a rotation the parts are copied
        ops.latent_rotate(moved, q_out, cache, i32(slots), q_off=0, n_heads=heads, head_dim=dim, rot_dim=rot, c_off=q_size,
                          kv_rank=rank, c_weight=dev(c_w), eps=1e-5, inv_freq=None, rot_scale=1.0, interleaved=True,
                          positions=i32(range(n)))
        assert np.array_equal(cache.view(96, rank + rot).float().cpu().numpy()[slots, rank:], proj[:, q_size + rank: q_size + rank + rot])
        assert np.array_equal(q_out[..., rank:].float().cpu().numpy(), q[..., dim:])


@pytest.mark.parametrize("n", [1, 7, 64, 65, 200])
@pytest.mark.parametrize("heads, rank, vdim", [(3, 18, 14), (5, 64, 32), (8, 136, 80), (2, 512, 16)])
def test_values_of_the_heads_with_gates_per_head_and_per_element(ops, heads, rank, vdim, n):
    rng = np.random.default_rng(n + rank)
    for dtype, bound in ((torch.float32, 2e-5), (torch.bfloat16, 1.5e-2)):
        x, m = rounded(rng.normal(size=(n, heads, rank)), dtype), rounded(rng.normal(size=(heads, rank, vdim)) * rank ** -0.5, dtype)
        wide = rounded(rng.normal(size=(n, 8 + heads * vdim)), dtype)
        plainly = np.einsum("thr,hrv->thv", x, m)
        got = ops.head_project(dev(x, dtype), dev(m, dtype), gate_logits=dev(wide, dtype)[:, 8: 8 + heads])
        close(got.float().cpu().numpy(), plainly * plain.sigmoid(wide[:, 8: 8 + heads])[:, :, None], bound, "per head")
        got = ops.head_project(dev(x, dtype), dev(m, dtype), gate_logits=dev(wide, dtype)[:, 8:])
        close(got.float().cpu().numpy(), plainly * plain.sigmoid(wide[:, 8:]).reshape(plainly.shape), bound, "per element")
        # with the matrix also output by output: the matrix cores where the sizes allow
        turned = dev(m, dtype).transpose(1, 2).contiguous()
        got = ops.head_project(dev(x, dtype), dev(m, dtype), gate_logits=dev(wide, dtype)[:, 8:], by_output=turned)
        close(got.float().cpu().numpy(), plainly * plain.sigmoid(wide[:, 8:]).reshape(plainly.shape), bound, "by output")
        gate = rng.uniform(size=(n, heads))
        got = ops.head_project(dev(x, dtype), dev(m, dtype), gate=dev(gate), by_output=turned)
        close(got.float().cpu().numpy(), plainly * gate[:, :, None], bound, "float gates")
        if n > 1 and n <= 64:  # a token's result does not depend on its batch
            one = ops.head_project(dev(x[-1:], dtype), dev(m, dtype), gate=dev(gate[-1:]), by_output=turned)
            assert torch.equal(one[0], got[-1])


def planted_rows(rng, n, heads, width, planted):
    """Queries, and rows among which the planted positions stand out along a direction that every query
    has a large share of."""
    direction = rng.normal(size=width)
    direction /= np.linalg.norm(direction)
    q = rng.normal(size=(n, heads, width)) + 4.0 * direction
    rows = rng.normal(size=(n, width)) * 0.5
    for j in planted:
        rows[j] += 6.0 * direction
    return q, rows


@pytest.mark.parametrize("size", [37, 64, 129, 1, 300, None])
@pytest.mark.parametrize("dtype, heads, width, rank, page", [
    (torch.float32, 3, 28, 18, 16), (torch.float32, 2, 96, 64, 64), (torch.float32, 2, 576, 512, 64),
    (torch.bfloat16, 7, 96, 64, 64), (torch.bfloat16, 9, 160, 112, 64), (torch.bfloat16, 3, 56, 40, 128),
    (torch.bfloat16, 17, 128, 96, 64), (torch.bfloat16, 32, 320, 256, 256), (torch.bfloat16, 40, 192, 128, 64),
    (torch.bfloat16, 5, 256, 104, 64), (torch.bfloat16, 16, 384, 248, 64), (torch.bfloat16, 4, 576, 512, 64),
    (torch.bfloat16, 20, 576, 512, 64), (torch.bfloat16, 100, 72, 64, 64), (torch.bfloat16, 1, 8, 8, 64)])
def test_attention_over_rows_at_the_edges_of_windows_and_pages(ops, size, dtype, heads, width, rank, page):
    """A 300-token request whose planted rows lie at position 0, at a page's last and first slot, just
    inside and just outside the window of many queries, and far back; pages scattered over a pool whose
    other slots hold NaN; whole, and as a portion over a cached first part; with and without a sink."""
    rng = np.random.default_rng(17 + (size or 0) + width)
    n = 300
    planted = sorted({0, page - 1, min(page, n - 1), min(2 * page, n - 1), 150, 151} | ({size - 1, size} if size and size < n else set()))
    q, rows = planted_rows(rng, n, heads, width, [j for j in planted if j < n])
    q, rows = rounded(q, dtype), rounded(rows, dtype)
    scale = 0.8 * width ** -0.5
    sink = 4.0 + 2.0 * rng.normal(size=heads)
    k = np.repeat(rows[:, None, :], heads, axis=1)
    mask = plain.visible(n, size)
    want = {True: plain.softmax_attention(q, k, k[..., :rank], scale, mask, sink),
            False: plain.softmax_attention(q, k, k[..., :rank], scale, mask)}
    assert np.abs(want[True] - want[False]).max() > 0.02
    pages = -(-n // page)
    pool = pages + 5
    order = rng.permutation(pool)[:pages]
    cache = torch.full((pool, page, 1, width), float("nan"), dtype=dtype, device=DEV)
    slots = np.array([order[j // page] * page + j % page for j in range(n)])
    cache.view(-1, width)[torch.tensor(slots, device=DEV)] = dev(rows, dtype)
    table = i32(order).view(1, -1)
    bound = 2e-5 if dtype == torch.float32 else 2e-2
    for with_sink, ref in want.items():
        z = dev(sink) if with_sink else None
        for first in (0, 143):
            out = ops.paged_attention(dev(q[first:], dtype), cache, cache, table, i32([0] * (n - first)), i32(range(first, n)),
                                      page_size=page, window=size, scale=scale, sink_logit=z, values_in_keys=rank)
            close(out.float().cpu().numpy(), ref[first:], bound, f"general, from {first}")
        if dtype != torch.bfloat16:
            continue
        assert ops.latent_attention_ok(dtype, width=width, rank=rank, page_size=page)
        options = dict(rank=rank, page_size=page, scale=scale, window=size, sink=z)
        for first in (0, 143):
            for count_rows in (64, 128):
                if count_rows < heads or (count_rows == 128 and rank > 256):
                    continue
                per = count_rows // heads
                tiles = i32(x for a in range(first, n, per) for x in (a - first, min(per, n - a), 0, a)).view(-1, 4)
                out = ops.latent_prefill(dev(q[first:], dtype), cache, table, tiles, rows=count_rows, **options)
                close(out.float().cpu().numpy(), ref[first:], bound, f"tiles of {count_rows} from {first}")
        for cuts in (1, 2, 8):
            out = ops.latent_decode(dev(q, dtype), cache, table.expand(n, -1).contiguous(), i32(range(n)), cuts=cuts, **options)
            close(out.float().cpu().numpy(), ref, bound, f"single tokens, {cuts} cuts")


def test_chunks_and_weights_beyond_bfloat16_over_rows(ops):
    """Chunks in place of a window; and many keys of nearly equal weight, whose sum a weight rounded to
    eight bits would miss by more than the outputs' own rounding allows."""
    rng = np.random.default_rng(5)
    n, heads, width, rank, page = 200, 4, 96, 64, 64
    q, rows = rounded(rng.normal(size=(n, heads, width)), torch.bfloat16), rounded(rng.normal(size=(n, width)), torch.bfloat16)
    rows[:, :rank] = 1.0  # every value the same: the output is 1 whatever the weights are
    cache = torch.zeros((4, page, 1, width), dtype=torch.bfloat16, device=DEV)
    cache.view(-1, width)[:n] = dev(rows, torch.bfloat16)
    table = i32(range(4)).view(1, -1)
    k = np.repeat(rows[:, None, :], heads, axis=1)
    i, j = np.arange(n)[:, None], np.arange(n)[None, :]
    mask = (j <= i) & (i // 50 == j // 50)
    sink = np.full(heads, 1.5)
    want = plain.softmax_attention(q, k, k[..., :rank], 0.1, mask, sink)
    options = dict(rank=rank, page_size=page, scale=0.1, chunk=50, sink=dev(sink))
    tiles = i32(x for a in range(0, n, 16) for x in (a, min(16, n - a), 0, a)).view(-1, 4)
    out = ops.latent_prefill(dev(q, torch.bfloat16), cache, table, tiles, rows=64, **options)
    close(out.float().cpu().numpy(), want, 4.1e-3)
    out = ops.latent_decode(dev(q, torch.bfloat16), cache, table.expand(n, -1).contiguous(), i32(range(n)), cuts=2, **options)
    close(out.float().cpu().numpy(), want, 4.1e-3)


def test_a_sink_that_takes_all_the_weight_and_one_that_takes_none(ops):
    rng = np.random.default_rng(1)
    n, heads, width, rank = 70, 2, 64, 48
    q, rows = rng.normal(size=(n, heads, width)), rng.normal(size=(n, width))
    q, rows = rounded(q, torch.bfloat16), rounded(rows, torch.bfloat16)
    sink = np.array([200.0, -200.0])
    cache = torch.zeros((2, 64, 1, width), dtype=torch.bfloat16, device=DEV)
    cache.view(-1, width)[:n] = dev(rows, torch.bfloat16)
    k = np.repeat(rows[:, None, :], heads, axis=1)
    want = plain.softmax_attention(q, k, k[..., :rank], 0.2, plain.visible(n, None), sink)
    table = i32([0, 1]).view(1, 2)
    tiles = i32(x for a in range(0, n, 32) for x in (a, min(32, n - a), 0, a)).view(-1, 4)
    options = dict(rank=rank, page_size=64, scale=0.2, sink=dev(sink))
    for out in (ops.latent_prefill(dev(q, torch.bfloat16), cache, table, tiles, rows=64, **options),
                ops.latent_decode(dev(q, torch.bfloat16), cache, table.expand(n, -1).contiguous(), i32(range(n)), cuts=1, **options),
                ops.latent_decode(dev(q, torch.bfloat16), cache, table.expand(n, -1).contiguous(), i32(range(n)), cuts=4, **options)):
        got = out.float().cpu().numpy()
        assert np.abs(got[:, 0]).max() < 1e-12
        close(got[:, 1], want[:, 1], 1e-2)


def test_the_row_kernels_refuse_what_they_cannot_do(ops):
    from pylon_amd.kernels import KernelError

    def run(width, rank, page, heads=2, rows=64):
        q = torch.zeros((3, heads, width), dtype=torch.bfloat16, device=DEV)
        cache = torch.zeros((2, page, 1, width), dtype=torch.bfloat16, device=DEV)
        return ops.latent_prefill(q, cache, i32([0, 1]).view(1, 2), i32([0, 3, 0, 0]).view(1, 4), rank=rank, page_size=page,
                                  scale=0.1, rows=rows)

    for width, rank, page in ((60, 32, 64), (640, 512, 64), (96, 96, 32), (64, 72, 64), (600, 64, 64)):
        assert not ops.latent_attention_ok(torch.bfloat16, width=width, rank=rank, page_size=page)
        with pytest.raises(KernelError):
            run(width, rank, page)
    with pytest.raises(KernelError, match="at most 64 heads"):
        run(96, 64, 64, heads=65)
    assert not ops.latent_attention_ok(torch.float32, width=96, rank=64, page_size=64)


# ---- whole models --------------------------------------------------------------------------------

class Case:
    def __init__(self, tmp, name, dtype, lengths, seed=3, config=None):
        self.folder = make_folder(tmp, name, dtype=dtype, seed=seed, config=config)
        self.cfg, self.weights = read_folder(self.folder)
        self.requests = {f"r{i}": tokens(self.cfg["vocab"], n, 50 + i) for i, n in enumerate(lengths)}
        self.want = {rid: plain.forward(self.cfg, self.weights, toks) for rid, toks in self.requests.items()}
        self.dtype = dtype
        self.bound = F32_BOUND if dtype == "float32" else BF16_BOUND

    def runner(self, page_size=16, num_pages=40, max_requests=3):
        from pylon_amd.engine import Runner

        return Runner.from_folder(self.folder, dtype=self.dtype, page_size=page_size, num_pages=num_pages,
                                  max_requests=max_requests)

    def check(self, rid, got, label):
        assert np.isfinite(got).all()
        want = self.want[rid][: len(got)]
        if self.dtype != "float32":
            # a head's read-out is normed: where its products nearly cancel, rounding is magnified.  One
            # position in twenty-five may be off by more than the bound, none by more than four times it.
            off = np.abs(got - want).max(axis=1) / np.abs(want).max(axis=1)
            assert off.max() <= 4 * self.bound, f"{label}: request {rid}, position {off.argmax()} is off by {off.max():.2e}"
            assert (off > self.bound).sum() <= max(1, len(off) // 25), f"{label}: request {rid}: {(off > self.bound).sum()} of {len(off)}"
            return
        ok, worst, frac = rows_within(got, want, self.bound)
        assert ok, f"{label}: request {rid}, position {worst} is off by {frac:.2e} of its largest logit"


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


@pytest.mark.parametrize("name, page", [("A", 16), ("B", 64), ("C", 16), ("D", 32), ("E", 64)])
def test_the_stream_after_every_layer_run(tmp, name, page):
    """The sum of the copies after every layer run, in float32, for a whole prompt and in two portions."""
    from pylon_amd.engine import StepEntry
    from pylon_amd.kernels import ops

    case = Case(tmp, name, "float32", (45,))
    runner = case.runner(page_size=page, num_pages=8)
    kept = []

    def after(resid, delta):
        """What the next norm's kernel will make of the copies, formed on a copy of them."""
        copies = resid.clone()
        norm = runner.model.final_norm
        ops.stream_norm(copies, delta.value, norm.weight(), 1e-6, torch.float32, centre=True, mix=delta.mix, write=delta.write)
        kept.append((copies.sum(dim=0) if copies.dim() == 3 else copies).cpu().numpy())

    for block in runner.model.blocks:
        def wrapped(resid, delta, ctx, cache, stores, inner=block.forward):
            resid, delta = inner(resid, delta, ctx, cache, stores)
            after(resid, delta)
            return resid, delta
        block.forward = wrapped
    toks = case.requests["r0"]
    want = []
    plain.forward(case.cfg, case.weights, toks, streams=want)
    seq = runner.open("a")
    runner.step([StepEntry(seq, toks, list(range(len(toks))))])
    runner.close(seq)
    assert len(kept) == len(want) == len(plain.run_order(case.cfg))
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
                                                ("D", "float32", 32), ("A", "bfloat16", 16), ("B", "bfloat16", 64),
                                                ("B", "bfloat16", 32), ("C", "bfloat16", 64), ("D", "bfloat16", 64),
                                                ("C", "float32", 64), ("E", "float32", 64), ("E", "bfloat16", 64),
                                                ("C", "bfloat16", 16), ("D", "bfloat16", 128)])
def test_whole_token_by_token_and_in_portions(tmp, name, dtype, page):
    """Pages of 16 and 32 tokens run the general attention kernel; over pages of 64 and 128 bfloat16
    models run on the matrix cores."""
    case = Case(tmp, name, dtype, (71, 38))
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


@pytest.mark.parametrize("name, dtype, page", [("A", "float32", 16), ("B", "float32", 16), ("D", "float32", 16),
                                                ("C", "bfloat16", 16), ("B", "bfloat16", 64), ("D", "bfloat16", 64),
                                                ("E", "bfloat16", 64), ("C", "bfloat16", 64)])
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


@pytest.mark.parametrize("name, dtype", [("B", "float32"), ("B", "bfloat16"), ("A", "float32"), ("C", "bfloat16")])
def test_long_decoding_after_a_prompt(tmp, name, dtype):
    """420 tokens, 320 of them one by one: the state goes through hundreds of single steps, windows of
    7 to 129 positions pass over decoded tokens, and the pages a window has left go back."""
    case = Case(tmp, name, dtype, (420,))
    runner = case.runner(page_size=64, num_pages=7, max_requests=2)
    got, _ = run_plan(runner, case, [{"r0": 100}] + [{"r0": 1}] * 320)
    case.check("r0", got["r0"], "long decoding")
    assert runner.manager.free_pages == 7


@pytest.mark.parametrize("name, dtype, page", [("A", "float32", 16), ("B", "bfloat16", 64)])
def test_requests_do_not_see_what_a_freed_slot_or_page_held(tmp, name, dtype, page):
    """The same request, alone in a fresh runner and after others have used every page and slot."""
    case = Case(tmp, name, dtype, (50, 64, 64))
    fresh, _ = run_plan(case.runner(page_size=page, num_pages=128 // page, max_requests=2), case, [{"r0": 50}])
    runner = case.runner(page_size=page, num_pages=128 // page, max_requests=2)
    for tensor in runner.manager.slots.tensors.values():
        tensor.fill_(float("nan"))
    for group in runner.manager.groups:
        for cache in list(group.k.values()) + [v for v in group.v.values() if v is not None]:
            cache.fill_(float("nan"))
    used, _ = run_plan(runner, case, [{"r1": 64, "r2": 64}, {"r1": 0, "r2": 0}, {"r0": 25}, {"r0": 25}])
    bound = 2e-5 if dtype == "float32" else 5e-2
    assert np.abs(used["r0"] - fresh["r0"]).max() <= bound * np.abs(fresh["r0"]).max()


def test_the_first_tokens_of_a_sequence_start_from_nothing(tmp):
    """Position 0 sees itself alone and its state starts empty: its logits are those of a one-token
    request, whatever follows it and whatever ran in its slot before."""
    case = Case(tmp, "D", "float32", (9, 30))
    runner = case.runner(num_pages=8, max_requests=1)
    first, _ = run_plan(runner, case, [{"r1": 30}, {"r1": 0}, {"r0": 1}])
    want = plain.forward(case.cfg, case.weights, case.requests["r0"][:1])
    assert np.abs(first["r0"] - want).max() <= F32_BOUND * np.abs(want).max()
    two, _ = run_plan(runner, case, [{"r0": 2}])
    assert np.abs(two["r0"] - case.want["r0"][:2]).max() <= F32_BOUND * np.abs(want).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_request_whole_and_with_its_tail_decoded(tmp, dtype):
    """700 tokens over eleven pages of 64: one mixer looks back over all of them, the states have gone
    through all of them."""
    case = Case(tmp, "C", dtype, (700,))
    runner = case.runner(page_size=64, num_pages=12, max_requests=1)
    whole, _ = run_plan(runner, case, [{"r0": 700}])
    case.check("r0", whole["r0"], "whole")
    tail, _ = run_plan(runner, case, [{"r0": 650}] + [{"r0": 1}] * 50)
    case.check("r0", tail["r0"], "tail decoded")


@pytest.mark.parametrize("name, dtype, graphs, page", [("A", "float32", False, 16), ("B", "float32", True, 16),
                                                         ("C", "bfloat16", True, 64), ("B", "bfloat16", True, 64),
                                                         ("D", "bfloat16", True, 64), ("E", "bfloat16", False, 64)])
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
            row = plain.forward(cfg, weights, sequence)[-1]
            assert produced == int(row.argmax()) or row.max() - row[produced] <= slack * np.abs(row).max(), \
                (prompt[:3], result.output_ids)
            sequence.append(produced)


@pytest.mark.parametrize("name, dtype", [("B", "float32"), ("D", "float32"), ("B", "bfloat16"), ("C", "bfloat16")])
def test_the_replay_program_as_a_user_runs_it(tmp, tmp_path, name, dtype):
    """``bin/trace_run`` as a subprocess over pages of 64 and four slots: up to four live requests,
    portions of some beside single tokens of others, pages and slots used again; the logits files
    against the plain model."""
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
    """A configuration drawn over what config.json allows: layers in any order, heads and sizes in
    steps of 8 and a few odd ones, windows that are no multiple of anything, with and without
    rotation, stretched frequencies, feed-forwards, loops, one to four copies of the stream."""
    rng = np.random.default_rng(9000 + seed)
    width = int(rng.choice([48, 64, 96, 136, 160, 256]))
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        kind = str(rng.choice(["gla", "latent_attention", "latent_attention_2"]))
        if kind == "gla":
            m = {"heads": int(rng.integers(1, 5)), "dim": int(rng.choice([8, 12, 16, 32, 64, 96, 128])),
                 "vdim": int(rng.choice([8, 16, 20, 32, 48, 64, 128])), "tau": float(rng.choice([1.0, 4.0, 16.0, 0.8])),
                 "decay_rank": int(rng.choice([1, 4, 16, 20]))}
        else:
            rot_dim = int(rng.choice([4, 8, 16, 32, 64]))
            m = {"heads": int(rng.choice([1, 2, 3, 6, 8, 12, 18])), "dim": int(rng.choice([8, 16, 32, 40, 64, 12])),
                 "rot_dim": rot_dim, "vdim": int(rng.choice([4, 8, 20, 32, 48, 64, 80])),
                 "kv_rank": int(rng.choice([16, 32, 64, 96, 128, 192, 20, 256])), "scale": float(rng.uniform(0.05, 0.3)),
                 "mask": {"size": int(rng.choice([int(rng.integers(3, 200)), 32, 64, 128, 1000]))}}
            m["rot"] = {"base": float(rng.choice([100.0, 1.0e4, 5.0e5])), "dims": rot_dim}
            if rng.random() < 0.6:
                m["rot"]["scaling"] = {"factor": float(rng.choice([2.0, 8.0, 32.0])), "original": float(rng.choice([16, 64, 2048])),
                                       "fast": float(rng.choice([4.0, 32.0])), "slow": float(rng.choice([1.0, 2.0]))}
        mlp = {"kind": "dense", "ff": int(rng.choice([40, 64, 100, 168, 256]))} if rng.random() > 0.15 else None
        layers.append({"type": kind, "mixer": m, "mlp": mlp})
    config = {"architecture": "Ranudra", "vocab": int(rng.integers(90, 700)), "width": width,
              "streams": int(rng.integers(1, 5)), "embedding": {"scale": float(rng.choice([1.0, 4.0, 12.0]))},
              "norm": {"eps": float(10 ** rng.uniform(-7, -4))}, "layers": layers}
    if rng.random() < 0.6:
        start = int(rng.integers(0, len(layers)))
        config["loop"] = {"start": start, "stop": int(rng.integers(start + 1, len(layers) + 1)), "times": int(rng.integers(1, 4))}
    return config, (int(rng.integers(1, 40)), int(rng.integers(60, 200)), int(rng.integers(200, 330)))


@pytest.mark.parametrize("seed, dtype", [(seed, "float32") for seed in range(8)] + [(seed, "bfloat16") for seed in range(12)])
def test_a_configuration_drawn_at_random_matches_the_plain_model(tmp, seed, dtype):
    """Pages of 64 and four slots: each request whole, the longest with its tail token by token, then
    all three side by side in portions over a pool too small for them to have pages to spare."""
    config, lengths = draw_config(seed)
    case = Case(tmp, f"drawn{seed}", dtype, lengths, seed=seed, config=config)
    pages = sum(-(-n // 64) for n in lengths)
    runner = case.runner(page_size=64, num_pages=pages, max_requests=4)
    whole, _ = run_plan(runner, case, [{"r0": lengths[0]}, {"r0": 0, "r1": lengths[1]}, {"r1": 0, "r2": lengths[2]}])
    for rid, got in whole.items():
        case.check(rid, got, f"whole (seed {seed})")
    tail, _ = run_plan(runner, case, [{"r2": lengths[2] - 70}] + [{"r2": 1}] * 70)
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
