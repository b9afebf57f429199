"""The Pinirax decoder in the engine against its plain statement (plain_pinirax.py), on the GPU: each mechanism alone, then
whole models under every way of cutting and batching, in 32-bit and in bfloat16, at sizes of the tests' own."""
import json
import os

import numpy as np
import pytest
import torch

import helpers as H
import plain_pinirax as pp
from test_pinirax import LEFT, RIGHT, PAR, SSM, MOE, config

pytestmark = pytest.mark.gpu

# Sizes that differ from one another wherever the design allows it: keys wider and narrower than values, heads that are and are not
# multiples of 8 or 16, one head, one group and as many groups as heads; windows shorter than a page, as long as one, of one
# token, and none; no cap; convolutions of one tap and of many; the norm in one part and in parts that cut through heads; one
# expert, top = all, identity experts and none; layers without a feed-forward; every order of the mixers.
MIX = config(96, 211, [
    (PAR(LEFT(4, 2, 12, 20, 0.9, size=11, cap=6.0), RIGHT(6, 3, 8, 12, 3), 0.7, 1.3), MOE(6, 2, 24, identity=2)),
    (SSM(6, 8, 20, 3, 4, 4), MOE(5, 3, 40, identity=1)),
    (PAR(LEFT(3, 1, 16, 8, 1.1, size=33, cap=3.0), RIGHT(2, 2, 20, 7, 4), 1.2, 0.8), None),
    (SSM(2, 12, 5, 1, 1, 1), MOE(1, 2, 8, identity=3)),
    (PAR(LEFT(2, 2, 24, 24, 0.7, cap=None), RIGHT(5, 1, 33, 20, 1), 1.0, 0.9), MOE(4, 4, 16)),
], eps=2e-6, scale=1.5)
WIDE = config(64, 150, [
    (SSM(4, 20, 70, 2, 8, 4), MOE(8, 1, 24, identity=1)),
    (PAR(LEFT(18, 1, 32, 16, 0.6, size=16, cap=10.0), RIGHT(4, 2, 130, 64, 4), 0.8, 0.9), None),
    (PAR(LEFT(1, 1, 40, 72, 0.5, size=1, cap=4.0), RIGHT(1, 1, 64, 64, 2), 1.5, 0.5), MOE(2, 1, 72)),
], eps=1e-5, scale=3.0)
TINY = config(40, 64, [(PAR(LEFT(1, 1, 4, 4, 1.0, size=3, cap=2.0), RIGHT(1, 1, 1, 1, 4), 1.0, 1.0), MOE(2, 1, 8, identity=1))], scale=1.0)
DEEP = config(56, 97, [
    (SSM(7, 4, 9, 7, 2, 5), MOE(7, 3, 20, identity=4)),
    (SSM(3, 5, 200, 1, 3, 7), None),
    (PAR(LEFT(6, 3, 9, 30, 0.8, size=70, cap=8.0), RIGHT(9, 3, 17, 5, 6), 0.5, 1.1), MOE(12, 1, 12)),
    (PAR(LEFT(2, 1, 56, 7, 0.4, size=8, cap=50.0), RIGHT(4, 4, 250, 40, 3), 1.1, 0.6), MOE(9, 5, 16, identity=2)),
], eps=1e-4, scale=0.5)
# sizes in steps of 8 and more, as larger models have them: the experts run over their own rows, the products stream their weights
EVEN = config(128, 120, [
    (SSM(8, 16, 64, 2, 2, 4), MOE(8, 2, 32, identity=2)),
    (PAR(LEFT(6, 2, 64, 64, 0.3, size=48, cap=15.0), RIGHT(4, 2, 64, 32, 4), 0.9, 1.1), MOE(6, 2, 64, identity=1)),
    (PAR(LEFT(8, 4, 32, 128, 0.4, size=25, cap=20.0), RIGHT(8, 4, 128, 128, 4), 1.0, 1.0), MOE(10, 3, 48)),
], eps=1e-5, scale=2.0)
CONFIGS = {"mix": (MIX, 8), "wide": (WIDE, 16), "tiny": (TINY, 16), "deep": (DEEP, 32), "even": (EVEN, 16)}
STD = 5.0


def make_folder(path, cfg, seed, std_scale=STD, edit=None):
    """A model folder with random weights, stored in bfloat16 as this design's checkpoints are (so the 32-bit engine, the
    bfloat16 engine and the plain statement all start from the same numbers); `edit(tensors)` may change them before they
    are written."""
    folder = H.make_model_folder(path, cfg, seed, "bfloat16", std_scale=std_scale)
    from safetensors.torch import load_file, save_file
    file = os.path.join(folder, "model.safetensors")
    tensors = {k: v.clone() for k, v in load_file(file).items()}
    (edit or sharpen)(tensors)
    save_file(tensors, file)
    return folder


def sharpen(tensors, std_scale=STD):
    """What the folder's wider draw would saturate keeps the spread its spec names; decays are made slow enough that a state
    holds what lies dozens of tokens back."""
    for name, t in tensors.items():
        if name.endswith((".router", ".correction", ".b", ".dt_bias", ".conv")):
            t /= std_scale
        if name.endswith(".A_log"):
            t /= std_scale
            t -= 3.0


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: make_folder(tmp_path_factory.mktemp(name), cfg, seed=i) for i, (name, (cfg, _)) in enumerate(CONFIGS.items())}


def runner_for(folder, name, dtype, tokens=1024, max_requests=4, **kw):
    from ginfer_amd import ModelRunner
    ps = CONFIGS[name][1]
    return ModelRunner(folder, dtype=dtype, page_size=ps, num_pages=-(-tokens // ps), max_requests=max_requests,
                       max_model_len=2048, **kw)


def requests_for(name, lengths, seed=20):
    return {"q%d" % i: H.random_tokens(n, CONFIGS[name][0]["vocab"], seed + i) for i, n in enumerate(lengths)}


_plain = {}


def plain(folder, ids):
    key = (folder, tuple(ids))
    if key not in _plain:
        _plain[key] = pp.forward(pp.read_config(folder), pp.read_weights(folder), list(ids)).numpy()
    return _plain[key]


def compare(got, requests, folder, tol, what, close_calls=0.0, median=0.5):
    """Every row against the plain statement.  close_calls: the share of rows that may miss the tolerance."""
    over, first, errors = 0, None, []
    for (rid, p), row in sorted(got.items()):
        ref = plain(folder, requests[rid])
        assert np.isfinite(row).all(), "%s: request %s position %d: non-finite logits" % (what, rid, p)
        err = float(np.abs(row.astype(np.float64) - ref[p]).max() / np.abs(ref).max())
        errors.append(err)
        if err > tol:
            over += 1
            first = first or "%s: first wrong place is request %s position %d of %d: error %.3g > %.3g" % (
                what, rid, p, len(requests[rid]), err, tol)
    assert over <= close_calls * len(got), "%s (%d of %d rows)" % (first, over, len(got))
    assert float(np.median(errors)) <= tol * median, "%s: the median row is off by %.3g" % (what, float(np.median(errors)))
    for rid, ids in requests.items():
        missing = [p for p in range(len(ids)) if (rid, p) not in got]
        assert not missing, "%s: request %s lacks logits at %s" % (what, rid, missing[:8])


# 32-bit differs from the 64-bit plain statement by the rounding of sums of a few hundred terms; bfloat16 rounds every stored
# activation to 8 bits, and where two experts' scores lie within that rounding the engine may take the other one: then that row,
# and rows that look at it, miss the tolerance.  So in bfloat16 the median row must stay within half the tolerance and a share
# of the rows may miss it; a mechanism that is wrong moves nearly every row, and in 32-bit, where no row may miss, every cutting
# and batching must give the whole request's bits.
TOL = {"float32": 1e-4, "bfloat16": 6e-2}
CLOSE = {"float32": 0.0, "bfloat16": 0.2}
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


class _Step:
    """The few arrays of a step that the kernels under test read."""

    def __init__(self, q_len, q_start):
        dev = torch.device("cuda")
        cu = np.concatenate([[0], np.cumsum(q_len)]).astype(np.int32)
        self.cu_tokens = torch.tensor(cu, device=dev)
        self.q_start = torch.tensor(q_start, dtype=torch.int32, device=dev)
        self.token_entry = torch.tensor(np.repeat(np.arange(len(q_len)), q_len), dtype=torch.int32, device=dev)
        self.positions = torch.tensor(np.concatenate([np.arange(s, s + n) for s, n in zip(q_start, q_len)]), dtype=torch.int32,
                                      device=dev)
        self.num_entries = len(q_len)
        self.host_q_len, self.host_q_start = list(q_len), list(q_start)
        rows = [(cu[e], q_start[e], e, 0) for e, n in enumerate(q_len) if n == 1]
        self.extra = {"decode_info": torch.tensor(rows, dtype=torch.int32, device=dev).reshape(-1, 4)}

    @property
    def max_q_len(self):
        return max(self.host_q_len)

    @property
    def max_kv_len(self):
        return max(s + n for s, n in zip(self.host_q_start, self.host_q_len))


# ----------------------------------------------------------------------------------------------- mechanisms alone

def test_scaled_embedding_with_positions():
    from ginfer_amd.parts.embedding import SinusoidalScaledEmbedding
    for width, dtype in ((7, torch.float32), (64, torch.bfloat16), (384, torch.bfloat16)):
        g = torch.Generator().manual_seed(width)
        table = torch.randn((50, width), generator=g).to(dtype)
        ids = torch.randint(0, 50, (9,), generator=g).to(torch.int32)
        pos = [0, 1, 2, 63, 64, 1000, 1999, 5, 0]
        part = SinusoidalScaledEmbedding(50, width, 2.5, dtype, "cuda")
        part.bind_weights({"": table.cuda()})
        step = _Step([1] * 9, pos)
        got = part.forward(ids.cuda(), step).cpu()
        want = 2.5 * table.double()[ids.long()] + pp.position_vectors(2000, width)[pos]
        assert got.dtype == torch.float32 and float((got - want).abs().max()) < 2e-4


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_head_norms_with_gates(dtype):
    """Heads narrower and wider than a wavefront's reach, weights shared and not, gates, factors, results as columns of a wider
    tensor; widths that 16-byte accesses do not fit."""
    from ginfer_amd.kernels import ops
    g = torch.Generator().manual_seed(1)
    for T, heads, V in ((5, 3, 4), (5, 2, 7), (3, 4, 64), (2, 5, 100), (9, 3, 128), (4, 2, 129), (3, 2, 896), (2, 3, 1500), (6, 1, 260), (3, 1, 1024)):
        x = torch.randn((T, heads, V), generator=g) * 3
        proj = torch.randn((T, heads * V + 12), generator=g)
        ref = pp.rms(x.double(), 1e-4)
        for own in (False, True):
            w = torch.randn((heads, V) if own else (V,), generator=g)
            for gate_start in (None, 4, 3):
                out = torch.zeros((T, heads * V + 8), dtype=dtype, device="cuda")
                view = out[:, 4:4 + heads * V]
                ops.head_norm_gate(x.cuda(), w.cuda(), 1e-4, dtype, proj=None if gate_start is None else proj.cuda(),
                                   gate_start=gate_start or 0, out=view, out_scale=0.75)
                want = ref * w.double()
                if gate_start is not None:
                    want = want * pp.silu(proj.double()[:, gate_start:gate_start + heads * V]).reshape(T, heads, V)
                assert H.rel_err(view.float().cpu(), 0.75 * want.reshape(T, -1)) < (2e-6 if dtype == torch.float32 else 1e-2), (T, heads, V)
                assert not out[:, :4].any() and not out[:, 4 + heads * V:].any()


CUTS = [None, [1, 1, 2, 5, 3, 16, 1, 17, 1, 64, 24, 15], [2] * 75, [1] * 150]


@pytest.mark.parametrize("chunked", [False, True])
@pytest.mark.parametrize("delta", [True, False])
@pytest.mark.parametrize("sizes", [(1, 1, 64, 4, 4), (6, 3, 8, 12, 3), (2, 2, 20, 7, 4), (5, 1, 33, 20, 1), (4, 2, 130, 64, 4), (9, 3, 17, 5, 6),
                                   (2, 1, 250, 40, 4), (3, 3, 128, 130, 2), (1, 1, 1, 1, 16), (4, 1, 192, 260, 4)])
def test_the_recurrences_alone(delta, sizes, chunked):
    """Whole, cut in several ways and token by token, beside a second request that starts and ends elsewhere, against the plain
    statement; the state is the plain one; slots that held something else (here: no numbers at all) show nowhere; all cuttings give
    the same bits, or, in chunks on the matrix cores, the same up to rounding."""
    from ginfer_amd.kernels import ops
    heads, groups, dim, vdim, taps = sizes
    g = torch.Generator().manual_seed(sum(sizes))
    T, C = 150, 2 * groups * dim + heads * vdim
    hv, gd = heads * vdim, groups * dim
    if delta:
        cols = dict(conv=0, q=0, k=gd, v=2 * gd, gate=C, b=C + hv, a=C + hv + heads)
        width = C + hv + 2 * heads + 3
    else:
        cols = dict(gate=0, conv=hv, v=0, k=hv, q=hv + gd, a=hv + C, b=hv + C)
        width = hv + C + heads + 3
    proj = torch.randn((T, width), generator=g)
    other = torch.randn((60, width), generator=g)
    w = torch.randn((C, taps), generator=g) * 0.6
    bias = None if delta else torch.randn((C,), generator=g) * 0.3
    rate, dt = torch.rand((heads,), generator=g) * 0.3 + 0.01, torch.randn((heads,), generator=g)
    skip, weight = torch.randn((heads,), generator=g), torch.randn((vdim,), generator=g)

    def reference(rows):
        p = rows.double()
        n = p.shape[0]
        c = pp.silu(pp.causal_convolution(p[:, cols["conv"]:cols["conv"] + C], w.double(), None if bias is None else bias.double()))
        of_head = [i // (heads // groups) for i in range(heads)]
        q, k = (c[:, cols[x]:cols[x] + gd].reshape(n, groups, dim)[:, of_head] for x in "qk")
        v = c[:, cols["v"]:cols["v"] + hv].reshape(n, heads, vdim)
        sp = pp.softplus(p[:, cols["a"]:cols["a"] + heads] + dt.double())
        a = torch.exp(-rate.double() * sp)
        gate = pp.silu(p[:, cols["gate"]:cols["gate"] + hv]).reshape(n, heads, vdim)
        if delta:
            o, S = pp.gated_delta_rule(pp.unit(q) * dim ** -0.5, pp.unit(k), v, a, torch.sigmoid(p[:, cols["b"]:cols["b"] + heads]))
            return (0.7 * pp.rms(o, 1e-5) * weight.double() * gate).reshape(n, hv), S
        y, S = pp.state_space(v, k, q, sp, a, skip.double())
        return y * gate, S

    want, S_want = reference(proj)
    want2, _ = reference(other)
    dev = lambda t: None if t is None else t.cuda()
    first = None
    for cut in CUTS:
        cut = cut or [T]
        state = torch.full((4,) + ops.delta_state_shape(heads, dim, vdim), float("nan"), device="cuda")
        ring = torch.full((4, taps, C), float("nan"), device="cuda") if taps > 1 else None
        got, got2, at, oat = [], [], 0, 0
        for i, n in enumerate(cut):
            k = min(1 if set(cut) == {1} else 1 + i % 4, 60 - oat)
            # the second request's rows come first in every other step, and its slot is another one
            entries = [(2, proj[at:at + n], at)] + ([(0, other[oat:oat + k], oat)] if k else [])
            if i % 2:
                entries.reverse()
            rows = torch.cat([e[1] for e in entries]).cuda()
            step = _Step([e[1].shape[0] for e in entries], [e[2] for e in entries])
            slots = torch.tensor([e[0] for e in entries], device="cuda")
            out = ops.delta_recurrence(rows, dev(w), dev(bias), dev(rate), dev(dt), dev(skip), ring, state, slots, step, heads, groups, dim, vdim,
                                       cols, delta, q_scale=dim ** -0.5, unit_eps=1e-6, weight=dev(weight) if delta else None, eps=1e-5,
                                       dtype=torch.float32, out_scale=0.7, chunked=chunked).cpu()
            mine = (k if i % 2 and k else 0)
            got.append(out[mine:mine + n])
            if k:
                theirs = 0 if i % 2 else n
                got2.append(out[theirs:theirs + k])
            at, oat = at + n, oat + k
        got, got2 = torch.cat(got), torch.cat(got2)
        assert H.rel_err(got, want) < 2e-5, (sizes, len(cut), H.rel_err(got, want))
        assert H.rel_err(got2, want2[:got2.shape[0]]) < 2e-5
        held = ops.delta_state_matrix(state[2].cpu(), dim, vdim)
        assert H.rel_err(held, S_want) < 2e-5
        first = first or (got, held)
        if chunked:
            continue
        assert torch.equal(got, first[0]) and torch.equal(held, first[1]), "%d steps differ from one" % len(cut)


def test_an_old_write_reaches_far_and_slow_decay_counts():
    """A key met once, 700 tokens back, read by a query that matches it: with a decay near one it decides the result, and with it
    taken away the result is another."""
    from ginfer_amd.kernels import ops
    T, dim, vdim = 720, 32, 16
    g = torch.Generator().manual_seed(3)
    C = 2 * dim + vdim
    cols = dict(conv=0, q=0, k=dim, v=2 * dim, gate=C, b=C + vdim, a=C + vdim + 1)
    proj = torch.zeros((T, C + vdim + 2))
    proj[:, :C] = torch.randn((T, C), generator=g)
    proj[:, 2] = proj[:, dim + 2] = -30.0            # silu of it is nothing: coordinate 2 is free in every key and query
    proj[:, C:C + vdim] = 2.0
    proj[:, cols["a"]] = -9.0                        # softplus ~ 1e-4: the state hardly fades
    proj[15, dim:2 * dim] = -30.0
    proj[15, dim + 2] = 8.0                          # the one key there
    proj[15, 2 * dim:C] = torch.arange(vdim, dtype=torch.float32) + 4.0
    proj[-1, :dim] = -30.0
    proj[-1, 2] = 8.0                                # and the query that asks for it
    w = torch.ones((C, 1))
    args = lambda rows, state, step, chunked: ops.delta_recurrence(
        rows.cuda(), w.cuda(), None, torch.ones(1, device="cuda"), torch.zeros(1, device="cuda"), None, None, state,
        torch.zeros(1, dtype=torch.int64, device="cuda"), step, 1, 1, dim, vdim, cols, True, q_scale=dim ** -0.5, unit_eps=1e-6,
        weight=torch.ones(vdim, device="cuda"), eps=1e-5, dtype=torch.float32, chunked=chunked)
    c = pp.silu(proj[:, :C].double())
    q, k, v = pp.unit(c[:, :dim])[:, None] * dim ** -0.5, pp.unit(c[:, dim:2 * dim])[:, None], c[:, 2 * dim:][:, None]
    a, b = torch.exp(-pp.softplus(proj[:, cols["a"]:cols["a"] + 1].double())), torch.sigmoid(proj[:, cols["b"]:cols["b"] + 1].double())
    o, _ = pp.gated_delta_rule(q, k, v, a, b)
    want = pp.rms(o[-1, 0], 1e-5) * pp.silu(torch.tensor(2.0, dtype=torch.float64))
    gone = pp.rms(pp.gated_delta_rule(q[16:], k[16:], v[16:], a[16:], b[16:])[0][-1, 0], 1e-5) * pp.silu(torch.tensor(2.0, dtype=torch.float64))
    assert H.rel_err(gone, want) > 0.3
    for cut, chunked in [(c, k) for c in ([720], [16, 1, 700, 3], [700] + [1] * 20) for k in (False, True)]:
        state = torch.zeros((1,) + ops.delta_state_shape(1, dim, vdim), device="cuda")
        at = 0
        for n in cut:
            out = args(proj[at:at + n], state, _Step([n], [at]), chunked)
            at += n
        assert H.rel_err(out[-1].cpu(), want) < 5e-5


@pytest.mark.parametrize("chunked", [False, True])
def test_the_same_key_again_and_again(chunked):
    """Every token writes under the same key with b near 1 and no decay to speak of: each write overwrites the one before, and what
    is read is the last value.  Inside a chunk the writes then cancel to first order, which a product of powers would lose."""
    from ginfer_amd.kernels import ops
    T, dim, vdim = 100, 64, 32
    g = torch.Generator().manual_seed(4)
    C = 2 * dim + vdim
    cols = dict(conv=0, q=0, k=dim, v=2 * dim, gate=C, b=C + vdim, a=C + vdim + 1)
    proj = torch.zeros((T, C + vdim + 2))
    proj[:, :2 * dim] = torch.randn((2 * dim,), generator=g)
    proj[:, 2 * dim:C] = torch.randn((T, vdim), generator=g) * 3
    proj[:, C:C + vdim] = 1.5
    proj[:, cols["b"]], proj[:, cols["a"]] = 12.0, -12.0
    proj[:, :dim] = proj[:, dim:2 * dim]
    state = torch.zeros((1,) + ops.delta_state_shape(1, dim, vdim), device="cuda")
    out = ops.delta_recurrence(proj.cuda(), torch.ones((C, 1), device="cuda"), None, torch.ones(1, device="cuda"), torch.zeros(1, device="cuda"), None,
                               None, state, torch.zeros(1, dtype=torch.int64, device="cuda"), _Step([T], [0]), 1, 1, dim, vdim, cols, True,
                               q_scale=dim ** -0.5, unit_eps=1e-6, weight=torch.ones(vdim, device="cuda"), eps=0.0, dtype=torch.float32, chunked=chunked)
    want = pp.rms(pp.silu(proj[:, 2 * dim:C].double()), 0.0) * pp.silu(torch.tensor(1.5, dtype=torch.float64))
    assert H.rel_err(out.cpu(), want) < 1e-3
    c = pp.silu(proj[:, :C].double())
    o, _ = pp.gated_delta_rule(pp.unit(c[:, None, :dim]) * dim ** -0.5, pp.unit(c[:, None, dim:2 * dim]), c[:, None, 2 * dim:],
                               torch.exp(-pp.softplus(proj[:, cols["a"]:cols["a"] + 1].double())), torch.sigmoid(proj[:, cols["b"]:cols["b"] + 1].double()))
    assert H.rel_err(out.cpu(), pp.rms(o[:, 0], 0.0) * pp.silu(torch.tensor(1.5, dtype=torch.float64))) < 2e-5


@pytest.mark.parametrize("experts,identity,top", [(1, 0, 1), (6, 2, 2), (5, 3, 8), (60, 4, 6), (200, 56, 8), (3, 1, 1)])
def test_softmax_routing_with_identity_experts(experts, identity, top):
    from ginfer_amd.kernels import ops
    E = experts + identity
    for T, width in ((1, 7), (33, 64), (5, 1030)):
        g = torch.Generator().manual_seed(E + T)
        z = torch.randn((T, E), generator=g) * 2
        corr = torch.randn((E,), generator=g) * 0.3
        x = torch.randn((T, width), generator=g)
        s = torch.softmax(z.double(), dim=-1)
        ids_ref = [sorted(range(E), key=lambda e: (-float(s[t, e] + corr[e]), e))[:top] for t in range(T)]
        for dtype in (torch.float32, torch.bfloat16):
            xd = x.to(dtype)
            chosen = torch.full((top, T, width), 7.0, device="cuda") if identity else None
            ids, weights, dense = ops.route_groups(z.cuda(), top, corr.cuda(), normalise=False, softmax=True, identity=identity, x=xd.cuda(), own_out=chosen)
            total = torch.full((T, width), 7.0, device="cuda") if identity else None
            ids2, weights2, dense2 = ops.route_groups(z.cuda(), top, corr.cuda(), normalise=False, softmax=True, identity=identity, x=xd.cuda(), own_out=total)
            assert torch.equal(ids, ids2) and torch.equal(weights, weights2) and torch.equal(dense, dense2) and dense.shape == (T, experts)
            for t in range(T):
                assert ids[t].tolist() == ids_ref[t], t
                want_dense, own = torch.zeros(experts, dtype=torch.float64), torch.zeros(width, dtype=torch.float64)
                for k, e in enumerate(ids_ref[t]):
                    assert abs(float(weights[t, k]) - float(s[t, e])) < 1e-6
                    if e < experts:
                        want_dense[e] = s[t, e]
                        if identity:
                            assert bool((chosen[k, t] == 7.0).all())
                    else:
                        own += s[t, e] * xd[t].double()
                        assert H.rel_err(chosen[k, t].cpu(), s[t, e] * xd[t].double()) < 1e-5
                assert float((dense[t].cpu() - want_dense).abs().max()) < 1e-6
                if identity:
                    assert float((total[t].cpu() - own).abs().max()) < 1e-5 * max(1.0, float(own.abs().max()))
        # scores that are no numbers (rows that pad a recorded step) still give choices inside the table
        z[0] = float("nan")
        ids, weights, _ = ops.route_groups(z.cuda(), top, corr.cuda(), normalise=False, softmax=True, identity=identity, x=x.cuda(),
                                           own_out=torch.empty((top, T, width), device="cuda") if identity else None)
        assert int(ids.min()) >= 0 and int(ids.max()) < E and len(set(ids[0].tolist())) == top


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(64, 6, 2, 24, 2), (64, 5, 4, 40, 1), (72, 1, 2, 16, 3), (128, 9, 2, 64, 1), (40, 4, 4, 8, 0), (36, 7, 3, 20, 2)])
def test_routed_feed_forwards_with_identity_experts(sizes, dtype):
    """The part in both of its ways (experts over their own rows, every expert over every row), from one row to hundreds."""
    from ginfer_amd.parts.mlp import RoutedGLU
    width, E, top, ff, identity = sizes
    g = torch.Generator().manual_seed(sum(sizes))
    part = RoutedGLU(width, E, top, ff, DT[dtype], "cuda", router_bias=False, scoring="softmax", correction=True, normalise=False, identity=identity)
    w = {n: (torch.randn(s.shape, generator=g) * (0.3 if n not in ("router", "correction") else 0.5)).to(torch.bfloat16)
         for n, s in part.weight_specs().items()}
    part.bind_weights({n: t.cuda().to(DT[dtype]) for n, t in w.items()})
    mlp = dict(router=dict(experts=E, top=top, identity=identity))
    for T in (1, 3, 17, 70, 300):
        x = torch.randn((T, width), generator=g).to(torch.bfloat16)
        y = part.forward(x.cuda().to(DT[dtype])).float().cpu()
        y = y.sum(dim=0) if y.dim() == 3 else y
        ref = pp.routed_feed_forward(x.double(), {n: t.double() for n, t in w.items()}, "", mlp)
        err = (y - ref).abs().max(dim=1).values / ref.abs().max()
        tol = 2e-5 if dtype == "float32" else 2e-2
        assert float((err > tol).double().mean()) <= (0.0 if dtype == "float32" else 0.05), (sizes, T, err.max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(4, 2, 12, 20, 11, 6.0), (1, 1, 4, 4, 3, 2.0), (18, 1, 32, 16, 16, 10.0), (6, 2, 64, 64, 40, 15.0), (3, 1, 128, 128, None, 30.0),
                                   (2, 2, 40, 72, 1, None), (5, 5, 130, 200, 70, 8.0), (8, 2, 64, 128, 200, 20.0), (7, 1, 256, 16, 33, 4.0)])
def test_capped_window_attention_with_a_gate_per_head(sizes, dtype):
    """The left mixer alone over pages in any order: biases, the norm per head, the cap, the window and the gates, whole and cut,
    beside another request's portions.  Scores reach far beyond the cap."""
    from ginfer_amd.parts import KVView
    from ginfer_amd.parts.conv_attention import ConvAttention
    heads, kv, D, V, window, cap = sizes
    W, T, page, dt = 48, 260, 16, DT[dtype]
    g = torch.Generator().manual_seed(sum(int(x or 0) for x in sizes))
    part = ConvAttention(W, heads, kv, D, V, 1.2, dt, "cuda", window=window, bias=True, out_bias=False, head_norm_eps=1e-5, soft_cap=cap, head_gate=True)
    w = {n: (torch.randn(s.shape, generator=g) * (0.3 if "norm" not in n else 1.0)).to(torch.bfloat16) for n, s in part.weight_specs().items()}
    part.bind_weights({n: t.cuda().to(dt if "norm" not in n else torch.float32) for n, t in w.items()})
    x = torch.randn((T, W), generator=g).to(torch.bfloat16)
    other = torch.randn((90, W), generator=g).to(torch.bfloat16)
    m = dict(heads=heads, kv_heads=kv, dim=D, vdim=V, scale=1.2, softcap=cap, mask=dict(size=window) if window else None)
    wd = {n: t.double() for n, t in w.items()}
    ref = pp.left_mixer(x.double(), wd, "", m, 1e-5)
    assert H.rel_err(pp.left_mixer(x.double(), wd, "", dict(m, softcap=None), 1e-5), ref) > 1e-3 or cap is None or window == 1
    P = part.padded
    width, n_pages = -(-T // page), -(-T // page) + 8
    outs = []
    for cut in ([T], [1, 1, 2, 5, 3, 16, 1, 31, 1, 64, 40, 95], [200] + [1] * 60):
        kp = torch.full((n_pages, kv, page, P), 7.0, dtype=dt, device="cuda")
        vp = torch.full((n_pages, kv, P, page), 7.0, dtype=dt, device="cuda")
        order = torch.randperm(n_pages, generator=g)
        table = torch.full((2, width), -1, dtype=torch.int32)
        table[0] = order[:width]
        table[1, :6] = order[width:width + 6]
        got, at, oat = [], 0, 0
        for i, n in enumerate(cut):
            k = min(1 + i % 3, 90 - oat)
            rows = torch.cat([x[at:at + n], other[oat:oat + k]]).cuda().to(dt)
            step = _Step([n, k], [at, oat])
            p = step.positions.cpu().long()
            slot = table[step.token_entry.cpu().long(), p // page].long() * page + p % page
            view = KVView(kp, vp, table.cuda(), slot.cuda(), page, True)
            y = part.forward(rows, step, [None, view])
            got.append((y.sum(dim=0) if y.dim() == 3 else y)[:n].float().cpu())
            at, oat = at + n, oat + k
        outs.append(torch.cat(got))
        err = float((outs[-1] - ref).abs().max() / ref.abs().max())
        assert err < (3e-5 if dtype == "float32" else 4e-2), (sizes, len(cut), err)
    if dtype == "float32":
        assert all(torch.equal(o, outs[0]) for o in outs)


# ----------------------------------------------------------------------------------------------- whole models

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_decoded_and_in_portions(folders, name, dtype):
    """Every request whole; then most of it in one step and the rest token by token; then in portions of 1 to 64 tokens, and
    in pairs.  In 32-bit the four agree to the bit."""
    reqs = requests_for(name, [1, 2, 5, 44, 131])
    runner = runner_for(folders[name], name, dtype)
    got = {}
    for what, steps in (("whole", H.steps_whole(reqs)), ("decoded", H.steps_last_decoded(reqs, last=48)),
                        ("portions", H.steps_portions(reqs)), ("pairs", H.steps_portions(reqs, sizes=(2,)))):
        got[what] = H.run_steps(runner, steps)
        runner.cache.check()
        compare(got[what], reqs, folders[name], TOL[dtype], "%s %s %s" % (name, dtype, what), CLOSE[dtype])
    if dtype == "float32":
        for what in ("decoded", "portions", "pairs"):
            for key, row in got["whole"].items():
                assert np.array_equal(row, got[what][key]), "%s: %s differs from whole at %s" % (name, what, key)
    assert not runner.cache.requests and all(g.pool.num_free == g.pool.num_pages for g in runner.cache.groups)


def test_the_stream_after_every_layer(folders):
    name = "mix"
    ids = H.random_tokens(37, CONFIGS[name][0]["vocab"], 5)
    runner = runner_for(folders[name], name, "float32", use_graphs=False)
    seen = []
    for block in runner.model.blocks:
        def wrapped(residual, delta, step, cache, inner=block.forward, **kw):
            out = inner(residual, delta, step, cache, **kw)
            seen.append(residual.cpu())
            return out
        block.forward = wrapped
    from ginfer_amd import StepEntry
    runner.step([StepEntry("a", ids, [0])])
    want = []
    pp.forward(pp.read_config(folders[name]), pp.read_weights(folders[name]), ids, want)
    assert len(seen) == len(want) == 5
    for i, s in enumerate(seen):
        assert H.rel_err(s, want[i]) < 1e-5, "after layer %d" % i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mix", "wide", "deep", "even"])
def test_unequal_requests_together_with_pages_and_slots_used_again(folders, name, dtype):
    """Seven requests through three state slots and a pool that holds three of them: portions of some beside single tokens
    of others, requests that sit a step out, and every page and slot used several times."""
    reqs = requests_for(name, [70, 3, 120, 33, 64, 17, 90], seed=50)
    steps = H.steps_mixed(reqs, max_live=3, seed=4)
    ps = CONFIGS[name][1]
    tokens = H.max_live_tokens(steps, round_to=ps)
    runner = runner_for(folders[name], name, dtype, tokens=tokens, max_requests=3)
    alone = H.run_steps(runner_for(folders[name], name, dtype), H.steps_whole(reqs)) if dtype == "float32" else None
    for rounds in range(2):                      # the second time the steps' shapes are known and recorded
        got = H.run_steps(runner, steps)
        runner.cache.check()
        compare(got, reqs, folders[name], TOL[dtype], "%s %s mixed, pass %d" % (name, dtype, rounds), CLOSE[dtype])
        if alone is not None:
            for key, row in alone.items():
                assert np.array_equal(row, got[key]), "%s: in a batch, %s differs from the request alone" % (name, key)
    assert not runner.cache.requests


def drawn_config(seed):
    """A configuration drawn at random."""
    rng = np.random.RandomState(seed)
    pick = lambda *xs: xs[rng.randint(len(xs))]
    layers = []
    for i in range(int(rng.randint(1, 6))):
        ff = None
        if rng.rand() < 0.8:
            experts, identity = int(pick(1, 2, 3, 4, 8, 16)), int(pick(0, 1, 2, 5))
            ff = MOE(experts, int(min(pick(1, 2, 3, 6), experts + identity)), int(pick(8, 16, 20, 33, 64)), identity=identity)
        groups = int(pick(1, 2, 3))
        if rng.rand() < 0.45:
            heads, vdim = groups * int(pick(1, 2, 4)), int(pick(1, 4, 5, 8, 20, 48))
            parts = [n for n in (1, 2, 3, 4, 6, 8) if heads * vdim % n == 0]
            layers.append((SSM(heads, vdim, int(pick(1, 4, 16, 33, 64, 100, 140)), groups, int(parts[rng.randint(len(parts))]), int(pick(1, 2, 4, 4, 7))), ff))
        else:
            kv = int(pick(1, 2, 3))
            left = LEFT(kv * int(pick(1, 2, 5)), kv, int(pick(1, 4, 7, 16, 32, 56, 130)), int(pick(1, 4, 20, 48, 64)), float(pick(0.3, 1.0, 1.5)),
                        size=pick(None, 1, 2, 7, 16, 17, 50), cap=pick(None, 2.0, 10.0, 50.0))
            layers.append((PAR(left, RIGHT(groups * int(pick(1, 2, 3)), groups, int(pick(1, 5, 16, 33, 64, 130)), int(pick(1, 6, 20, 32, 70)),
                                           int(pick(1, 2, 4, 4, 9))), float(pick(0.5, 1.0, 1.3)), float(pick(0.4, 1.0, 1.2))), ff))
    return config(int(pick(24, 40, 50, 52, 64, 66, 96, 136, 75)), int(pick(50, 128, 301)), layers, eps=float(pick(1e-6, 1e-5, 1e-4)),
                  scale=float(pick(0.5, 1.0, 4.0)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(tmp_path, seed, dtype):
    cfg = drawn_config(seed)
    folder = make_folder(tmp_path / "m", cfg, seed=seed)
    reqs = {"q%d" % i: H.random_tokens(n, cfg["vocab"], 200 + seed + i) for i, n in enumerate([1, 23, 70])}
    from ginfer_amd import ModelRunner
    page = [8, 16, 32][seed % 3]
    runner = ModelRunner(folder, dtype=dtype, page_size=page, num_pages=-(-256 // page), max_requests=3, max_model_len=512)
    for what, steps in (("whole", H.steps_whole(reqs)), ("decoded", H.steps_last_decoded(reqs, last=20)),
                        ("mixed", H.steps_mixed(reqs, max_live=3, seed=seed))):
        got = H.run_steps(runner, steps)
        runner.cache.check()
        compare(got, reqs, folder, TOL[dtype], "drawn configuration %d (%s) %s %s" % (seed, json.dumps(cfg), dtype, what),
                1.5 * CLOSE[dtype], median=1.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(folders, dtype):
    """A short prompt and 400 decoded tokens, recorded steps replayed throughout; windows pass over decoded tokens."""
    reqs = requests_for("mix", [420], seed=70)
    runner = runner_for(folders["mix"], "mix", dtype)
    got = H.run_steps(runner, H.steps_last_decoded(reqs, last=400))
    compare(got, reqs, folders["mix"], TOL[dtype], "long decoding " + dtype, CLOSE[dtype])
    if runner.use_graphs:
        assert runner.counts["replayed_decode"] > 300


def _marked(m):
    """Edits that make a single parallel layer's left mixer read the tokens themselves: token 7 is the marked key, token 8 the
    query that matches it; every other score is small.  The right mixer adds nothing."""
    def edit(t):
        sharpen(t)
        for n in t:
            if "norm1" in n or n == "final.norm":
                t[n].zero_()                       # gains around zero: plain norms
            if n.endswith((".q.norm", ".k.norm")):
                t[n].fill_(1.0)
            if n.endswith(("left.q.b", "left.k.b", "left.v.b")):
                t[n].zero_()
        e = t["embed"]
        r = torch.randn(e.shape, generator=torch.Generator().manual_seed(1)) * 6
        r[:, -4:] = 0
        e.copy_(r.to(e.dtype))
        e[7].zero_()
        e[8].zero_()
        # sines of the slowest angles, to which positions add little over the test's lengths
        mark, asks = e.shape[1] - 2, e.shape[1] - 4
        e[7, mark] = 40.0                          # the marked key
        e[8, asks] = 40.0                          # the query that matches it
        q, k = t["l0.mix.left.q"], t["l0.mix.left.k"]
        D = m["dim"]
        for w, at in ((q, asks), (k, mark)):
            w[:, -4:] = 0
            w[0::D].zero_()
            w[0::D, at] = 5.0
        t["l0.mix.left.g"].zero_()
        t["l0.mix.right.o"].zero_()
        t["l0.norm1b"].fill_(7.0)                  # what the mixer brings is as large as the stream itself
    return edit


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes,window", [((2, 1, 16, 12), 40), ((3, 3, 24, 32), 64), ((4, 2, 64, 64), 17), ((2, 1, 128, 128), 300)])
def test_keys_just_inside_and_just_outside_the_window(tmp_path, sizes, window, dtype):
    """One marked key at the window's last place, one before it and one behind, asked for from a prompt, by decoding and in
    portions; at page borders.  Inside it decides the last token, outside it is not seen."""
    heads, kv, D, V = sizes
    left = LEFT(heads, kv, D, V, 24.0 / D, size=window, cap=12.0)
    cfg = config(32, 40, [(PAR(left, RIGHT(1, 1, 4, 4, 2), 1.0, 1.0), None)], scale=1.0)
    folder = make_folder(tmp_path / "m", cfg, seed=3, std_scale=1.0, edit=_marked(left))
    rows = {}
    for T in (window + 30, 352 + window % 2):
        for back in (window - 1, window, window - 2, window + 1):
            ids = [int(x) % 6 for x in H.random_tokens(T, 40, T)]
            ids[T - 1 - back] = 7
            ids[-1] = 8
            reqs = {"a": ids}
            runner = runner_for(folder, "wide", dtype, tokens=1024)
            for what, steps in (("whole", H.steps_whole(reqs)), ("decoded", H.steps_last_decoded(reqs, last=30)),
                                ("portions", H.steps_portions(reqs, sizes=(7, 2, 33, 64)))):
                got = H.run_steps(runner, steps)
                compare(got, reqs, folder, TOL[dtype], "marked key %d back, window %d, %s %s" % (back, window, what, dtype))
            moved = list(ids)
            moved[T - 1 - back] = 1
            rows[(T, back)] = H.rel_err(plain(folder, moved)[-1], plain(folder, ids)[-1])
        assert min(rows[(T, window - 1)], rows[(T, window - 2)]) > 0.2 and max(rows[(T, window)], rows[(T, window + 1)]) < 1e-9, rows


def test_pages_before_the_window_go_back_while_a_request_runs(folders):
    """A pool far smaller than the request: the layers with a window give pages back as it moves on."""
    cfg = config(48, 90, [(PAR(LEFT(2, 1, 16, 16, 0.5, size=20, cap=5.0), RIGHT(2, 1, 8, 8, 4)), MOE(4, 2, 16, identity=1)),
                          (SSM(2, 8, 8, 1, 1, 4), None)])
    from ginfer_amd import ModelRunner
    import tempfile
    folder = make_folder(tempfile.mkdtemp(), cfg, seed=4)
    reqs = {"a": H.random_tokens(300, 90, 1), "b": H.random_tokens(50, 90, 2)}
    for dtype in ("float32", "bfloat16"):
        runner = ModelRunner(folder, dtype=dtype, page_size=8, num_pages=16, max_requests=2, max_model_len=512)
        got = H.run_steps(runner, H.steps_portions(reqs, sizes=(13, 2, 40, 1, 7)))
        compare(got, reqs, folder, TOL[dtype], "short pool " + dtype, CLOSE[dtype])


LARGER = config(384, 1000, [
    (SSM(12, 64, 128, 4, 4, 4), MOE(16, 2, 96, identity=2)),
    (PAR(LEFT(12, 2, 64, 128, 0.2, size=300, cap=50.0), RIGHT(6, 3, 128, 128, 4), 0.9, 1.1), MOE(6, 1, 256, identity=1)),
    (PAR(LEFT(6, 3, 128, 96, 0.2, size=100, cap=30.0), RIGHT(4, 4, 96, 48, 4), 1.1, 0.9), None),
], eps=1e-6, scale=2.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_long_prompt_at_larger_sizes(tmp_path, dtype):
    """1,300 tokens at once (products of many rows), then 30 decoded tokens and a second request in
    portions beside them."""
    folder = make_folder(tmp_path / "m", LARGER, seed=11, std_scale=2.0, edit=lambda t: sharpen(t, 2.0))
    reqs = {"long": H.random_tokens(1330, 1000, 1), "short": H.random_tokens(150, 1000, 2)}
    from ginfer_amd import ModelRunner, StepEntry
    runner = ModelRunner(folder, dtype=dtype, page_size=16, num_pages=-(-1600 // 16), max_requests=4, max_model_len=1600)
    got = {}
    logits = runner.step([StepEntry("long", reqs["long"][:1300], [0, 1, 640, 1299])]).cpu().numpy()
    got.update({("long", p): row for p, row in zip([0, 1, 640, 1299], logits)})
    at = 0
    for k in range(30):
        n = min(7, 150 - at)
        entries = [StepEntry("long", reqs["long"][1300 + k:1301 + k], [0])] + ([StepEntry("short", reqs["short"][at:at + n], [n - 1])] if n else [])
        logits = runner.step(entries).cpu().numpy()
        got[("long", 1300 + k)] = logits[0]
        if n:
            got[("short", at + n - 1)] = logits[1]
            at += n
    runner.cache.check()
    worst = []
    for (rid, p), row in sorted(got.items()):
        ref = plain(folder, reqs[rid])
        worst.append(float(np.abs(row.astype(np.float64) - ref[p]).max() / np.abs(ref).max()))
    assert np.isfinite(worst).all()
    if dtype == "float32":
        assert max(worst) < TOL[dtype], worst
    else:
        assert float(np.median(worst)) < TOL[dtype] / 2 and sum(w > TOL[dtype] for w in worst) <= CLOSE[dtype] * len(worst), worst


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_recorded_steps_equal_launched_ones(folders, dtype):
    reqs = requests_for("mix", [60, 25, 41], seed=80)
    steps = H.steps_mixed(reqs, max_live=3, seed=9)
    outs = []
    for graphs in (True, False):
        runner = runner_for(folders["mix"], "mix", dtype, use_graphs=graphs)
        for rounds in range(3):
            got = H.run_steps(runner, steps)
        outs.append(got)
        if graphs:
            assert runner.use_graphs and runner.counts["replayed_decode"] + runner.counts["replayed_padded"] > 0
    for key, row in outs[0].items():
        if dtype == "float32":
            assert np.array_equal(row, outs[1][key]), key
    if dtype == "bfloat16":
        compare(outs[0], reqs, folders["mix"], TOL[dtype], "recorded", CLOSE[dtype])
        compare(outs[1], reqs, folders["mix"], TOL[dtype], "launched", CLOSE[dtype])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_program(folders, tmp_path, dtype):
    reqs = requests_for("mix", [40, 9, 77], seed=90)
    steps = H.steps_mixed(reqs, max_live=2, seed=2)
    cfg_vocab = CONFIGS["mix"][0]["vocab"]
    import plain_model
    orig = plain_model.read_config
    plain_model.read_config = lambda folder: {"vocab_size": cfg_vocab}          # the helper only asks for the vocabulary
    try:
        got = H.run_trace(folders["mix"], dtype, steps, tmp_path / "out", H.max_live_tokens(steps), page_size=16)
    finally:
        plain_model.read_config = orig
    compare(got, reqs, folders["mix"], TOL[dtype], "trace replay " + dtype, CLOSE[dtype])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(folders, dtype):
    """Engine.generate with its scheduler: five prompts through three slots under a budget of 48 tokens a step.  Every token is
    the plain statement's greedy choice after the engine's own tokens so far (in bfloat16: or within rounding of it)."""
    from ginfer_amd import Engine, EngineConfig, SamplingParams
    name = "mix"
    folder = folders[name]
    prompts = list(requests_for(name, [3, 30, 11, 64, 1], seed=100).values())
    eng = Engine(EngineConfig(model_path=folder, dtype=dtype, max_num_batched_tokens=48, max_num_seqs=3, max_seq_len=256,
                              kvcache_block_size=8, num_kvcache_blocks=96))
    outs = eng.generate(prompts, SamplingParams(max_tokens=24, ignore_eos=True))
    cfg, w = pp.read_config(folder), pp.read_weights(folder)
    far = 0
    for p, o in zip(prompts, outs):
        assert len(o.token_ids) == 24
        logits = pp.forward(cfg, w, (p + o.token_ids)[:-1])
        for k, tok in enumerate(o.token_ids):
            row = logits[len(p) - 1 + k]
            best = int(torch.argmax(row))
            gap = float(row[best] - row[tok]) / float(row.abs().max())
            if dtype == "float32":
                assert tok == best or gap <= 1e-5, "token %d after a prompt of %d: engine %d, plain %d (gap %.3g)" % (k, len(p), tok, best, gap)
            else:
                far += not (tok == best or gap <= 6e-2)
    assert far <= 0.08 * 24 * len(prompts)      # bfloat16: where an expert's choice is a close call, a token and those behind it
    eng.runner.cache.check()


def test_the_pool_is_planned_beside_states_and_windows(folders):
    """No page counts given: the engine plans the groups' pages (windows, all keys) beside the state slots."""
    from ginfer_amd import Engine, EngineConfig, SamplingParams
    folder = folders["mix"]
    eng = Engine(EngineConfig(model_path=folder, dtype="float32", max_num_batched_tokens=64, max_num_seqs=4, max_seq_len=512,
                              kvcache_block_size=8, gpu_memory_utilization=0.05))
    assert sorted(g.window or 0 for g in eng.runner.cache.groups) == [0, 11, 33]
    prompt = requests_for("mix", [90], seed=300)["q0"]
    o = eng.generate([prompt], SamplingParams(max_tokens=12, ignore_eos=True))[0]
    logits = pp.forward(pp.read_config(folder), pp.read_weights(folder), (prompt + o.token_ids)[:-1])
    for k, tok in enumerate(o.token_ids):
        row = logits[len(prompt) - 1 + k]
        assert tok == int(torch.argmax(row)) or float(row.max() - row[tok]) / float(row.abs().max()) <= 1e-5


def test_command_line_generates(folders):
    import subprocess
    import sys
    folder = folders["deep"]
    cmd = [sys.executable, os.path.join(H.ROOT, "bin", "ginfer"), "generate", "--model-path", folder, "--dtype", "float32",
           "--prompt-ids", "1,2,3,4,5", "--max-tokens", "6", "--ignore-eos", "--max-num-seqs", "2", "--max-seq-len", "64",
           "--num-kvcache-blocks", "16"]
    out = subprocess.run(cmd, capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr[-2000:]
    cfg, w = pp.read_config(folder), pp.read_weights(folder)
    ids = [1, 2, 3, 4, 5]
    for _ in range(6):
        ids.append(int(torch.argmax(pp.forward(cfg, w, ids)[-1])))
    assert json.loads(out.stdout.strip().splitlines()[0])["token_ids"] == ids[5:]
