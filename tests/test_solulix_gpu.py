"""Solulix on the GPU: each mechanism's kernels alone against the plain functions of tests/plain, then the model through
the step function, the cache and the generation entry point, in float32 and bfloat16."""
import random

import pytest
import torch

from trapetum_amd.config import SolulixConfig
from trapetum_amd.engine.batch import StepContext
from trapetum_amd.weights import write_model_folder

from . import model_cases as mc
from . import ref_ops
from . import solulix_tiny as st
from .plain import solulix_plain as plain
from .test_lutovik_gpu import DEV, LENS, PART_TOL, STEPS, WIDTH, acts, bound, rnd, rt, run_mixers  # noqa: F401  (rt is the fixture)
from .tiny import random_tokens, rel_l2

pytestmark = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": mc.Rounded(4e-2)}
EPS = 1e-5


def sequences(rt, seed, scale=1.0, lens=LENS):
    seqs, wide = {}, {}
    for i, n in lens.items():
        seqs[i], wide[i] = acts(rt, rnd(n, WIDTH, seed=seed + i) * scale)
    return seqs, wide


def tolerance(rt):
    return PART_TOL[rt.dtype] * (3 if rt.dtype == torch.float32 else 1.5)


# ---- the gated delta rule ---------------------------------------------------------------------------------------------------
SCAN_LENS = (1, 7, 33, 64, 97, 130, 257)
SCAN_SLOTS = (5, 0, 3, 9, 1, 7, 2)


@pytest.mark.parametrize("chunks", [False, True, None])
@pytest.mark.parametrize("heads,kv,dk,dv,rate", [
    (4, 2, 64, 64, 0.0), (3, 1, 128, 48, -4.0), (2, 2, 16, 20, 2.0), (6, 3, 96, 33, -2.0), (2, 1, 256, 128, -3.0), (1, 1, 40, 16, 0.0),
    (2, 2, 192, 64, -6.0), (3, 3, 10, 7, 0.0)])
def test_delta_scan(rt, heads, kv, dk, dv, rate, chunks):
    """Sequences of unequal lengths from states that are not zero, row by row and in chunks (a last chunk of one row, a
    sequence shorter than a chunk, one exactly a chunk long), against float64; the decays range from almost none to almost
    all, and some keys repeat so that what is written is unlearned again."""
    if chunks and (rt.dtype == torch.float32 or dk % 8):
        pytest.skip("rows of this kind have no chunks")
    cu = torch.tensor([0] + list(torch.tensor(SCAN_LENS).cumsum(0)), dtype=torch.int32)
    slots, M = torch.tensor(SCAN_SLOTS, dtype=torch.int32), sum(SCAN_LENS)
    width = 2 * kv * dk + heads * dv + 2 * heads
    rows = rnd(M, width + (-width % 8), seed=60, scale=0.7)
    k = rows[:, kv * dk:2 * kv * dk]
    k[3::5] = k[2::5][:k[3::5].shape[0]]                  # a key right after itself
    rows[:, 2 * kv * dk + heads * dv + heads:] *= 2.0     # the decays' sums spread widely
    rows, wide = acts(rt, rows)
    cut = lambda t: (t[:, :kv * dk], t[:, kv * dk:2 * kv * dk], t[:, 2 * kv * dk:2 * kv * dk + heads * dv],
                     t[:, 2 * kv * dk + heads * dv:2 * kv * dk + heads * dv + heads], t[:, 2 * kv * dk + heads * dv + heads:width])
    a_log, dt_bias = rnd(heads, seed=61, scale=0.5) + rate, rnd(heads, seed=62, scale=0.5)
    state = rnd(10, heads, dk, dv, seed=66, scale=0.3)
    want_state, got_state = state.double(), state.to(rt.device)
    want = ref_ops.delta_scan(*cut(wide), a_log, dt_bias, want_state, slots, cu, max(SCAN_LENS), heads, kv, dk, dv, dk ** -0.5)
    got = rt.ops.delta_scan(*cut(rows), a_log.to(rt.device), dt_bias.to(rt.device), got_state, slots.to(rt.device), cu.to(rt.device),
                            max(SCAN_LENS), heads, kv, dk, dv, dk ** -0.5, chunks=chunks)
    for i in range(len(SCAN_LENS)):
        assert rel_l2(got[cu[i]:cu[i + 1]], want[cu[i]:cu[i + 1]]) < 1e-5, i
        assert rel_l2(got_state[SCAN_SLOTS[i]], want_state[SCAN_SLOTS[i]].float()) < 1e-5, i
    assert torch.equal(got_state[[4, 6, 8]].cpu(), state[[4, 6, 8]])          # slots of no sequence are left alone


def delta_tensors(H, G, dim, vdim, taps, seed=0, a_log=0.0):
    T = {"q": rnd(G * dim, WIDTH, seed=seed + 1, scale=0.25), "k": rnd(G * dim, WIDTH, seed=seed + 2, scale=0.25),
         "v": rnd(H * vdim, WIDTH, seed=seed + 3, scale=0.3), "g": rnd(H * vdim, WIDTH, seed=seed + 4, scale=0.3),
         "b": rnd(H, WIDTH, seed=seed + 5, scale=0.3), "a": rnd(H, WIDTH, seed=seed + 6, scale=0.3),
         "A_log": rnd(H, seed=seed + 7, scale=0.5) + a_log, "dt_bias": rnd(H, seed=seed + 8, scale=0.5),
         "norm": 1.0 + rnd(vdim, seed=seed + 9, scale=0.3), "o": rnd(WIDTH, H * vdim, seed=seed + 10, scale=0.2)}
    for i, s in enumerate("qkv"):
        T[s + ".conv"] = rnd(T[s].shape[0], taps, seed=seed + 11 + i, scale=0.5)
    return T


def delta_part(rt, H, G, dim, vdim, taps, **kw):
    ref = ("gated_delta", dict(hidden_size=WIDTH, num_heads=H, num_kv_heads=G, key_dim=dim, value_dim=vdim, conv_taps=taps, norm_eps=EPS))
    part, W = bound(rt, "mixer", ref, delta_tensors(H, G, dim, vdim, taps, **kw))
    return part, W, {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "conv": taps}


@pytest.mark.parametrize("H,G,dim,vdim,taps,a_log", [
    (4, 2, 24, 40, 4, 0.0), (3, 3, 72, 70, 2, -3.0), (1, 1, 16, 16, 1, 0.0), (6, 2, 48, 64, 3, -5.0), (2, 1, 136, 200, 4, -2.0), (4, 1, 4, 6, 5, 1.0),
    (2, 2, 64, 32, 8, -4.0)])
def test_delta_part(rt, H, G, dim, vdim, taps, a_log):
    """The mixer in prompts, single tokens and portions down to two rows (fewer than the convolutions' taps), two sequences
    side by side."""
    part, W, sizes = delta_part(rt, H, G, dim, vdim, taps, a_log=a_log)
    seqs, wide = sequences(rt, 29)
    got = run_mixers(rt, [(part, 0)], seqs, STEPS)
    for i in seqs:
        # bfloat16: a head whose output is small is divided by its small root mean square, its rounding with it
        assert rel_l2(got[i][0], plain.delta(wide[i], W, "", sizes, EPS)) < tolerance(rt) * (1 if rt.dtype == torch.float32 else 2), i


@pytest.mark.parametrize("m,n,c,taps,slices,act", [(1, 40, 40, 3, 0, None), (5, 700, 333, 4, 3, "silu"), (8, 96, 64, 1, 5, "silu"), (3, 130, 130, 2, 1, None),
                                                   (64, 300, 20, 6, 2, "silu")])
def test_convolution_of_single_rows(rt, m, n, c, taps, slices, act):
    """One row per sequence, from a product in K slices or in one piece: the first columns are convolved, the others pass; the
    states move on by the rows as they were used."""
    rows = rnd(slices, m, n, seed=1) if slices else acts(rt, rnd(m, n, seed=1))[1].to(rt.dtype)
    w_t, state = rnd(taps, c, seed=2, scale=0.5), rnd(m + 3, max(taps - 1, 1), c, seed=3)
    slots = torch.randperm(m + 3, generator=torch.Generator().manual_seed(4))[:m].to(torch.int32)
    want_state, got_state = state.clone(), state.to(rt.device)
    x = ref_ops.SplitRows(rows) if slices else rows
    want = ref_ops.conv_step(x, w_t, want_state if taps > 1 else None, slots, rt.dtype, act)
    x = rt.ops.SplitRows(rows.to(rt.device)) if slices else rows.to(rt.device)
    got = rt.ops.conv_step(x, w_t.to(rt.device), got_state if taps > 1 else None, slots.to(rt.device), rt.dtype, act)
    assert got.shape == (m, n) and rel_l2(got, want) < (1e-6 if rt.dtype == torch.float32 else 3e-3)
    assert rel_l2(got_state, want_state) < (1e-6 if rt.dtype == torch.float32 else 3e-3)
    untouched = [s for s in range(m + 3) if s not in slots.tolist()]
    assert torch.equal(got_state[untouched].cpu(), state[untouched])


def test_delta_remembers_and_unlearns(rt):
    """Decays of almost one and steps of almost one: hundreds of tokens after its first tokens the memory still answers to a
    key with what was written there last, not with what that key held before."""
    dk = dv = 32
    n = 300
    q, k = torch.zeros(n, dk), torch.zeros(n, dk)
    v = torch.zeros(n, dv)
    k[:, 5] = 3.0                                        # every later token writes nothing to key 5 ...
    k[0], k[1] = torch.eye(dk)[0], torch.eye(dk)[0]
    v[0], v[1] = rnd(dv, seed=1), rnd(dv, seed=2)        # key 0 takes a value, then another
    q[:, 0] = 1.0
    gates = torch.full((n, 2), 12.0)                     # beta = sigmoid(12)
    gates[:, 1] = -12.0                                  # softplus(-12) = 6e-6
    rows, _ = acts(rt, torch.cat([q, k, v, gates], dim=1))
    one = lambda x: torch.tensor([x], device=rt.device)
    for chunks in (False, None):
        state = torch.zeros(1, 1, dk, dv, device=rt.device)
        y = rt.ops.delta_scan(rows[:, :dk], rows[:, dk:2 * dk], rows[:, 2 * dk:3 * dk], rows[:, 3 * dk:3 * dk + 1], rows[:, 3 * dk + 1:], one(0.0), one(0.0),
                              state, torch.zeros(1, dtype=torch.int32, device=rt.device), torch.tensor([0, n], dtype=torch.int32, device=rt.device),
                              n, 1, 1, dk, dv, 1.0, chunks=chunks).cpu()
        want = v[1].to(rt.dtype).float()
        assert rel_l2(y[0], v[0].to(rt.dtype).float()) < 1e-4
        assert rel_l2(y[1], want) < 1e-4
        assert rel_l2(y[-1], want) < 5e-3, chunks


# ---- attention: convolutions on q, k and v, a window beside the first positions, one in the denominator -----------------------
def conv_attention(rt, H, G, dim, vdim, taps, size, keep, scale=0.3, seed=0, edit=None):
    ref = ("attention", dict(hidden_size=WIDTH, num_heads=H, num_kv_heads=G, head_dim=dim, value_dim=vdim, query_scale=scale, window=size,
                             keep_first=keep, conv=taps, sink=0.0, position=("none", {}), precise_weights=True, tensors=("q", "k", "v", "o")))
    T = {"q": rnd(H * dim, WIDTH, seed=seed + 1, scale=0.25), "k": rnd(G * dim, WIDTH, seed=seed + 2, scale=0.25),
         "v": rnd(G * vdim, WIDTH, seed=seed + 3, scale=0.3), "o": rnd(WIDTH, H * vdim, seed=seed + 4, scale=0.2)}
    for i, s in enumerate("qkv"):
        T[s + ".conv"] = rnd(T[s].shape[0], taps, seed=seed + 5 + i, scale=0.5)
    if edit is not None:
        edit(T)
    part, W = bound(rt, "mixer", ref, T)
    return part, W, {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "conv": taps, "scale": scale, "mask": {"size": size, "keep_first": keep}}


@pytest.mark.parametrize("page", [16, 64])
@pytest.mark.parametrize("H,G,dim,vdim,taps,size,keep", [
    (4, 2, 16, 24, 4, 11, 5), (3, 3, 24, 8, 2, 20, 19), (2, 1, 32, 32, 1, 16, 16), (1, 1, 12, 12, 3, 1, 1), (8, 2, 64, 64, 3, 33, 20),
    (6, 3, 48, 80, 2, 40, 0), (4, 4, 128, 64, 4, 7, 33), (10, 1, 40, 72, 5, 64, 17), (2, 2, 80, 96, 3, 1000, 4), (32, 2, 16, 16, 2, 50, 64)])
def test_conv_attention_part(rt, H, G, dim, vdim, taps, size, keep, page):
    part, W, sizes = conv_attention(rt, H, G, dim, vdim, taps, size, keep)
    seqs, wide = sequences(rt, 9)
    got = run_mixers(rt, [(part, 0)], seqs, STEPS, page=page)
    for i in seqs:
        assert rel_l2(got[i][0], plain.attention(wide[i], W, "", sizes, EPS)) < tolerance(rt), i


def rows_differ(a, b):
    return float(((a - b).norm(dim=1) / b.norm(dim=1)).max())


@pytest.mark.parametrize("at", [4, 5, 6])
@pytest.mark.parametrize("page,first", [(16, 24), (16, 25), (16, 26), (16, 27), (16, 32), (16, 33), (64, 64), (64, 6)])
def test_one_key_at_the_edges(rt, page, first, at):
    """One early key is made to stand out for every later query: the last kept position, the first that is not, the next.
    A kept one decides every later output; another decides as long as the window holds it.  The step's border is put just
    before, on and just after the window's edge, in a prompt, a portion and single tokens."""
    H, G, dim, vdim, size, keep = 4, 2, 16, 24, 20, 5

    def mark(T):                                         # a head's last element: keys read column 5 of the input, queries column 7
        for name, heads, col in (("k", G, 5), ("q", H, 7)):
            w = T[name].view(heads, dim, WIDTH)
            w[:, dim - 1, :] = 0.0
            w[:, dim - 1, col] = 1.0
            taps = T[name + ".conv"].view(heads, dim, -1)
            taps[:, dim - 1] = 0.0
            taps[:, dim - 1, -1] = 1.0
    part, W, sizes = conv_attention(rt, H, G, dim, vdim, 3, size, keep, scale=0.25, seed=7, edit=mark)
    n = max(first, 34) + 2 * page + 9
    x = rnd(n, WIDTH, seed=3) * 0.3
    x[:, 5] = 0.0
    x[at, 5] = 16.0                                      # the marked key
    x[:, 7] = 4.0                                        # every query meets it with a large score
    x_dev, xw = acts(rt, x)
    want = plain.attention(xw, W, "", sizes, EPS)
    steps = [{0: first}, {0: 2 * page + 1}] + [{0: 1}] * (n - first - 2 * page - 1)
    got = run_mixers(rt, [(part, 0)], {0: x_dev}, steps, page=page)[0][0]
    assert rel_l2(got, want) < (2e-5 if rt.dtype == torch.float32 else 2e-2)
    assert rows_differ(got.double().cpu(), want) < (1e-4 if rt.dtype == torch.float32 else 6e-2)
    # and the outputs do rest on the edges: a window one longer or shorter, a kept position more or fewer, shows
    other = {4: (0, -1), 5: (0, 1), 6: (1, 0)}[at]
    mask = {"size": size + other[0], "keep_first": keep + other[1]}
    assert rows_differ(plain.attention(xw, W, "", dict(sizes, mask=mask), EPS), want) > 0.3


def test_one_in_the_denominator(rt):
    """Scores far below zero: with one added to the denominator a head's output vanishes; without it it would not."""
    def low(T):                                          # every score is about -60
        for name, heads, dim, sign in (("k", 1, 16, 1.0), ("q", 2, 16, -1.0)):
            T[name].view(heads, dim, WIDTH)[:, 0, :] = 0.0
            T[name].view(heads, dim, WIDTH)[:, 0, 3] = sign
            T[name + ".conv"][:] = 0.0
            T[name + ".conv"][:, -1] = 1.0
    part, W, sizes = conv_attention(rt, 2, 1, 16, 16, 2, 9, 2, scale=1.0, seed=17, edit=low)
    x = rnd(60, WIDTH, seed=4) * 0.1
    x[:30, 3] = 8.0
    x[30:, 3] = 1.5                                      # then scores about zero: the one takes its share
    x_dev, xw = acts(rt, x)
    want = plain.attention(xw, W, "", sizes, EPS)
    got = run_mixers(rt, [(part, 0)], {0: x_dev}, [{0: 20}, {0: 3}] + [{0: 1}] * 37)[0][0].double().cpu()
    assert float(want[5:30].abs().max()) < 1e-9 and float(got[5:30].abs().max()) < 1e-9
    assert rel_l2(got[42:], want[42:]) < tolerance(rt) and float(want[42:].abs().max()) > 1e-3


def test_matrix_core_kernels_over_many_tiles():
    """Sequences long enough for every wave of a block to take several tiles of keys and for a decode step's keys to be
    cut in slices: the matrix-core kernels against the plain kernels on the same rows."""
    from trapetum_amd.engine.runtime import Runtime
    rt = Runtime(dtype="bfloat16", device=DEV)
    for H, G, dim, size, keep in ((8, 4, 128, 300, 100), (4, 2, 64, 129, 7), (2, 1, 256, 500, 64), (12, 2, 32, 64, 200)):
        part, W, sizes = conv_attention(rt, H, G, dim, dim, 4, size, keep, scale=0.5)
        seqs, _ = sequences(rt, 59, lens={0: 1500, 1: 180})
        steps = [{0: 700, 1: 100}, {0: 1, 1: 1}, {0: 150, 1: 2}, {0: 500}] + [{0: 1, 1: 1}] * 49 + [{0: 100, 1: 28}]
        got = run_mixers(rt, [(part, 0)], seqs, steps, page=64)
        rt.ops.force_plain_attention = True
        try:
            slow = run_mixers(rt, [(part, 0)], seqs, steps, page=64)
        finally:
            rt.ops.force_plain_attention = False
        for i in seqs:
            assert rel_l2(got[i][0], slow[i][0]) < 6e-3, (H, G, dim, size, keep, i)


# ---- feed-forwards, the router, the block's add ----------------------------------------------------------------------------------
def run_ff(rt, part, x):
    class Ctx:
        ops, dtype = rt.ops, rt.dtype
    return rt.ops.rows(part.forward(Ctx, x), torch.float32)


@pytest.mark.parametrize("m,d,f", [(1, 64, 40), (2, 96, 200), (5, 72, 33), (8, 256, 512), (40, 72, 100), (300, 128, 136), (700, 256, 300)])
def test_squared_relu_feed_forward(rt, m, d, f):
    T = {"up": rnd(f, d, seed=1, scale=0.2), "down": rnd(d, f, seed=2, scale=0.2)}
    part, W = bound(rt, "feed_forward", ("plain_mlp", dict(hidden_size=d, intermediate_size=f)), T)
    x, xw = acts(rt, rnd(m, d, seed=3))
    assert rel_l2(run_ff(rt, part, x), plain.squared_relu_expert(xw, W, "")) < PART_TOL[rt.dtype]


@pytest.mark.parametrize("m,d,f,e,identity,top,shared", [
    (1, 64, 40, 4, 2, 3, 24), (5, 72, 33, 5, 1, 6, None), (9, 128, 64, 1, 1, 1, 64), (40, 96, 48, 7, 0, 2, 30), (300, 128, 64, 12, 3, 4, 96),
    (700, 64, 128, 3, 2, 2, None), (400, 256, 72, 2, 1, 3, 40), (20, 64, 1024, 3, 1, 2, None), (3, 50, 18, 2, 3, 4, 18)])
def test_router_identity_and_shared_experts(rt, m, d, f, e, identity, top, shared):
    """The correction moves the choice and not the weights; identity outputs stand after the experts; rows chosen by the plain
    router of the same rounded inputs."""
    T = {"router": rnd(e + identity, d, seed=1, scale=0.25), "correction": rnd(e + identity, seed=2, scale=0.2)}
    for k in range(e):
        T[f"e{k}.up"], T[f"e{k}.down"] = rnd(f, d, seed=10 + 2 * k, scale=0.2), rnd(d, f, seed=11 + 2 * k, scale=0.2)
    ref = dict(hidden_size=d, intermediate_size=f, n_experts=e, identity=identity, top=top, limit=None, expert_kind="relu2", tensors=("up", "down"),
               renormalize=True, correction="correction", weight_scale=1.7)
    if shared is not None:
        T["shared.up"], T["shared.down"] = rnd(shared, d, seed=7, scale=0.2), rnd(d, shared, seed=8, scale=0.2)
        ref["shared"] = ("plain_mlp", dict(hidden_size=d, intermediate_size=shared, prefix="shared."))
    part, W = bound(rt, "feed_forward", ("routed_experts", ref), T)
    x, xw = acts(rt, rnd(m, d, seed=3))
    cfg = {"kind": "moe", "expert": {"ff": f}, "router": {"experts": e, "identity": identity, "scale": 1.7, "top": top}}
    if shared is not None:
        cfg["shared"] = {"ff": shared}
    want = plain.feed_forward(xw, W, "", cfg)
    got = run_ff(rt, part, x).double().cpu()
    # a close call between two choices may fall the other way in float32: such rows are left out, and they are few
    s = torch.softmax(xw @ W["router"].T, dim=1) + W["correction"]
    ordered = s.sort(dim=1, descending=True).values
    clear = ordered[:, top - 1] - ordered[:, top] > 1e-5 if top < e + identity else torch.ones(m, dtype=torch.bool)
    assert int((~clear).sum()) <= m // 50
    assert rel_l2(got[clear], want[clear]) < PART_TOL[rt.dtype]
    if identity:
        chosen, _ = plain.router_choice(xw, W, "", cfg["router"])
        assert bool((chosen >= e).any()), "the case is meant to choose identity outputs too"


@pytest.mark.parametrize("m,d", [(1, 50), (3, 64), (8, 2304), (200, 96), (300, 2304), (5, 3584), (2, 9000), (150, 1001), (4, 8192)])
def test_join_rms_norm(rt, m, d):
    """Rows of both kinds and K slices, the vector and the earlier rows, each there or not."""
    ops = rt.ops
    gain = (1 + rnd(d, seed=1, scale=0.3)).to(DEV)
    stream0, origin, vec = rnd(m, d, seed=2), rnd(m, d, seed=3), rnd(d, seed=4)
    slices = rnd(3, m, d, seed=5)
    plain_rows = rnd(m, d, seed=6).to(rt.dtype)
    f32_rows = rnd(m, d, seed=7)
    if d > 8192 and d % 4:
        pytest.skip("no kernel")
    cases = [(plain_rows, None), (plain_rows, slices), (slices, f32_rows), (None, None), (f32_rows, plain_rows)]
    for a, b in cases:
        for with_vec, with_origin, with_gain in ((False, False, True), (True, False, True), (True, True, True), (True, True, False)):
            dev = lambda t: None if t is None else (ops.SplitRows(t.to(DEV)) if t.dim() == 3 else t.to(DEV))
            stream = stream0.to(DEV)
            out = ops.join_rms_norm(stream, dev(a), dev(b), gain if with_gain else None, 1e-5, rt.dtype, vec=vec.to(DEV) if with_vec else None,
                                    origin=origin.to(DEV) if with_origin else None)
            want = stream0.double()
            for t in (a, b):
                if t is not None:
                    want = want + (t.double().sum(0) if t.dim() == 3 else t.double())
            want = want + (origin.double() if with_origin else 0) + (vec.double() if with_vec else 0)
            assert rel_l2(stream, want) < 1e-6
            if with_gain:
                assert rel_l2(out, plain.over_rms(want, 1e-5) * gain.double().cpu()) < (1e-6 if rt.dtype == torch.float32 else 4e-3)
            else:
                assert out is None


# ---- the model ---------------------------------------------------------------------------------------------------------------------
def loaded(tmp_path_factory, which, dtype, tol):
    from .gpu_engine import load_gpu_model
    folder = st.make_folder(tmp_path_factory.mktemp("s"), which)
    model, cfg = load_gpu_model(folder, dtype)
    pcfg, pw = plain.read_folder(folder)
    return model, cfg, pcfg, pw, tol


@pytest.fixture(scope="module", params=[("P", "float32"), ("Q", "float32"), ("R", "float32"), ("P", "bfloat16"), ("Q", "bfloat16"), ("R", "bfloat16")],
                ids=lambda p: "-".join(p))
def m(request, tmp_path_factory):
    which, dtype = request.param
    return loaded(tmp_path_factory, which, dtype, TOL[dtype])


@pytest.fixture(scope="module")
def sharp(tmp_path_factory):
    return loaded(tmp_path_factory, "S", "float32", 4e-3)


def test_whole_and_token_by_token(m):
    mc.whole_and_token_by_token(m)


def test_prompt_then_long_decode(m):
    mc.prompt_then_decode(m, n=150, tail=100)


def test_portions(m):
    mc.portions(m)


def test_unequal_batches_and_reuse(m):
    mc.unequal_batches_and_reuse(m)


def test_slot_after_a_longer_sequence(m):
    mc.slot_after_a_longer_sequence(m)


def test_sharp_scores_at_the_edges(sharp):
    mc.sharp_scores_far_keys(sharp, n=110)


def test_layers_one_by_one(m):
    """The residual stream after every run of a layer, a looped layer's passes included (what comes before the next pass is
    added in the same kernel and is in the stream by then)."""
    model, cfg, pcfg, pw, tol = m
    toks = random_tokens(41, cfg.vocab_size, 5)
    want = []
    plain.forward(pcfg, pw, toks, layers_out=want)
    start = plain.over_rms(pw["embed"][torch.tensor(toks)], pcfg["norm"]["eps"]) * pw["embed.norm"]
    for i, (_, turn) in enumerate(plain.running_order(pcfg)[1:]):
        if turn is not None:
            want[i] = want[i] + pw["loop.step"][turn] + (start if turn > 0 else 0.0)
    got = []
    cache = model.new_cache(max_tokens=128, page_size=16)
    s = cache.acquire()
    counts, starts, rows, tok = model.prepare(cache, [s], toks, counts=[len(toks)], want=[])
    ctx = StepContext(model.rt, cache, [s], counts, starts, rows)
    ctx.dump = lambda stage, x: got.append(x.clone()) if stage == "layer_out" else None
    model.run(ctx, tok)
    assert len(got) == len(want) == len(model.schedule)
    for i, (a, b) in enumerate(zip(got, want)):
        mc.rows_close(a, b, tol, i)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", range(8))
def test_random_configuration(case, dtype, tmp_path):
    """A configuration drawn at random: a prompt whole, then in two portions and single tokens."""
    from .gpu_engine import load_gpu_model
    rng = random.Random(1300 + case)
    cfg = st.draw(rng)
    folder = str(tmp_path)
    write_model_folder(SolulixConfig.from_dict(cfg), folder, seed=case, sigma=0.1, sigma_norm=0.2)
    model, c = load_gpu_model(folder, dtype)
    pcfg, pw = plain.read_folder(folder)
    toks = random_tokens(90, c.vocab_size, case)
    ref = plain.forward(pcfg, pw, toks)
    cache = model.new_cache(max_tokens=192, page_size=16)
    s = cache.acquire()
    got = [model.step(cache, [s], toks[:20], counts=[20], want=list(range(20))),
           model.step(cache, [s], toks[20:79], counts=[59], want=list(range(59)))]
    got += [model.step(cache, [s], [t]) for t in toks[79:]]
    mc.rows_close(torch.cat(got), ref, 5e-5 if dtype == "float32" else mc.Rounded(6e-2), cfg)


@pytest.mark.parametrize("which,dtype", [("P", "float32"), ("Q", "float32"), ("P", "bfloat16"), ("R", "bfloat16")])
def test_greedy_generation_through_the_entry_point(which, dtype, tmp_path):
    from trapetum_amd import load_model
    folder = st.make_folder(tmp_path, which)
    pcfg, pw = plain.read_folder(folder)
    prompts = [random_tokens(n, pcfg["vocab"], 90 + n) for n in (7, 1, 19, 4, 33)]
    engine = load_model(folder, dtype=dtype, max_tokens_in_cache=64 * 3, max_batch=3)      # graphs on; slots are used again
    got = engine.generate(prompts, max_tokens=24, stop_ids=())
    assert [len(g) for g in got] == [24] * len(prompts)
    if dtype == "float32":
        assert got == [plain.greedy_generate(pcfg, pw, p, 24) for p in prompts]
    again = engine.generate(prompts[::-1], max_tokens=24, stop_ids=())       # replayed graphs, other slots
    assert again == got[::-1]
    assert engine.cache.live_slots() == []


def test_replayed_steps_are_the_eager_ones(tmp_path):
    """A decode step replayed from its graph, again and again with eager work between the replays, gives the eager step's
    logits bit for bit."""
    from trapetum_amd.engine.graphs import GraphedDecode
    from .gpu_engine import load_gpu_model
    model, cfg = load_gpu_model(st.make_folder(tmp_path, "P"), "bfloat16")
    caches = [model.new_cache(max_tokens=512, page_size=64, max_slots=4) for _ in range(2)]
    toks = [random_tokens(40, cfg.vocab_size, 7 + i) for i in range(3)]
    slots = [[c.acquire() for _ in toks] for c in caches]
    for c, s in zip(caches, slots):
        model.step(c, s, sum((t[:9] for t in toks), []), counts=[9] * 3)
    graphs = GraphedDecode(model, caches[1])
    for j in range(9, 40):
        step = [t[j] for t in toks]
        eager = model.step(caches[0], slots[0], step)
        torch.cuda.synchronize()
        assert torch.equal(graphs.step(slots[1], step), eager), j


def test_command_line_and_trace_runner(tmp_path):
    """`python -m trapetum_amd random | run` and bin/trace_run on a Solulix folder: the model class comes from config.json,
    the ids and logits are the plain implementation's."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    from . import trace_schedules as ts
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

    def run(cmd, **kw):
        p = subprocess.run(cmd, cwd=root, capture_output=True, text=True, timeout=100, **kw)
        assert p.returncode == 0, p.stderr[-2000:]
        return p.stdout
    cfg, init = st.CONFIGS["P"]
    config = tmp_path / "config.json"
    config.write_text(json.dumps(cfg))
    folder = tmp_path / "model"
    module = [sys.executable, "-m", "trapetum_amd"]
    assert "wrote" in run(module + ["random", "--config", str(config), "--out", str(folder), "--seed", str(init["seed"]),
                                    "--sigma", str(init["sigma"]), "--sigma-norm", str(init["sigma_norm"])])
    pcfg, pw = plain.read_folder(str(folder))
    prompt = random_tokens(13, pcfg["vocab"], 95)
    out = run(module + ["run", str(folder), "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "7", "--dtype", "float32"])
    assert out.strip() == f"continuation ids: {plain.greedy_generate(pcfg, pw, prompt, 7)}"
    requests = {f"r{i}": random_tokens(n, pcfg["vocab"], 20 + i) for i, n in enumerate([40, 3, 21])}
    ref = {rid: plain.forward(pcfg, pw, t) for rid, t in requests.items()}
    for name, steps in (("tail", ts.last_one_by_one(requests, 12)), ("batches", ts.batches(requests, 3))):
        out_dir = tmp_path / name
        stdout = run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(folder), "--dtype", "float32", "--out", str(out_dir),
                      "--max-tokens", str(ts.held_tokens(steps))], input="".join(json.dumps(s) + "\n" for s in steps))
        assert [l for l in stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
        outputs = {s["step"]: np.fromfile(out_dir / f"{s['step']}.f32", dtype="<f4") for s in steps if any(e["want"] for e in s["entries"])}
        got = ts.collect(steps, outputs, pcfg["vocab"])
        for rid in requests:
            mc.rows_close(torch.from_numpy(got[rid]), ref[rid], 2e-5, (name, rid))
