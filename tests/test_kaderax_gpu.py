"""Kaderax on the GPU: each mechanism's kernels alone against the plain functions of tests/plain, then the model through
the step function, the cache and the generation entry point, in float32 and bfloat16."""
import random

import pytest
import torch

from trapetum_amd.config import KaderaxConfig
from trapetum_amd.engine.batch import StepContext
from trapetum_amd.weights import write_model_folder

from . import kaderax_tiny as kt
from . import model_cases as mc
from . import ref_ops
from .plain import kaderax_plain as plain
from .test_lutovik_gpu import DEV, LENS, PART_TOL, STEPS, WIDTH, acts, bound, rnd, rt, run_mixers  # noqa: F401  (rt is the fixture)
from .tiny import random_tokens, rel_l2

pytestmark = pytest.mark.gpu
TOL = {"float32": 2e-5, "bfloat16": 4e-2}
EPS = 1e-5


def sequences(rt, seed, scale=1.0, lens=LENS):
    seqs, wide = {}, {}
    for i, n in lens.items():
        seqs[i], wide[i] = acts(rt, rnd(n, WIDTH, seed=seed + i) * scale)
    return seqs, wide


def tolerance(rt):
    return PART_TOL[rt.dtype] * (3 if rt.dtype == torch.float32 else 1.5)


def rows_differ(a, b):
    return float(((a - b).norm(dim=1) / b.norm(dim=1)).max())


# ---- linear attention with a constant decay -----------------------------------------------------------------------------------
SCAN_LENS = (1, 7, 33, 64, 97, 130, 600)
SCAN_SLOTS = (5, 0, 3, 9, 1, 7, 2)
DECAYS = (0.999, 0.3, 0.95, 0.0, 1.0, 0.7)


@pytest.mark.parametrize("chunks", [False, True, None])
@pytest.mark.parametrize("heads,dk,dv", [(4, 64, 64), (3, 128, 48), (2, 16, 24), (6, 96, 40), (2, 256, 128), (1, 40, 16), (2, 192, 72), (3, 10, 7),
                                         (2, 32, 200), (1, 8, 8), (5, 36, 33)])
def test_linear_scan(rt, heads, dk, dv, chunks):
    """Sequences of unequal lengths from states that are not zero, row by row and in chunks (a last chunk of one row, a
    sequence shorter than a chunk, one exactly a chunk long), against float64; decays of 0, 1 and in between."""
    if chunks and (rt.dtype == torch.float32 or dk % 8 or dv % 8):
        pytest.skip("rows of this kind have no chunks")
    cu = torch.tensor([0] + list(torch.tensor(SCAN_LENS).cumsum(0)), dtype=torch.int32)
    slots, M = torch.tensor(SCAN_SLOTS, dtype=torch.int32), sum(SCAN_LENS)
    width = heads * (2 * dk + dv)
    rows, wide = acts(rt, rnd(M, width + (-width % 8), seed=60, scale=0.7))
    cut = lambda t: (t[:, :heads * dk], t[:, heads * dk:2 * heads * dk], t[:, 2 * heads * dk:width])
    decay = torch.tensor(DECAYS[:heads])
    state = rnd(10, heads, dv, dk, seed=66, scale=0.3)
    want_state, got_state = state.double(), state.to(rt.device)
    args = (heads, dk, dv)
    want = ref_ops.linear_scan(*cut(wide), decay, want_state, slots, cu, max(SCAN_LENS), *args)
    got = rt.ops.linear_scan(*cut(rows), decay.to(rt.device), got_state, slots.to(rt.device), cu.to(rt.device), max(SCAN_LENS), *args, chunks=chunks)
    for i in range(len(SCAN_LENS)):
        assert rel_l2(got[cu[i]:cu[i + 1]], want[cu[i]:cu[i + 1]]) < 3e-6, i
        assert rel_l2(got_state[SCAN_SLOTS[i]], want_state[SCAN_SLOTS[i]].float()) < 3e-6, i
        for h in range(heads):                            # a head whose memory fades is not drowned by one whose memory stays
            a, b = (t.reshape(M, heads, dv)[cu[i]:cu[i + 1], h] for t in (got.cpu(), want))
            assert rel_l2(a, b) < 1e-5, (i, h)
    assert torch.equal(got_state[[4, 6, 8]].cpu(), state[[4, 6, 8]])          # slots of no sequence are left alone


def linear_part(rt, dim, vdim, decay, seed=0):
    H = len(decay)
    T = {"q": rnd(H * dim, WIDTH, seed=seed + 1, scale=0.25), "k": rnd(H * dim, WIDTH, seed=seed + 2, scale=0.25),
         "v": rnd(H * vdim, WIDTH, seed=seed + 3, scale=0.3), "g": rnd(H * vdim, WIDTH, seed=seed + 4, scale=0.3),
         "norm": 1.0 + rnd(H * vdim, seed=seed + 5, scale=0.3), "o": rnd(WIDTH, H * vdim, seed=seed + 6, scale=0.2)}
    part, W = bound(rt, "mixer", ("linear_attention", dict(hidden_size=WIDTH, num_heads=H, key_dim=dim, value_dim=vdim, decay=decay, norm_eps=EPS)), T)
    return part, W, {"heads": H, "dim": dim, "vdim": vdim, "decay": list(decay)}


@pytest.mark.parametrize("dim,vdim,decay", [(24, 40, (0.6, 0.9, 0.99, 0.9995)), (72, 70, (0.5, 0.8, 0.97)), (16, 16, (0.9,)), (48, 64, (0.3, 0.6, 0.9, 0.99)),
                                            (136, 200, (0.9, 0.999)), (4, 6, (1.0, 0.5, 0.0)), (64, 32, (0.99, 0.7)), (128, 128, (0.95, 0.5, 0.99))])
def test_linear_part(rt, dim, vdim, decay):
    """The mixer in prompts, single tokens and portions down to two rows, two sequences side by side."""
    part, W, sizes = linear_part(rt, dim, vdim, decay)
    seqs, wide = sequences(rt, 29)
    got = run_mixers(rt, [(part, 0)], seqs, STEPS)
    for i in seqs:
        assert rel_l2(got[i][0], plain.lightning(wide[i], W, "", sizes, EPS)) < tolerance(rt), i


def test_linear_memory_of_a_first_token(rt):
    """What a first token wrote answers to its key hundreds of tokens later, decayed by exactly so many powers, in a prompt,
    in portions and in single tokens."""
    dk, dv, n, g = 16, 8, 400, 0.995
    q, k, v = torch.zeros(n, dk), torch.zeros(n, dk), torch.zeros(n, dv)
    k[0, 2], v[0] = 1.0, rnd(dv, seed=1)
    k[1:, 5], v[1:] = 1.0, rnd(n - 1, dv, seed=2)          # every later token writes to another key
    q[:, 2] = 1.0
    rows, wide = acts(rt, torch.cat([q, k, v], dim=1))
    want = torch.stack([float(torch.tensor(g, dtype=torch.float32)) ** t * wide[0, 2 * dk:] for t in range(n)])
    for cuts in ((n,), (200, 200), (130, 2, 1, 1, 66, 200), (64, 64, 64, 208)):
        state, at, got = torch.zeros(1, 1, dv, dk, device=rt.device), 0, []
        for c in cuts:
            r = rows[at:at + c]
            got.append(rt.ops.linear_scan(r[:, :dk], r[:, dk:2 * dk], r[:, 2 * dk:], torch.tensor([g], device=rt.device), state,
                                          torch.zeros(1, dtype=torch.int32, device=rt.device), torch.tensor([0, c], dtype=torch.int32, device=rt.device),
                                          c, 1, dk, dv))
            at += c
        assert rel_l2(torch.cat(got), want) < 1e-5, cuts
        assert rel_l2(torch.cat(got)[-1], want[-1]) < 1e-4, cuts


@pytest.mark.parametrize("m,d,heads,act", [(1, 2304, 1, "sigmoid"), (7, 384, 1, "sigmoid"), (40, 1000, 1, "silu"), (300, 2048, 2, "sigmoid"), (3, 5000, 1, "silu"),
                                           (2, 9000, 1, "sigmoid"), (5, 257, 1, "sigmoid"), (4, 64, 1, "sigmoid")])
def test_long_rows_norm_and_gate(rt, m, d, heads, act):
    y, gain = rnd(m, d, seed=1), 1 + rnd(d, seed=2, scale=0.3)
    g, gw = acts(rt, rnd(m, d + 24, seed=3))
    got = rt.ops.head_norm_gate(y.to(DEV), gain.to(DEV), g[:, 8:8 + d], EPS, heads, act, rt.dtype)
    want = ref_ops.head_norm_gate(y, gain, gw[:, 8:8 + d], EPS, heads, act, torch.float32)
    assert rel_l2(got, want) < (1e-6 if rt.dtype == torch.float32 else 4e-3)


@pytest.mark.parametrize("m", [1, 2, 5, 8, 20, 64, 130, 600])
@pytest.mark.parametrize("n,k,columns", [(96, 64, 96), (200, 72, 100), (1000, 256, 1), (77, 50, 33), (4096, 512, 3000)])
def test_silu_on_the_first_columns(rt, m, n, k, columns):
    """A product whose first columns pass SiLU: every kernel that a number of rows leads to."""
    x, xw = acts(rt, rnd(m, k, seed=1))
    w, ww = acts(rt, rnd(n, k, seed=2, scale=0.3))
    got = rt.ops.linear_act(x, w, rt.dtype, "silu", columns=columns)
    y = xw @ ww.T
    want = torch.cat([plain.silu(y[:, :columns]), y[:, columns:]], dim=1)
    tol = 1e-6 if rt.dtype == torch.float32 else 4e-3
    assert rel_l2(got[:, :columns], want[:, :columns]) < tol and (columns == n or rel_l2(got[:, columns:], want[:, columns:]) < tol)


def test_norm_of_a_view(rt):
    x, xw = acts(rt, rnd(37, 300, seed=1))
    gain = 1 + rnd(100, seed=2, scale=0.3)
    got = rt.ops.rms_norm(x[:, 120:220], gain.to(DEV), EPS, rt.dtype, groups=2)
    want = ref_ops.rms_norm(xw[:, 120:220].contiguous(), gain, EPS, torch.float32, groups=2)
    assert rel_l2(got, want) < (1e-6 if rt.dtype == torch.float32 else 4e-3)


# ---- attention: a temperature of the query's position, a bias per distance, a gate per head --------------------------------------
def biased_part(rt, H, G, dim, vdim, reach, rows, coef=0.4, every=7, cap=8.0, scale=0.3, seed=0, edit=None):
    ref = ("attention", dict(hidden_size=WIDTH, num_heads=H, num_kv_heads=G, head_dim=dim, value_dim=vdim, query_scale=scale, softcap=cap,
                             position=("none", {}), output_gate="head", query_temperature=(coef, every), distance_bias="rel", bias_reach=reach,
                             bias_rows=rows, precise_weights=True, tensors=("q", "k", "v", "o", "g")))
    T = {"q": rnd(H * dim, WIDTH, seed=seed + 1, scale=0.25), "k": rnd(G * dim, WIDTH, seed=seed + 2, scale=0.25),
         "v": rnd(G * vdim, WIDTH, seed=seed + 3, scale=0.3), "o": rnd(WIDTH, H * vdim, seed=seed + 4, scale=0.2),
         "g": rnd(H, WIDTH, seed=seed + 5, scale=0.3), "rel": rnd(rows, H, seed=seed + 6)}
    if edit is not None:
        edit(T)
    part, W = bound(rt, "mixer", ref, T)
    return part, W, {"heads": H, "kv_heads": G, "dim": dim, "vdim": vdim, "scale": scale, "softcap": cap, "bias_max": reach,
                     "q_temp": {"coef": coef, "every": every}}


@pytest.mark.parametrize("page", [16, 64])
@pytest.mark.parametrize("H,G,dim,vdim,reach,rows,coef,every", [
    (4, 2, 16, 24, 40, 16, 0.4, 7), (3, 3, 24, 8, 9, 4, 0.5, 1), (2, 1, 32, 32, 300, 32, -0.1, 16), (1, 1, 12, 12, 5, 2, 0.3, 1000),
    (8, 2, 64, 64, 33, 64, 0.2, 64), (6, 3, 48, 96, 100, 32, 0.5, 10), (4, 4, 128, 64, 17, 32, 0.4, 32), (10, 1, 40, 72, 64, 8, 0.4, 5),
    (2, 2, 80, 96, 1000, 24, 0.4, 8), (32, 2, 16, 16, 50, 20, 0.3, 3)])
def test_biased_attention_part(rt, H, G, dim, vdim, reach, rows, coef, every, page):
    part, W, sizes = biased_part(rt, H, G, dim, vdim, reach, rows, coef, every)
    seqs, wide = sequences(rt, 9)
    got = run_mixers(rt, [(part, 0)], seqs, STEPS, page=page)
    for i in seqs:
        assert rel_l2(got[i][0], plain.biased_attention(wide[i], W, "", sizes, EPS)) < tolerance(rt), i


@pytest.mark.parametrize("dim,vdim", [(16, 24), (64, 64)])
@pytest.mark.parametrize("page,first", [(16, 24), (16, 31), (16, 32), (16, 33), (64, 64), (64, 6)])
def test_biases_that_pick_a_distance(rt, page, first, dim, vdim):
    """One row of the table is so large that a query's softmax picks the keys of that row's distances alone: a row one place
    off, or a distance taken one too long or too short, shows whole.  The row is the query's own key, a distance below half
    the rows, the first and the last of a logarithmic stretch, and all beyond the reach; in a prompt, a portion and single
    tokens, at page borders."""
    H, G, reach, rows = 4, 2, 37, 12
    n = max(first, 34) + 2 * page + 9
    x, xw = acts(rt, rnd(n, WIDTH, seed=3))
    steps = [{0: first}, {0: 2 * page + 1}] + [{0: 1}] * (n - first - 2 * page - 1)
    row_of = [plain.bucket(k, rows, reach) for k in range(n)]
    for row in (0, 3, 6, 8, rows - 1):
        def pick(T):
            T["rel"][row] += 40.0
        part, W, sizes = biased_part(rt, H, G, dim, vdim, reach, rows, seed=7, edit=pick)
        want = plain.biased_attention(xw, W, "", sizes, EPS)
        got = run_mixers(rt, [(part, 0)], {0: x}, steps, page=page)[0][0].double().cpu()
        assert rows_differ(got, want) < (1e-4 if rt.dtype == torch.float32 else 8e-2), row
        # and the outputs do rest on which keys those are
        moved = dict(W, rel=torch.roll(W["rel"], 1, dims=0))
        assert rows_differ(plain.biased_attention(xw, moved, "", sizes, EPS), want) > 0.3
        other = plain.biased_attention(xw, W, "", dict(sizes, bias_max=reach + 6), EPS)
        assert rows_differ(other, want) > 0.3 or row in (0, 3, 6), (row, row_of)


@pytest.mark.parametrize("page,first", [(16, 64), (16, 63), (16, 65), (64, 129)])
def test_one_far_key_stands_out(rt, page, first):
    """One early key is made to stand out for every later query, beyond the reach of the biases: its score is capped and
    multiplied by the temperature of the query's position before the cap."""
    H, G, dim, vdim = 4, 2, 16, 24

    def mark(T):                                         # a head's last element: keys read column 5 of the input, queries column 7
        for name, heads, col in (("k", G, 5), ("q", H, 7)):
            w = T[name].view(heads, dim, WIDTH)
            w[:, dim - 1, :] = 0.0
            w[:, dim - 1, col] = 1.0
    part, W, sizes = biased_part(rt, H, G, dim, vdim, 20, 8, coef=0.6, every=30, cap=12.0, scale=0.25, seed=7, edit=mark)
    n = first + 2 * page + 9
    x = rnd(n, WIDTH, seed=3) * 0.3
    x[:, 5] = 0.0
    x[3, 5] = 8.0                                        # the marked key
    x[:, 7] = 4.0                                        # every query meets it with a score of about 8 before the temperature
    x_dev, xw = acts(rt, x)
    want = plain.biased_attention(xw, W, "", sizes, EPS)
    steps = [{0: first}, {0: 2 * page + 1}] + [{0: 1}] * (n - first - 2 * page - 1)
    got = run_mixers(rt, [(part, 0)], {0: x_dev}, steps, page=page)[0][0].double().cpu()
    assert rows_differ(got, want) < (1e-4 if rt.dtype == torch.float32 else 8e-2)
    lost = xw.clone()
    lost[3, 5] = 0.0
    assert rows_differ(plain.biased_attention(lost, W, "", sizes, EPS)[first:], want[first:]) > 0.3


@pytest.mark.parametrize("at", [28, 29, 30])
def test_temperature_changes_at_its_position(rt, at):
    """With a coefficient so large that the temperature decides between a head's keys, the change at position every - 1 shows
    from there on and not one position earlier, whatever the step that brings it."""
    H, G, dim, vdim, every = 2, 1, 16, 16, 30
    part, W, sizes = biased_part(rt, H, G, dim, vdim, 20, 8, coef=6.0, every=every, cap=60.0, scale=1.0, seed=11)
    n = 70
    x, xw = acts(rt, rnd(n, WIDTH, seed=5) * 0.4)
    want = plain.biased_attention(xw, W, "", sizes, EPS)
    for steps in ([{0: n}], [{0: at}, {0: n - at}], [{0: at}] + [{0: 1}] * (n - at), [{0: at - 2}, {0: 2}, {0: 2}, {0: n - at - 2}]):
        got = run_mixers(rt, [(part, 0)], {0: x}, steps)[0][0].double().cpu()
        assert rows_differ(got, want) < (2e-4 if rt.dtype == torch.float32 else 1e-1)
    late = plain.biased_attention(xw, W, "", dict(sizes, q_temp={"coef": 6.0, "every": every + 1}), EPS)
    assert torch.equal(late[:every - 1], want[:every - 1]) and rows_differ(late[every - 1:every], want[every - 1:every]) > 0.05


def test_matrix_core_kernels_over_many_tiles():
    """Sequences long enough for every wave of a block to take several tiles of keys and for a decode step's keys to be cut
    in slices: the matrix-core kernels against the plain kernels on the same rows, biases near and far."""
    from trapetum_amd.engine.runtime import Runtime
    rt = Runtime(dtype="bfloat16", device=DEV)
    for H, G, dim, reach, rows in ((8, 4, 128, 128, 32), (4, 2, 64, 700, 64), (4, 1, 80, 33, 16), (12, 2, 32, 64, 32)):
        part, W, sizes = biased_part(rt, H, G, dim, dim, reach, rows, coef=0.3, every=100, scale=0.5)
        seqs, _ = sequences(rt, 59, lens={0: 1500, 1: 180})
        steps = [{0: 700, 1: 100}, {0: 1, 1: 1}, {0: 150, 1: 2}, {0: 500}] + [{0: 1, 1: 1}] * 49 + [{0: 100, 1: 28}]
        got = run_mixers(rt, [(part, 0)], seqs, steps, page=64)
        rt.ops.force_plain_attention = True
        try:
            slow = run_mixers(rt, [(part, 0)], seqs, steps, page=64)
        finally:
            rt.ops.force_plain_attention = False
        for i in seqs:
            assert rel_l2(got[i][0], slow[i][0]) < 6e-3, (H, G, dim, reach, i)


# ---- attention through a latent: a sink per head, a gate per element, one input product ------------------------------------------
def latent_part(rt, H, dim, rot_dim, vdim, rank, q_rank, scale=0.3, base=200.0, seed=0, edit=None, joint=True):
    ref = ("latent_attention", dict(hidden_size=WIDTH, num_heads=H, nope_dim=dim, rope_dim=rot_dim, value_dim=vdim, latent_rank=rank, scale=scale,
                                    latent_eps=EPS, position=("rope", {"rotary_dim": rot_dim, "theta": base, "pairing": "neighbours"}),
                                    query_rank=q_rank, output_gate="g", gate_per="element", sink="sink", joint_input=joint, precise_weights=True))
    T = {"dq": rnd(q_rank, WIDTH, seed=seed + 1, scale=0.25), "dq.norm": 1 + rnd(q_rank, seed=seed + 2, scale=0.3),
         "uq": rnd(H * (dim + rot_dim), q_rank, seed=seed + 3, scale=0.25), "dkv": rnd(rank + rot_dim, WIDTH, seed=seed + 4, scale=0.25),
         "dkv.norm": 1 + rnd(rank, seed=seed + 5, scale=0.3), "uk": rnd(H * dim, rank, seed=seed + 6, scale=0.25),
         "uv": rnd(H * vdim, rank, seed=seed + 7, scale=0.25), "sink": rnd(H, seed=seed + 8, scale=2.0),
         "g": rnd(H * vdim, WIDTH, seed=seed + 9, scale=0.3), "o": rnd(WIDTH, H * vdim, seed=seed + 10, scale=0.2)}
    if edit is not None:
        edit(T)
    part, W = bound(rt, "mixer", ref, T)
    return part, W, {"heads": H, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "q_rank": q_rank, "scale": scale,
                     "rot": {"base": base, "dims": rot_dim}}


@pytest.mark.parametrize("joint", [True, False])
@pytest.mark.parametrize("H,dim,rot_dim,vdim,rank,q_rank", [
    (4, 16, 8, 24, 24, 20), (3, 24, 16, 16, 32, 40), (1, 10, 2, 12, 10, 6), (8, 32, 32, 64, 64, 48), (16, 64, 16, 32, 96, 72), (6, 40, 8, 20, 56, 33),
    (2, 128, 64, 128, 192, 100), (12, 16, 16, 16, 48, 16)])
def test_sink_latent_part(rt, H, dim, rot_dim, vdim, rank, q_rank, joint):
    part, W, sizes = latent_part(rt, H, dim, rot_dim, vdim, rank, q_rank, joint=joint)
    seqs, wide = sequences(rt, 19)
    got = run_mixers(rt, [(part, 0)], seqs, STEPS)
    for i in seqs:
        # in bfloat16 a row passes several roundings more than a plain attention's (the queries' latent, the queries, the gate)
        assert rel_l2(got[i][0], plain.latent_attention(wide[i], W, "", sizes, EPS)) < tolerance(rt) * (1 if rt.dtype == torch.float32 else 1.5), i


@pytest.mark.parametrize("page,first", [(16, 20), (16, 33), (64, 65)])
def test_sink_takes_its_share(rt, page, first):
    """One head's sink above every score, one's far below, one's about as large: lost, counted twice, scaled or multiplied by
    a value it would show."""
    def set_sinks(T):
        T["sink"][:] = torch.tensor([8.0, -30.0, 2.5])
    part, W, sizes = latent_part(rt, 3, 16, 8, 12, 24, 20, seed=30, edit=set_sinks)
    n = first + 2 * page + 9
    x, xw = acts(rt, rnd(n, WIDTH, seed=3))
    want = plain.latent_attention(xw, W, "", sizes, EPS)
    steps = [{0: first}, {0: 2 * page + 1}] + [{0: 1}] * (n - first - 2 * page - 1)
    got = run_mixers(rt, [(part, 0)], {0: x}, steps, page=page)[0][0]
    assert rel_l2(got, want) < tolerance(rt) * (1 if rt.dtype == torch.float32 else 1.5)
    for other in (W["sink"] - 1e9, W["sink"] * sizes["scale"], W["sink"] + 0.6931):
        assert rel_l2(plain.latent_attention(xw, dict(W, sink=other), "", sizes, EPS), want) > 0.05


def test_latent_far_key_at_page_borders(rt):
    """One early row is made to stand out for every later query through the part without a position."""
    H, dim, rot_dim, vdim, rank, q_rank = 2, 8, 4, 8, 12, 12
    part, W, sizes = latent_part(rt, H, dim, rot_dim, vdim, rank, q_rank, scale=40.0, seed=50)
    for first in (31, 32, 33, 64):
        n = first + 40
        x, xw = acts(rt, rnd(n, WIDTH, seed=7))
        want = plain.latent_attention(xw, W, "", sizes, EPS)
        got = run_mixers(rt, [(part, 0)], {0: x}, [{0: first}, {0: 20}] + [{0: 1}] * 20)[0][0]
        assert rel_l2(got, want) < (1e-3 if rt.dtype == torch.float32 else 0.25), first      # sharp scores carry a rounded row's error into the choice


# ---- the stream: constants on what is added, made anew before a pass -----------------------------------------------------------------
@pytest.mark.parametrize("m,d", [(1, 50), (3, 64), (8, 2304), (200, 96), (300, 2304), (5, 3584), (150, 1001)])
def test_stream_with_constants_and_terms(rt, m, d):
    ops = rt.ops
    gain = (1 + rnd(d, seed=1, scale=0.3)).to(DEV)
    stream0, origin, slices, rows = rnd(m, d, seed=2), rnd(m, d, seed=3), rnd(3, m, d, seed=5), rnd(m, d, seed=6).to(rt.dtype)
    dev = lambda t: None if t is None else (ops.SplitRows(t.to(DEV)) if t.dim() == 3 else t.to(DEV))
    total = lambda t: 0 if t is None else (t.double().sum(0) if t.dim() == 3 else t.double())
    for a, b in ((rows, None), (rows, slices), (slices, rows)):
        for fresh in (False, True):
            stream = stream0.to(DEV)
            out = ops.join_rms_norm(stream, dev(a), dev(b), gain, EPS, rt.dtype, wa=0.3, wb=-1.7, fresh=fresh)
            want = (0 if fresh else stream0.double()) + 0.3 * total(a) - 1.7 * total(b)
            assert rel_l2(stream, want) < 1e-6
            assert rel_l2(out, plain.over_rms(want, EPS) * gain.double().cpu()) < (1e-6 if rt.dtype == torch.float32 else 4e-3)
        for terms in (1, 2):
            stream = stream0.to(DEV)
            got = ops.join_rms_norm(stream, dev(a), dev(b), None, 0.0, rt.dtype, origin=origin.to(DEV), wa=0.3, wb=-1.7, stack=terms)
            want = stream0.double() + 0.3 * total(a) - 1.7 * total(b)
            if rt.dtype == torch.float32:
                assert got.shape == (m, 2 * d) and rel_l2(got, torch.cat([want, origin.double()], dim=1)) < 1e-6
                continue
            assert got.shape == (m, (2 + terms) * d)
            g = got.double().cpu()
            assert rel_l2(g[:, :d] + g[:, d:2 * d], want) < 1e-5                # two terms: 16 bits
            assert rel_l2(g[:, 2 * d:3 * d] + (g[:, 3 * d:] if terms == 2 else 0), origin.double()) < (1e-5 if terms == 2 else 4e-3)
    stream = stream0.to(DEV)
    assert ops.join_rms_norm(stream, None, None, None, 0.0, rt.dtype, origin=origin.to(DEV), stack=1).shape[0] == m and torch.equal(stream.cpu(), stream0)


@pytest.mark.parametrize("m,d", [(1, 64), (9, 96), (130, 72)])
def test_stream_made_anew(rt, m, d):
    class Ctx:
        ops, dtype = rt.ops, rt.dtype
    part, W = bound(rt, "stream_add", ("stream_mix", dict(size=d)), {"in": rnd(d, 2 * d, seed=1, scale=0.2)})
    stream, start, rows = rnd(m, d, seed=2), rnd(m, d, seed=3).to(torch.bfloat16).float(), rnd(m, d, seed=4).to(rt.dtype)
    Ctx.origin = start.to(DEV)
    got, gain = stream.to(DEV), 1 + rnd(d, seed=5, scale=0.3)
    normed = part.forward(Ctx, got, rows.to(DEV), None, 0.4, 1.0, gain.to(DEV), EPS, rt.dtype)
    want = torch.cat([stream.double() + 0.4 * rows.double(), start.double()], dim=1) @ W["in"].T
    assert rel_l2(got, want) < (2e-6 if rt.dtype == torch.float32 else 2e-5)       # not rounded to bfloat16 on the way
    assert rel_l2(normed, plain.over_rms(want, EPS) * gain.double()) < (2e-6 if rt.dtype == torch.float32 else 4e-3)


# ---- the model ---------------------------------------------------------------------------------------------------------------------
def loaded(tmp_path_factory, which, dtype, tol):
    from .gpu_engine import load_gpu_model
    folder = kt.make_folder(tmp_path_factory.mktemp("k"), which)
    model, cfg = load_gpu_model(folder, dtype)
    pcfg, pw = plain.read_folder(folder)
    return model, cfg, pcfg, pw, tol


@pytest.fixture(scope="module", params=[(w, d) for d in ("float32", "bfloat16") for w in "PQRT"], ids=lambda p: "-".join(p))
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


def test_sharp_scores(sharp):
    mc.sharp_scores_far_keys(sharp, n=110)


def test_layers_one_by_one(m):
    """The residual stream after every run of a layer, a looped layer's passes included (where the stream is made anew before
    the next run, the kernels that close the layer have done so by then)."""
    model, cfg, pcfg, pw, tol = m
    toks = random_tokens(41, cfg.vocab_size, 5)
    want = []
    plain.forward(pcfg, pw, toks, layers_out=want)
    start = pw["embed"][torch.tensor(toks)]
    for i, (_, enters) in enumerate(plain.running_order(pcfg)[1:]):
        if enters:
            want[i] = torch.cat([want[i], start], dim=1) @ pw["loop.in"].T
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
@pytest.mark.parametrize("case", range(10))
def test_random_configuration(case, dtype, tmp_path):
    """A configuration drawn at random: a prompt whole, then in two portions and single tokens."""
    from .gpu_engine import load_gpu_model
    rng = random.Random(1500 + case)
    cfg = kt.draw(rng)
    folder = str(tmp_path)
    write_model_folder(KaderaxConfig.from_dict(cfg), folder, seed=case, sigma=0.1, sigma_norm=0.2)
    model, c = load_gpu_model(folder, dtype)
    pcfg, pw = plain.read_folder(folder)
    toks = random_tokens(90, c.vocab_size, case)
    ref = plain.forward(pcfg, pw, toks)
    cache = model.new_cache(max_tokens=192, page_size=16)
    s = cache.acquire()
    got = [model.step(cache, [s], toks[:20], counts=[20], want=list(range(20))),
           model.step(cache, [s], toks[20:79], counts=[59], want=list(range(59)))]
    got += [model.step(cache, [s], [t]) for t in toks[79:]]
    mc.rows_close(torch.cat(got), ref, 5e-5 if dtype == "float32" else mc.Rounded(6e-2), cfg)     # (ten runs of layers of width 24: roundings add up)


@pytest.mark.parametrize("which,dtype", [("P", "float32"), ("Q", "float32"), ("P", "bfloat16"), ("R", "bfloat16")])
def test_greedy_generation_through_the_entry_point(which, dtype, tmp_path):
    from trapetum_amd import load_model
    folder = kt.make_folder(tmp_path, which)
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
    """A decode step replayed from its graph, again and again with eager work between the replays, gives the logits of the
    eager step of the same launch geometry bit for bit."""
    from trapetum_amd.engine.graphs import GraphedDecode, length_bound
    from .gpu_engine import load_gpu_model
    model, cfg = load_gpu_model(kt.make_folder(tmp_path, "P"), "bfloat16")
    caches = [model.new_cache(max_tokens=512, page_size=64, max_slots=4) for _ in range(2)]
    toks = [random_tokens(40, cfg.vocab_size, 7 + i) for i in range(4)]
    slots = [[c.acquire() for _ in toks] for c in caches]
    for c, s in zip(caches, slots):
        model.step(c, s, sum((t[:9] for t in toks), []), counts=[9] * 4)
    graphs = GraphedDecode(model, caches[1])
    for j in range(9, 40):
        step = [t[j] for t in toks]
        counts, starts, want, tok = model.prepare(caches[0], slots[0], step)
        eager = model.run(StepContext(model.rt, caches[0], slots[0], counts, starts, want, length_bound=length_bound(j + 1, caches[0].max_context)), tok)
        torch.cuda.synchronize()
        assert bool((graphs.step(slots[1], step) == eager).all()), j


def test_command_line_and_trace_runner(tmp_path):
    """`python -m trapetum_amd random | run` and bin/trace_run on a Kaderax folder: the model class comes from config.json,
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
    cfg, init = kt.CONFIGS["P"]
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
