"""The Gemepel design on the GPU against the plain implementation (tests/plain/gemepel_plain.py): the new kernels one by
one, then whole models under every way of cutting requests into steps (whole prompts, the last tokens one by one, from the
first token on, batches of unequal requests whose slots, pages and states are used again), keys far away under a sharp
query, a recurrent state that must carry a token over hundreds of steps, the previous token across a step's edge, choices
of experts at a group's edge, greedy generation through generate() and the command line, the trace runner, and
configurations drawn at random."""
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import gemepel_configs as GC
import helpers
import schedules
from plain import gemepel_plain as P
from plain import reference_model as R

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"
F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16]


def gen(seed):
    return torch.Generator().manual_seed(seed)


def randn(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=gen(seed), dtype=torch.float32) * scale


f32 = lambda t: t.to(torch.float32).to(DEV).contiguous()
i32 = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)


def close(got, want, dtype, f32_tol=2e-6, bf16_tol=1e-2):
    tol = f32_tol if dtype == torch.float32 else bf16_tol
    got = got.float().cpu().to(F64)
    assert torch.allclose(got, want, rtol=tol, atol=tol), float((got - want).abs().max())


# ------------------------------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R_,D", [(1, 1), (3, 7), (5, 80), (2, 1024), (3, 1030), (9, 4096), (2, 5000), (1, 17000)])
def test_layer_norm_kernels(R_, D, dtype):
    """The norm alone (with and without chosen rows), the norm of the weighted sum, and the same followed by the norm that
    reads the stream next.  The rows' mean is far from zero."""
    from yalm_amd.ops import kernels
    x, y = randn(R_, D, seed=1, scale=2.0) + 30.0, randn(R_, D, seed=2)
    w, b, w2, b2 = (randn(D, seed=s) + (1.0 if s % 2 else 0.0) for s in (3, 4, 5, 6))
    d = lambda t: t.to(F64)
    tol = dict(f32_tol=2e-5)                       # float32's share of a mean of 30
    out = torch.full((R_, D), float("nan"), dtype=dtype, device=DEV)
    kernels.layer_norm(x.to(DEV), w.to(DEV), b.to(DEV), 1e-5, out)
    close(out, P.layer_norm(d(x), d(w), d(b), 1e-5), dtype, **tol)
    rows = [R_ - 1, 0]
    out = torch.full((2, D), float("nan"), dtype=dtype, device=DEV)
    kernels.layer_norm(x.to(DEV), w.to(DEV), b.to(DEV), 1e-5, out, row_index=i32(rows))
    close(out, P.layer_norm(d(x)[rows], d(w), d(b), 1e-5), dtype, **tol)
    want = P.layer_norm(1.7 * d(x) + d(y), d(w), d(b), 1e-5)
    h = torch.full((R_, D), float("nan"), dtype=dtype, device=DEV)
    for h_out in (None, h):
        xd = x.clone().to(DEV)
        kernels.layer_norm_sum(y.to(DEV), w.to(DEV), b.to(DEV), 1e-5, 1.7, xd, h_out)
        close(xd, want, torch.float32, f32_tol=4e-5)
    close(h, want, dtype, f32_tol=4e-5, bf16_tol=2e-2)
    xd = x.clone().to(DEV)
    kernels.layer_norm_sum(y.to(DEV), w.to(DEV), b.to(DEV), 1e-5, 1.7, xd, h, next_norm=(w2.to(DEV), b2.to(DEV), 3e-6))
    close(xd, want, torch.float32, f32_tol=4e-5)
    if D > 1:
        close(h, P.layer_norm(want, d(w2), d(b2), 3e-6), dtype, f32_tol=2e-4, bf16_tol=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,V,bigram", [(5, 11, (7, 3, 2)), (300, 50, (1, 5, 9)), (1100, 40, (487, 101, 13)), (64, 90000, (65521, 1 << 20, 999983))])
def test_embedding_of_token_pairs(D, V, bigram, dtype):
    """Two texts in pieces of several tokens and of one, beside a padding row; products of token and multiplier beyond 32
    bits; the previous token is kept per slot."""
    from yalm_amd.ops import kernels
    emb = {"scale": 0.37, "bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    w = {"embed": randn(V, D, seed=1).to(dtype), "bigram": randn(bigram[0] + 1, D, seed=2).to(dtype)}
    g = np.random.default_rng(3)
    texts = [g.integers(0, V, size=12).tolist(), g.integers(0, V, size=9).tolist()]
    want = [P.embed(t, emb, w, {}) for t in texts]
    table, pairs = w["embed"].to(DEV), w["bigram"].to(DEV)
    last = torch.full((4, 1), 123, dtype=torch.int32, device=DEV)
    slots, at = [3, 1], [0, 0]
    for lens in ([4, 1], [1, 0], [3, 5], [1, 1], [1, 1], [2, 1]):
        toks, seq, pos, cu, ss = [], [], [], [0], []
        for b in (0, 1):
            if lens[b]:
                toks += texts[b][at[b]:at[b] + lens[b]]
                seq += [len(ss)] * lens[b]
                pos += list(range(at[b], at[b] + lens[b]))
                cu.append(len(toks)); ss.append(slots[b])
        toks.append(-1); seq.append(len(ss)); pos.append(0); cu.append(len(toks)); ss.append(-1)
        out = torch.full((len(toks), D), float("nan"), dtype=torch.float32, device=DEV)
        kernels.embed_pairs(table, pairs, i32(toks), i32(seq), i32(pos), i32(cu), i32(ss), last, bigram[1], bigram[2], 0.37, out)
        row = 0
        for b in (0, 1):
            assert torch.allclose(out[row:row + lens[b]].cpu().to(F64), want[b][at[b]:at[b] + lens[b]], rtol=1e-6, atol=1e-6)
            row += lens[b]
            at[b] += lens[b]
            if lens[b]:
                assert int(last[slots[b]]) == texts[b][at[b] - 1]
        assert float(out[row:].abs().max()) == 0.0
    assert at == [12, 9] and int(last[0]) == 123 and int(last[2]) == 123


@pytest.mark.parametrize("E,top,groups,keep,scale", [(14, 5, 2, 1, 1.8), (12, 3, 4, 2, 1.0), (1, 1, 1, 1, 0.5), (6, 2, 6, 3, 1.5), (6, 6, 1, 1, 1.0),
                                                     (64, 8, 8, 4, 2.5), (256, 8, 8, 4, 2.5), (300, 5, 100, 2, 1.0), (1024, 9, 2, 2, 1.0)])
def test_choice_inside_groups(E, top, groups, keep, scale):
    """Corrections from strongly negative to strongly positive (all choice scores negative, all positive, mixed), so that
    a mask of zeros or weights with the correction in them would show."""
    from yalm_amd.ops import kernels
    T = 50
    for shift, seed in ((-3.0, 1), (0.0, 2), (2.0, 3)):
        z, corr = randn(T, E, seed=seed, scale=1.5), randn(E, seed=seed + 10, scale=0.6) + shift
        router = {"experts": E, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}}
        w = {"router": torch.eye(E, dtype=F64), "correction": corr}
        chosen, weight = P.route(z.to(F64), router, w, "")
        sure = P.route_margin(z.to(F64), router, w, "") > 1e-5
        ids = torch.full((T, top), -7, dtype=torch.int32, device=DEV)
        wts = torch.full((T, top), float("nan"), dtype=torch.float32, device=DEV)
        kernels.moe_select_groups(z.to(DEV), corr.to(DEV), ids, wts, groups, keep, scale)
        got_ids, got_w = ids.cpu().long(), wts.cpu().to(F64)
        assert sure.float().mean() > 0.8
        # the order among the chosen may differ where two choice scores are within rounding: compare by expert
        dense = lambda i, v: torch.zeros(T, E, dtype=F64).scatter_(1, i, v)
        a, b = dense(got_ids, got_w)[sure], dense(chosen, weight)[sure]
        assert torch.allclose(a, b, rtol=1e-5, atol=1e-6), float((a - b).abs().max())
        assert torch.allclose(got_w.sum(-1), torch.full((T,), scale, dtype=F64), rtol=1e-5)


def test_choice_among_equals_and_without_correction():
    from yalm_amd.ops import kernels
    ids, wts = torch.empty(1, 2, dtype=torch.int32, device=DEV), torch.empty(1, 2, dtype=torch.float32, device=DEV)
    kernels.moe_select_groups(torch.zeros(1, 8, device=DEV), None, ids, wts, 4, 2, 1.0)
    assert ids.tolist() == [[0, 1]] and torch.allclose(wts.cpu(), torch.tensor([[0.5, 0.5]]))
    kernels.moe_select_groups(torch.full((1, 8), -200.0, device=DEV), None, ids, wts, 4, 2, 1.0)      # scores that vanish: no division by zero
    assert bool(torch.isfinite(wts).all())
    with pytest.raises(ValueError):
        kernels.moe_select_groups(torch.zeros(1, 8, device=DEV), None, ids, wts, 8, 1, 1.0)           # two of one group of one


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,D,F,E,top", [(1, 8, 8, 3, 1), (5, 50, 11, 4, 2), (7, 80, 96, 6, 6), (33, 64, 40, 5, 2), (300, 192, 64, 16, 4), (90, 320, 264, 3, 3)])
def test_squared_relu_experts(T, D, F, E, top, dtype):
    """Two-matrix experts pair by pair, and grouped by expert on the matrix cores where the sizes allow it."""
    from yalm_amd.ops import kernels
    h = randn(T, D, seed=1).to(dtype)
    wu, wd = randn(E, F, D, seed=2, scale=D ** -0.5).to(dtype), randn(E, D, F, seed=3, scale=F ** -0.5).to(dtype)
    g = gen(4)
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)])
    wts = torch.rand(T, top, generator=g)
    mids = torch.relu(torch.einsum("td,tkfd->tkf", h.to(F64), wu.to(F64)[ids])) ** 2
    want = torch.einsum("tk,tkf,tkdf->td", wts.to(F64), mids, wd.to(F64)[ids])
    hd, wud, wdd, idd, wtd = h.to(DEV), wu.to(DEV), wd.to(DEV), i32(ids), wts.to(DEV)
    mid = torch.full((T * top, F), float("nan"), dtype=dtype, device=DEV)
    out = torch.full((T, D), float("nan"), dtype=torch.float32, device=DEV)
    kernels.moe_pair_gate_up(hd, None, wud, idd, 0.0, 1.0, mid)
    close(mid, mids.reshape(T * top, F), dtype, f32_tol=1e-5)
    kernels.moe_pair_down(mid, wdd, idd, wtd, out)
    close(out, want, dtype, f32_tol=2e-5, bf16_tol=2e-2)
    if kernels.can_moe_grouped(D, F, dtype, T * top, E):
        held = {}
        scratch = lambda n, s, t: held.setdefault(n, torch.empty(s, dtype=t, device=DEV))
        got = torch.full((T, D), float("nan"), dtype=torch.float32, device=DEV)
        kernels.moe_grouped(hd, None, wud, wdd, idd, wtd, 0.0, 1.0, scratch, got)
        close(got, want, dtype, bf16_tol=2e-2)
        kernels.moe_grouped(hd, None, wud, wdd, idd, wtd, 0.0, 1.0, scratch, got, accumulate=True)
        close(got, 2 * want, dtype, bf16_tol=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R_,n,row", [(1, 1, 1), (5, 20, 68), (3, 80, 80), (70, 1536, 2112), (9, 7, 30)])
def test_latent_norm(R_, n, row, dtype):
    from yalm_amd.ops import kernels
    x, w = randn(R_, row, seed=1, scale=3.0), (randn(n, seed=2) + 1.0).to(dtype)
    out = torch.full((R_, n), float("nan"), dtype=dtype, device=DEV)
    kernels.latent_norm(x.to(DEV), n, w.to(DEV), 1e-5, out)
    close(out, P.rms_norm(x.to(F64)[:, :n], w.to(F64), 1e-5), dtype)


@pytest.mark.parametrize("n_first", [3, 40])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,rank,tau", [(1, 4, 4, 1, 1.0), (4, 32, 64, 16, 16.0), (3, 5, 9, 3, 0.5), (2, 64, 40, 20, 16.0), (1, 128, 70, 16, 8.0),
                                             (1, 200, 33, 64, 16.0), (2, 16, 200, 7, 4.0), (5, 36, 31, 256, 2.0), (2, 256, 16, 256, 16.0), (3, 44, 60, 17, 12.0)])
def test_gla_kernel(H, d, dv, rank, tau, dtype, n_first):
    """Two sequences and a padding row: first pieces as a step of prompts, then single tokens, against the plain recurrence
    over the whole texts; the state left behind against the plain one (it is kept column by column)."""
    from yalm_amd.ops import kernels
    lens = [n_first + 6, 7]
    g = gen(H * 100 + d)
    rn = lambda *s, sc=1.0: (torch.randn(*s, generator=g, dtype=F64) * sc).float().to(F64)
    Hd, Hv = H * d, H * dv
    w2, bias, w_norm = rn(Hd, rank, sc=2.0 * rank ** -0.5), rn(Hd), 1 + rn(dv, sc=0.2)
    projs = [rn(n, 2 * Hd + 2 * Hv + rank, sc=1.5) for n in lens]
    want, S_want = [], []
    for pr in projs:
        n = pr.shape[0]
        q, k = (pr[:, i * Hd:(i + 1) * Hd].reshape(n, H, d) for i in (0, 1))
        v, gate = pr[:, 2 * Hd:2 * Hd + Hv].reshape(n, H, dv), pr[:, 2 * Hd + Hv:2 * Hd + 2 * Hv]
        m = {"heads": H, "dim": d, "tau": tau}
        a = P.decays(pr[:, 2 * Hd + 2 * Hv:], m, {"a1": torch.eye(rank), "a2": w2, "a2.b": bias}, "")
        outs, states = zip(*[P.gla_scan(q[:, i] * d ** -0.5, k[:, i], v[:, i], a[:, i], torch.zeros(d, dv, dtype=F64)) for i in range(H)])
        want.append(P.rms_norm(torch.stack(outs, dim=1), w_norm, 1e-5).reshape(n, Hv) * P.silu(gate))
        S_want.append(torch.stack(states))
    state = torch.zeros(4, kernels.gla_state_elements(H, d, dv), dtype=torch.float32, device=DEV)
    state[1].fill_(float("nan"))
    slots = [2, 0]
    w2p = torch.zeros(Hd, kernels.gla_padded_rank(rank), dtype=F64)
    w2p[:, :rank] = w2

    def step(rows, cu, seq_slot):
        proj = f32(torch.cat(rows))
        T = proj.shape[0]
        raw = torch.full((T, Hv), float("nan"), dtype=torch.float32, device=DEV)
        out = torch.full((T, Hv), float("nan"), dtype=dtype, device=DEV)
        kernels.gla(proj, f32(w2p), f32(bias), f32(w_norm), state, raw, i32(cu), i32(seq_slot), out, H, d, dv, rank, d ** -0.5, tau, 1e-5)
        return out.float().cpu().to(F64)

    first = [n_first, 1]
    got = [[], []]
    out = step([projs[0][:first[0]], projs[1][:first[1]]], [0, first[0], first[0] + first[1]], slots)
    got[0].append(out[:first[0]]); got[1].append(out[first[0]:])
    for t in range(lens[0] - first[0]):
        rows, ss = [projs[0][first[0] + t:first[0] + t + 1], torch.zeros(1, projs[0].shape[1], dtype=F64)], [slots[0], -1]
        more = first[1] + t < lens[1]
        if more:
            rows.append(projs[1][first[1] + t:first[1] + t + 1]); ss.append(slots[1])
        out = step(rows, list(range(len(rows) + 1)), ss)
        assert float(out[1].abs().max()) == 0.0      # the padding row
        got[0].append(out[0:1])
        if more:
            got[1].append(out[2:3])
    tol = 3e-5 if dtype == torch.float32 else 2e-2
    for b in range(2):
        assert torch.allclose(torch.cat(got[b]), want[b], rtol=tol, atol=tol), (b, float((torch.cat(got[b]) - want[b]).abs().max()))
        S = state[slots[b]].cpu().to(F64).reshape(H, dv, d).transpose(1, 2)
        assert torch.allclose(S, S_want[b], rtol=1e-5, atol=1e-5)
    assert bool(torch.isnan(state[1]).all()) and float(state[3].abs().sum()) == 0.0


@pytest.mark.parametrize("tau,shift", [(16.0, 0.0), (1.0, 1.0), (16.0, 6.0), (0.5, -4.0)])
@pytest.mark.parametrize("H,d,dv,rank", [(1, 4, 4, 1), (3, 5, 9, 3), (4, 32, 64, 16), (2, 33, 17, 20), (2, 64, 40, 16), (1, 128, 128, 16), (3, 100, 200, 7),
                                         (2, 128, 70, 96)])
def test_gla_prompts_tile_by_tile(H, d, dv, rank, tau, shift):
    """Prompts of unequal lengths (one token to several tiles, one that ends a tile and one just behind it), from states that
    are not zero: read-outs and states as the recurrence gives them.  Decays from nearly none to e^-15 a token, so that
    their products over a tile run far below float32's range."""
    from yalm_amd.ops import kernels
    lens = [1, 64, 65, 200, 17]
    g = gen(H * 100 + d)
    rn = lambda *s, sc=1.0: (torch.randn(*s, generator=g, dtype=F64) * sc).float().to(F64)
    Hd, Hv = H * d, H * dv
    w2, bias, w_norm = rn(Hd, rank, sc=2.0 * rank ** -0.5), rn(Hd) + shift, 1 + rn(dv, sc=0.2)
    projs = [rn(n, 2 * Hd + 2 * Hv + rank, sc=1.5) for n in lens]
    slots = [2, 0, 5, 3, 1]
    S0 = rn(6, H, d, dv, sc=0.3)
    w2p = torch.zeros(Hd, kernels.gla_padded_rank(rank), dtype=F64)
    w2p[:, :rank] = w2
    state = f32(S0.transpose(2, 3).reshape(6, -1))
    cu, tile0 = np.concatenate([[0], np.cumsum(lens)]), np.concatenate([[0], np.cumsum([(n + 63) // 64 for n in lens])])
    T = int(cu[-1])
    raw = torch.full((T, Hv), float("nan"), dtype=torch.float32, device=DEV)
    out = torch.full((T, Hv), float("nan"), dtype=torch.float32, device=DEV)
    scratch = lambda name, shape, dt: torch.full(shape, float("nan"), dtype=dt, device=DEV)
    kernels.gla_tiles(f32(torch.cat(projs)), f32(w2p), f32(bias), f32(w_norm), state, raw, i32(cu), i32(slots), i32(tile0), int(tile0[-1]),
                      out, H, d, dv, rank, d ** -0.5, tau, 1e-5, scratch)
    for b, pr in enumerate(projs):
        n = pr.shape[0]
        q, k = (pr[:, i * Hd:(i + 1) * Hd].reshape(n, H, d) for i in (0, 1))
        v, gate = pr[:, 2 * Hd:2 * Hd + Hv].reshape(n, H, dv), pr[:, 2 * Hd + Hv:2 * Hd + 2 * Hv]
        a = P.decays(pr[:, 2 * Hd + 2 * Hv:], {"heads": H, "dim": d, "tau": tau}, {"a1": torch.eye(rank), "a2": w2, "a2.b": bias}, "")
        outs, states = zip(*[P.gla_scan(q[:, i] * d ** -0.5, k[:, i], v[:, i], a[:, i], S0[slots[b], i]) for i in range(H)])
        o = torch.stack(outs, dim=1)
        got = raw[cu[b]:cu[b + 1]].cpu().to(F64).reshape(n, H, dv)
        assert float((got - o).abs().max()) <= 3e-5 * max(1.0, float(o.abs().max())), (b, float((got - o).abs().max()))
        S = state[slots[b]].cpu().to(F64).reshape(H, dv, d).transpose(1, 2)
        assert float((S - torch.stack(states)).abs().max()) <= 2e-5 * max(1.0, float(S.abs().max()))
        want = P.rms_norm(o, w_norm, 1e-5).reshape(n, Hv) * P.silu(gate)
        err = (out[cu[b]:cu[b + 1]].cpu().to(F64) - want).abs()
        assert float(err.max()) <= 2e-3 and float(err.mean()) <= 1e-5
    assert torch.equal(state[4].cpu(), S0[4].transpose(1, 2).reshape(-1).float())


@pytest.mark.parametrize("n", [300, 2048])
def test_gla_state_is_carried_in_32_bits(n):
    """Decays close to one (0.999 and above) and far from it (a channel whose z is -60, one whose z is 60), in steps of 1 to
    50 tokens: the state stays within 2e-5 of its scale of the float64 recurrence."""
    from yalm_amd.ops import kernels
    H, d, dv, rank, tau = 2, 16, 24, 4, 16.0
    g = gen(5)
    proj = (torch.randn(n, 2 * H * d + 2 * H * dv + rank, generator=g, dtype=F64)).float().to(F64)
    w2 = (torch.randn(H * d, rank, generator=g, dtype=F64) * 0.2).float().to(F64)
    bias = torch.full((H * d,), 6.0, dtype=F64)
    bias[3], bias[20] = -60.0, 60.0
    a = P.decays(proj[:, 2 * H * (d + dv):], {"heads": H, "dim": d, "tau": tau}, {"a1": torch.eye(rank), "a2": w2, "a2.b": bias}, "")
    k, v = proj[:, H * d:2 * H * d].reshape(n, H, d), proj[:, 2 * H * d:2 * H * d + H * dv].reshape(n, H, dv)
    S = torch.stack([P.gla_scan(k[:, i], k[:, i], v[:, i], a[:, i], torch.zeros(d, dv, dtype=F64))[1] for i in range(H)])
    state = torch.zeros(1, H * d * dv, dtype=torch.float32, device=DEV)
    at, j = 0, 0
    while at < n:
        m = min(n - at, 1 + (7 * j) % 50)
        raw = torch.empty(m, H * dv, dtype=torch.float32, device=DEV)
        kernels.gla(f32(proj[at:at + m]), f32(w2), f32(bias), torch.ones(dv, device=DEV), state, raw, i32([0, m]), i32([0]),
                    torch.empty(m, H * dv, dtype=torch.float32, device=DEV), H, d, dv, rank, 1.0, tau, 1e-5)
        at, j = at + m, j + 1
    got = state[0].cpu().to(F64).reshape(H, dv, d).transpose(1, 2)
    assert float(S.abs().max()) > 5.0
    assert float((got - S).abs().max()) <= 2e-5 * float(S.abs().max())


# ------------------------------------------------------------------------------------------ whole models
def make_folder(tmp, name, cfg, seed, stored, change=None):
    """A folder with random weights; the decays' biases are moved up, so that the recurrences remember (tau near 1 forgets
    in a few tokens otherwise); change(name, tensor) may replace tensors."""
    from yalm_amd.weights import TensorSource, write_file, write_random_model
    folder = os.path.join(str(tmp), "%s_%d_%s" % (name, seed, str(stored).split(".")[-1]))
    if os.path.exists(os.path.join(folder, "model.safetensors")):
        return folder
    write_random_model(folder, cfg, seed=seed, dtype=torch.float32)
    src = TensorSource(folder)
    t = {n: src.get(n).clone() for n in src.names()}
    for n in t:
        if n.endswith(".a2.b"):
            t[n] = t[n] * 2.0 + 1.5
        if change is not None:
            t[n] = change(n, t[n])
    write_file(os.path.join(folder, "model.safetensors"), {n: v.to(stored).contiguous() for n, v in t.items()})
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("gemepel")
    return {(name, dt): make_folder(tmp, name, cfg, 5, helpers.torch_dtype(dt))
            for name, cfg in GC.ALL.items() for dt in ("float32", "bfloat16")}


_engines, _plain = {}, {}


def engine_for(folders, name, dtype, max_tokens=4096, **kw):
    from yalm_amd.engine import Engine, Model
    key = (folders[(name, dtype)], dtype, max_tokens, tuple(sorted(kw.items())))
    if key not in _engines:
        model = Model.from_folder(folders[(name, dtype)], dtype=helpers.torch_dtype(dtype), device=DEV, strict=True)
        _engines[key] = Engine(model, max_tokens=max_tokens, **kw)
    return _engines[key]


def plain_result(folder, tokens):
    """(logits [T, vocab], whether something earlier or now stands on a close call at each position [T])."""
    key = (folder, tuple(tokens))
    if key not in _plain:
        cfg, w = R.read_folder(folder)
        margins, faint = [], []
        logits = P.forward(cfg, w, list(tokens), margins_out=margins, faint_out=faint).float().numpy()
        close = np.zeros(len(tokens), dtype=bool)
        for m in margins:
            close |= m.numpy() < CLOSE_CALL
        for f in faint:
            close |= f.numpy() < FAINT
        _plain[key] = (logits, np.maximum.accumulate(close))
    return _plain[key]


CLOSE_CALL = 0.06          # a router choice whose margin (plain.route_margin) is below this may fall otherwise in bfloat16
FAINT = 0.3                # a recurrent head whose read-out is this small beside the layer's median: its norm divides by it


def check_request(got, folder, dtype, toks, what):
    """float32: every position within the tolerance.  bfloat16: the same, except that a position may differ more if a
    router choice at or before it in its request was a close call (the other expert is then as good an answer, and later
    positions read that token's keys and states) or a recurrent head read next to nothing from its state.  Returns the
    number of such positions; the caller bounds it."""
    want, close = plain_result(folder, toks)
    tol = (helpers.F32_TOL if dtype == "float32" else helpers.BF16_MAX_TOL) * max(1.0, np.abs(want).max())
    err = np.abs(np.asarray(got, np.float64) - want).max(axis=1)
    assert np.isfinite(err).all(), "%s: logits that are not finite" % what
    bad = np.nonzero(err > tol)[0]
    if len(bad) and (dtype == "float32" or not close[bad[0]]):
        raise AssertionError("%s: first wrong position %d of %d (error %.3g, allowed %.3g)" % (what, bad[0], len(toks), err[bad[0]], tol))
    return len(bad)


def requests_for(cfg, lengths, seed=0):
    g = np.random.default_rng(seed)
    return {"r%d" % i: g.integers(0, cfg["vocab"], size=n).tolist() for i, n in enumerate(lengths)}


def poison_when_idle(engine):
    """Between batches, when no sequence is alive, pages and states are filled with what must not reach a new sequence's
    logits (NaN; a token for the embedding's state): pages behind its length are never read, its states are cleared."""
    def before(step):
        if not engine.cache.slots.held:
            for g in engine.cache.kv_groups:
                g.k_pages.fill_(float("nan"))
                g.v_pages.fill_(float("nan"))
            for g in engine.cache.state_groups:
                g.data.fill_(float("nan") if g.data.is_floating_point() else 3)
    return before


def compare(folders, name, dtype, steps, requests, engine, what):
    out = schedules.replay_in_process(engine, steps, before_step=poison_when_idle(engine))
    got = schedules.per_request(steps, out, requests)
    differ = sum(check_request(got[rid], folders[(name, dtype)], dtype, toks, "%s %s %s request %s" % (name, dtype, what, rid))
                 for rid, toks in requests.items())
    total = sum(len(t) for t in requests.values())
    assert differ <= max(3, 0.15 * total), "%s %s %s: %d of %d positions differ behind close calls" % (name, dtype, what, differ, total)
    assert not engine.cache.slots.held
    for g in engine.cache.kv_groups:
        assert g.pool.n_free == g.n_pages


LENGTHS = {"mixed": [1, 2, 23, 64, 65, 150, 230], "medium": [300, 70, 131], "wide_latent": [2, 100, 250], "odd": [1, 9, 10, 70, 129],
           "only_gla": [1, 2, 17, 140], "only_latent": [3, 64, 65, 130], "only_state": [1, 2, 70]}
GROUPS = {"mixed": [([0, 2, 4, 5], [1, 23, 60, 100]), ([6, 1, 3], [221, 2, 64]), ([5, 4], [2, 1])],
          "medium": [([0, 1, 2], [250, 3, 100]), ([2, 1], [1, 64])],
          "wide_latent": [([0, 1, 2], [2, 60, 222]), ([2, 1], [1, 99])],
          "odd": [([0, 1, 2, 3], [1, 3, 10, 64]), ([4, 3], [100, 1])],
          "only_gla": [([0, 1, 2, 3], [1, 1, 9, 100]), ([3, 2], [1, 16])],
          "only_latent": [([0, 1, 2], [2, 63, 64]), ([3, 1], [100, 1])], "only_state": [([0, 1, 2], [1, 1, 40]), ([2, 1], [69, 1])]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LENGTHS))
def test_whole_prompts(folders, name, dtype):
    requests = requests_for(GC.ALL[name], LENGTHS[name])
    compare(folders, name, dtype, schedules.whole(requests), requests, engine_for(folders, name, dtype), "whole prompts")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LENGTHS))
def test_last_tokens_one_by_one(folders, name, dtype):
    requests = requests_for(GC.ALL[name], LENGTHS[name], seed=1)
    compare(folders, name, dtype, schedules.tail_one_by_one(requests, tail=80), requests, engine_for(folders, name, dtype),
            "last 80 tokens one by one")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "medium", "odd", "only_gla"])
def test_token_by_token_from_the_first(folders, name, dtype):
    requests = requests_for(GC.ALL[name], [150], seed=2)
    compare(folders, name, dtype, schedules.tail_one_by_one(requests, tail=10 ** 6), requests, engine_for(folders, name, dtype),
            "token by token")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(GROUPS))
def test_unequal_batches_with_reuse(folders, name, dtype):
    """Batches of unequal requests one after another and overlapping in time, in a cache with room for little more than
    one batch: slots, pages, recurrent states and previous tokens are given back and taken again."""
    base = requests_for(GC.ALL[name], LENGTHS[name], seed=3)
    reqs, plan, firsts = {}, [], {}
    for gi, (idx, lens) in enumerate(GROUPS[name]):
        row = []
        for i, n in zip(idx, lens):
            rid = "g%d_r%d" % (gi, i)
            reqs[rid] = base["r%d" % i]
            firsts[rid] = min(n, len(reqs[rid]))
            row.append(rid)
        plan.append(row)
    steps = schedules.batches(reqs, plan, firsts)
    compare(folders, name, dtype, steps, reqs, engine_for(folders, name, dtype, max_tokens=schedules.max_tokens_needed(steps) + 64),
            "batches")
    if len(plan) > 1:
        steps = schedules.interleaved(reqs, plan, firsts, [0] + [3 * i for i in range(1, len(plan))])
        compare(folders, name, dtype, steps, reqs, engine_for(folders, name, dtype), "overlapping batches")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,n_requests", [("mixed", 20), ("mixed", 70), ("mixed", 140), ("medium", 70)])
def test_batches_of_many_requests(folders, name, n_requests, dtype):
    """Decode batches beyond 16, 64 and 128 rows take other product kernels and graph buckets."""
    g = np.random.default_rng(n_requests)
    lengths = [int(n) for n in g.integers(1, 14, size=n_requests)]
    lengths[0], lengths[1] = 30, 26
    requests = requests_for(GC.ALL[name], lengths, seed=6)
    firsts = {rid: max(1, len(t) - int(g.integers(0, 6))) for rid, t in requests.items()}
    steps = schedules.batches(requests, [list(requests)], firsts)
    compare(folders, name, dtype, steps, requests, engine_for(folders, name, dtype, max_tokens=n_requests * 64 + 64), "many requests")


@pytest.mark.parametrize("name", ["mixed", "medium"])
def test_without_graphs_and_on_the_float32_arithmetic_kernels(folders, name, monkeypatch):
    """The same logits from decode steps launched kernel by kernel, and from the kernels of the 32-bit path on bfloat16
    storage."""
    from yalm_amd.ops import kernels
    requests = requests_for(GC.ALL[name], [90, 20], seed=7)
    steps = schedules.batches(requests, [list(requests)], {"r0": 50, "r1": 3})
    compare(folders, name, "bfloat16", steps, requests, engine_for(folders, name, "bfloat16", use_graphs=False), "no graphs")
    monkeypatch.setattr(kernels, "FORCE_SIMPLE", True)
    compare(folders, name, "bfloat16", steps, requests, engine_for(folders, name, "bfloat16", use_graphs=False, max_graphs=3),
            "float32-arithmetic kernels")


# ------------------------------------------------------------------------------------------ faults that random weights would hide
def logits_of(engine, toks, decode_from=None):
    """Logits of every position: the whole text as one prompt, or its tail from decode_from on token by token."""
    s = engine.start(1)
    n0 = len(toks) if decode_from is None else decode_from
    rows = [engine.step(s, [toks[:n0]], [list(range(n0))]).float().cpu().numpy().copy()]
    for t in toks[n0:]:
        rows.append(engine.step(s, [[t]], [[0]]).float().cpu().numpy().copy())
    engine.release(s)
    return np.concatenate(rows)


def changed_engine(tmp_path, name, dtype, change):
    from yalm_amd.engine import Engine, Model
    folder = make_folder(tmp_path, name + "_changed", GC.ALL[name], 7, helpers.torch_dtype(dtype), change=change)
    return folder, Engine(Model.from_folder(folder, dtype=helpers.torch_dtype(dtype), device=DEV), max_tokens=1024)


@pytest.mark.parametrize("name,n", [("only_latent", 449), ("wide_latent", 300), ("mixed", 300)])
def test_sharp_attention_over_hundreds_of_keys(tmp_path, name, n):
    """The queries' latent norms scaled up: attention is nearly one-hot on single keys among hundreds, so that a key lost
    far back, at a page's border or among the first tokens shows in float32's tolerance."""
    folder, engine = changed_engine(tmp_path, name, "float32", lambda k, v: v * 9.0 if k.endswith(".dq.norm") else v)
    toks = requests_for(GC.ALL[name], [n], seed=9)["r0"]
    want, _ = plain_result(folder, toks)
    for decode_from in (None, n - 160):
        err = np.abs(logits_of(engine, toks, decode_from) - want).max(axis=1)
        bad = np.nonzero(err > 3 * helpers.F32_TOL * max(1.0, np.abs(want).max()))[0]
        assert not len(bad), "first wrong position %d (error %.3g)" % (bad[0], err[bad[0]])


@pytest.mark.parametrize("decode_from", [None, 20, 66])
def test_every_earlier_key_is_seen_and_no_later_one(tmp_path, decode_from):
    """One attention layer without anything else that mixes tokens (no table of pairs' influence beyond the next token):
    changing ONE token changes the logits of every position from it on, and of none before it."""
    def change(k, v):
        return torch.zeros_like(v) if k == "bigram" else (v * 4.0 if k.endswith(".uk") else v)
    _, engine = changed_engine(tmp_path, "only_latent", "float32", change)
    toks = requests_for(GC.ONLY_LATENT, [70], seed=8)["r0"]
    base = logits_of(engine, toks, decode_from)
    for j in (0, 1, 19, 63, 64, 65, 69):
        other = list(toks)
        other[j] = (other[j] + 1) % GC.ONLY_LATENT["vocab"]
        moved = np.abs(logits_of(engine, other, decode_from) - base).max(axis=1) > 1e-7
        assert not moved[:j].any() and moved[j:].mean() > 0.95, (j, np.nonzero(moved)[0].tolist())


@pytest.mark.parametrize("decode_from", [None, 2, 150])
def test_the_recurrent_state_carries_the_first_token(tmp_path, decode_from):
    """One recurrence under decays close to one (0.9999 and above): the engine agrees with the plain recurrence over 300
    positions, through a prompt, through decoding and through both, and the first token still moves the last logits."""
    folder, engine = changed_engine(tmp_path, "only_state", "float32", lambda k, v: v * 0.1 + 7.5 if k.endswith(".a2.b") else v)
    toks = requests_for(GC.ONLY_STATE, [300], seed=10)["r0"]
    got = logits_of(engine, toks, decode_from)
    want, _ = plain_result(folder, toks)
    assert np.abs(got - want).max() <= helpers.F32_TOL * max(1.0, np.abs(want).max())
    other = [(toks[0] + 1) % GC.ONLY_STATE["vocab"]] + toks[1:]
    assert np.abs(logits_of(engine, other, decode_from)[299] - got[299]).max() > 1e-4


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decode_from", [None, 1, 2, 3, 12])
def test_a_token_sees_the_one_before_it_across_a_step(tmp_path, decode_from, dtype):
    """A model whose mixers give nothing: a token sees its predecessor through the table of pairs alone.  Changing token j
    moves the logits of j and j + 1 and of no other position, wherever the prompt ended; a sequence that takes the slot
    afterwards starts afresh."""
    folder, engine = changed_engine(tmp_path, "only_latent", dtype, lambda k, v: torch.zeros_like(v) if k.endswith(".mix.o") else v)
    toks = requests_for(GC.ONLY_LATENT, [20], seed=15)["r0"]
    base = logits_of(engine, toks, decode_from)
    want, _ = plain_result(folder, toks)
    tol = helpers.F32_TOL if dtype == "float32" else helpers.BF16_MAX_TOL
    assert np.abs(base - want).max() <= tol * max(1.0, np.abs(want).max())
    for j in (0, 1, 2, 3, 11, 12, 19):
        other = list(toks)
        other[j] = (other[j] + 1) % GC.ONLY_LATENT["vocab"]
        moved = np.abs(logits_of(engine, other, decode_from) - base).max(axis=1) > 1e-6
        assert (moved == np.array([j <= i <= j + 1 for i in range(20)])).all(), (j, np.nonzero(moved)[0].tolist())


def test_a_layer_reads_the_keys_of_the_layer_it_names(folders, tmp_path):
    """Changing the key projection of layer 0 moves what layers 2 and 5 read: with layer 0's own result switched off, the
    logits still follow the plain implementation."""
    folder, engine = changed_engine(tmp_path, "mixed", "float32", lambda k, v: torch.zeros_like(v) if k == "l0.mix.o" else v)
    toks = requests_for(GC.MIXED, [90], seed=16)["r0"]
    want, _ = plain_result(folder, toks)
    for decode_from in (None, 1, 50):
        assert np.abs(logits_of(engine, toks, decode_from) - want).max() <= helpers.F32_TOL * max(1.0, np.abs(want).max())
    cfg, w = R.read_folder(folder)
    w2 = dict(w)
    w2["l0.mix.dkv"] = w["l0.mix.dkv"] * -1.0
    assert float((P.forward(cfg, w2, toks[:9]) - P.forward(cfg, w, toks[:9])).abs().max()) > 1e-3


def test_long_decoding(folders):
    """400 tokens one by one after a short prompt: the recurrent states are read and written 400 times, seven pages fill."""
    requests = requests_for(GC.MIXED, [410], seed=11)
    compare(folders, "mixed", "float32", schedules.tail_one_by_one(requests, tail=400), requests,
            engine_for(folders, "mixed", "float32"), "long decoding")


# ------------------------------------------------------------------------------------------ the library's entry points
def plain_greedy(folder, prompt, n_new):
    cfg, w = R.read_folder(folder)
    seq, memory = list(prompt), {}
    logits = P.forward(cfg, w, seq, memory=memory)
    for i in range(n_new):
        seq.append(int(torch.argmax(logits[-1])))
        logits = P.forward(cfg, w, seq[-1:], memory=memory, start=len(seq) - 1)
    return seq[len(prompt):]


def test_greedy_generation_and_command_line(folders):
    from yalm_amd.generate import generate
    folder = folders[("mixed", "float32")]
    engine = engine_for(folders, "mixed", "float32")
    prompts = [[5, 17, 3, 100, 9], [7], list(range(60, 90))]
    got = generate(engine, prompts, max_new_tokens=12, temperature=0.0, stop_ids=())
    for p, g in zip(prompts, got):
        assert g == plain_greedy(folder, p, 12), (p, g)
        assert generate(engine, [p], max_new_tokens=12, temperature=0.0, stop_ids=())[0] == g
    assert not engine.cache.slots.held
    p = subprocess.run([sys.executable, "-m", "yalm_amd", folder, "-m", "c", "--tokens", ",".join(map(str, prompts[0])),
                        "-n", "12", "-t", "0", "--dtype", "float32"], cwd=ROOT, stdout=subprocess.PIPE,
                       stderr=subprocess.PIPE, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-3000:]
    printed = p.stdout.split("\n\n")[0].split("\n", 1)[1].split()
    assert [int(t) for t in printed] == got[0]


def test_token_probabilities(folders):
    engine = engine_for(folders, "odd", "float32")
    toks = requests_for(GC.ODD, [50], seed=13)["r0"]
    want, _ = plain_result(folders[("odd", "float32")], toks)
    s = engine.start(1)
    probs = engine.step(s, [toks[:-1]], [list(range(49))], targets=[toks[1:]]).cpu().numpy()
    engine.release(s)
    ref = torch.softmax(torch.tensor(want[:-1], dtype=F64), dim=-1).numpy()[np.arange(49), toks[1:]]
    assert np.allclose(probs, ref, rtol=2e-3, atol=1e-6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(folders, tmp_path, dtype):
    requests = requests_for(GC.MIXED, [1, 30, 90], seed=14)
    steps = schedules.batches(requests, [list(requests)], {"r0": 1, "r1": 12, "r2": 70})
    out = schedules.replay_trace_run(folders[("mixed", dtype)], dtype, steps, str(tmp_path / "out"),
                                     schedules.max_tokens_needed(steps))
    got = schedules.per_request(steps, out, requests)
    differ = sum(check_request(got[rid], folders[("mixed", dtype)], dtype, toks, "trace_run %s %s" % (dtype, rid))
                 for rid, toks in requests.items())
    assert differ <= 12


# ------------------------------------------------------------------------------------------ configurations drawn at random
def random_config(seed):
    """A Gemepel configuration whose every size, count, constant and the order of its layers are drawn from `seed`."""
    g = np.random.default_rng(seed)
    pick = lambda lo, hi: int(g.integers(lo, hi + 1))
    width = pick(17, 150)
    layers = []
    for i in range(pick(2, 6)):
        makers = [j for j in range(i) if layers[j]["type"] == "latent_attention" and "kv_from" not in layers[j]["mixer"]]
        if g.random() < 0.45:
            mixer = GC.gla(pick(1, 5), pick(2, 140), pick(2, 90), float(2.0 ** g.uniform(-1, 4)), pick(1, 30))
        elif makers and g.random() < 0.5:
            j = int(g.choice(makers))
            o = layers[j]["mixer"]
            mixer = GC.latent(pick(1, 6), pick(2, 60), o["rot_dim"], pick(2, 60), pick(2, 90), o["kv_rank"], float(g.uniform(0.05, 0.5)),
                              base=o["rot"]["base"], kv_from=j)
        else:
            mixer = GC.latent(pick(1, 6), pick(2, 60), 2 * pick(1, 16), pick(2, 60), pick(2, 90), pick(2, 150),
                              float(g.uniform(0.05, 0.5)), base=float(10.0 ** g.uniform(1, 6)))
        groups = pick(1, 4)
        per = pick(1, 5)
        keep = pick(1, groups)
        mlp = None if g.random() < 0.15 else GC.moe(groups * per, pick(1, keep * per), pick(3, 100), float(g.uniform(0.5, 3.0)), (groups, keep))
        layers.append(GC.layer(mixer, mlp))
    return GC.model(pick(30, 400), width, float(10.0 ** g.uniform(-7, -4)), float(g.uniform(0.5, 4.0)), layers, float(g.uniform(0.3, 3.0)),
                    (pick(1, 600), pick(1, 1000), pick(1, 1000)) if g.random() < 0.85 else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [31, 32, 33, 34, 35, 36, 37, 38])
def test_configurations_drawn_at_random(tmp_path, seed, dtype):
    """A whole prompt, a prompt with its last tokens one by one, and two unequal requests in one batch."""
    from yalm_amd.engine import Engine, Model
    cfg = random_config(seed)
    folder = make_folder(tmp_path, "random%d" % seed, cfg, seed, helpers.torch_dtype(dtype))
    engine = Engine(Model.from_folder(folder, dtype=helpers.torch_dtype(dtype), device=DEV, strict=True), max_tokens=2048)
    requests = requests_for(cfg, [150, 41], seed=seed)
    folders = {("r", dtype): folder}
    compare(folders, "r", dtype, schedules.whole(requests), requests, engine, "random %d whole" % seed)
    compare(folders, "r", dtype, schedules.tail_one_by_one(requests, tail=60), requests, engine, "random %d tail" % seed)
    compare(folders, "r", dtype, schedules.batches(requests, [list(requests)], {"r0": 97, "r1": 3}), requests, engine,
            "random %d batch" % seed)
