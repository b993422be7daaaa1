"""The Zebivik design on the GPU against the plain implementation (tests/plain/zebivik_plain.py): the new kernels one by
one, then whole models under every way of cutting requests into steps (whole prompts, the last tokens one by one, from the
first token on, batches of unequal requests whose slots, pages and states are used again), keys far away under a sharp
query, recurrent states and convolution inputs that must carry a token over hundreds of steps, choices of experts at a group's
edge, greedy generation through generate() and the command line, the trace runner, and configurations drawn at random."""
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers
import schedules
import zebivik_configs as ZC
from plain import reference_model as R
from plain import zebivik_plain as P

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
nan = lambda *shape, dtype=torch.float32: torch.full(shape, float("nan"), dtype=dtype, device=DEV)
d64 = lambda t: t.to(F64)
scratch = lambda name, shape, dt: torch.full(shape, float("nan"), dtype=dt, device=DEV)


def inside(t, left, right):
    """The same values as columns of a wider matrix (NaN around them)."""
    wide = torch.full((t.shape[0], left + t.shape[1] + right), float("nan"), dtype=t.dtype, device=t.device)
    wide[:, left:left + t.shape[1]] = t
    return wide[:, left:left + t.shape[1]]


def close(got, want, dtype, f32_tol=2e-6, bf16_tol=1e-2):
    tol = f32_tol if dtype == torch.float32 else bf16_tol
    got = got.float().cpu().to(F64)
    assert torch.allclose(got, want, rtol=tol, atol=tol), float((got - want).abs().max())


# ------------------------------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R_,D", [(1, 1), (3, 7), (5, 80), (2, 1024), (3, 1030), (9, 4096), (2, 5001)])
def test_squash_kernels(R_, D, dtype):
    """The squash alone (with and without chosen rows, into float32 too), a sublayer's result under it added to the stream (with
    and without a bias), and the same followed by the squash that reads the stream next.  Values from far inside to far
    outside the curve's bend."""
    from yalm_amd.ops import kernels
    x, y = randn(R_, D, seed=1, scale=4.0), randn(R_, D, seed=2) ** 3
    w, b, w2, b2, yb = (randn(D, seed=s) for s in (3, 4, 5, 6, 7))
    n = lambda v, a, ww, bb: torch.tanh(a * d64(v)) * d64(ww) + d64(bb)
    out = nan(R_, D, dtype=dtype)
    kernels.squash(x.to(DEV), 0.37, w.to(DEV), b.to(DEV), out)
    close(out, n(x, 0.37, w, b), dtype)
    rows = [R_ - 1, 0]
    for dt in (dtype, torch.float32):
        out = nan(2, D, dtype=dt)
        kernels.squash(x.to(DEV), -1.9, w.to(DEV), b.to(DEV), out, row_index=i32(rows))
        close(out, n(x[rows], -1.9, w, b), dt)
    for bias in (None, yb):
        want = d64(x) + 0.3 * n(y if bias is None else d64(y) + d64(bias), 0.8, w, b)
        h = nan(R_, D, dtype=dtype)
        for h_out in (None, h):
            xd = x.clone().to(DEV)
            kernels.squash_add(y.to(DEV), 0.8, w.to(DEV), b.to(DEV), 0.3, xd, h_out, y_bias=None if bias is None else bias.to(DEV))
            close(xd, want, torch.float32, f32_tol=4e-6)
        close(h, want, dtype, f32_tol=4e-6)
        xd, h = x.clone().to(DEV), nan(R_, D, dtype=dtype)
        kernels.squash_add(y.to(DEV), 0.8, w.to(DEV), b.to(DEV), 0.3, xd, h, next_norm=(0.21, w2.to(DEV), b2.to(DEV)),
                           y_bias=None if bias is None else bias.to(DEV))
        close(xd, want, torch.float32, f32_tol=4e-6)
        close(h, n(want, 0.21, w2, b2), dtype, f32_tol=4e-6)
    tiny = torch.full((R_, D), 1e-4)                # no digits are lost near zero
    out = nan(R_, D)
    kernels.squash(tiny.to(DEV), 0.5, torch.ones(D, device=DEV), torch.zeros(D, device=DEV), out)
    assert torch.allclose(d64(out.cpu()), torch.tanh(0.5 * d64(tiny)), rtol=1e-5, atol=0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R_,n", [(1, 1), (3, 60), (5, 1000), (2, 1500), (7, 4096), (2, 9001)])
def test_rms_gate(R_, n, dtype):
    from yalm_amd.ops import kernels
    x, w, z = randn(R_, n, seed=1, scale=3.0), randn(n, seed=2), randn(R_, n, seed=3, scale=2.0)
    want = P.rms_norm(d64(x), d64(w), 1e-5) * torch.sigmoid(d64(z))
    for gate, out in ((z.to(DEV), nan(R_, n, dtype=dtype)), (inside(z.to(DEV), 3, 5), inside(nan(R_, n, dtype=dtype), 4, 2))):
        kernels.rms_gate(x.to(DEV), w.to(DEV), 1e-5, gate, out)
        close(out, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,dv", [(1, 1, 16), (1, 6, 48), (5, 3, 80), (300, 8, 128), (9, 32, 128)])
def test_head_gate(T, H, dv, dtype):
    """In place and into columns of a wider row, whose other columns stay as they are."""
    from yalm_amd.ops import kernels
    o, g = randn(T, H * dv, seed=1).to(dtype), randn(T, H, seed=2, scale=2.0)
    want = (d64(o).reshape(T, H, dv) * torch.sigmoid(d64(g))[..., None] * 1.3).reshape(T, H * dv)
    od = o.clone().to(DEV)
    kernels.head_gate(od, inside(g.to(DEV), 2, 1), H, 1.3)
    close(od, want, dtype)
    wide = torch.full((T, H * dv + 7), 5.0, dtype=dtype, device=DEV)
    kernels.head_gate(o.to(DEV), g.to(DEV), H, 1.3, wide[:, 3:3 + H * dv])
    close(wide[:, 3:3 + H * dv], want, dtype)
    assert bool((wide[:, :3] == 5.0).all()) and bool((wide[:, 3 + H * dv:] == 5.0).all())


def test_softcap():
    from yalm_amd.ops import kernels
    z = randn(7, 1003, seed=1, scale=40.0)
    got = kernels.softcap(z.clone().to(DEV), 30.0)
    close(got, 30.0 * torch.tanh(d64(z) / 30.0), torch.float32, f32_tol=4e-6)
    with pytest.raises(Exception):
        kernels.softcap(z.to(DEV), 0.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,taps,row", [(5, 3, 11), (64, 4, 192), (40, 1, 40), (24, 2, 48), (33, 7, 35), (4096, 4, 8192)])
def test_convolution_with_biases_on_columns_of_a_wider_row(D, taps, row, dtype):
    """Two texts in pieces of several tokens and of one (with and without the one-launch form), beside a padding row.  The bias of
    the inputs is not part of the zeros in front of a text."""
    from yalm_amd.ops import kernels
    x = {b: randn(n, D, seed=b).to(dtype) for b, n in ((0, 12), (1, 9))}
    ib, ob, w = randn(D, seed=5), randn(D, seed=6), randn(D, taps, seed=7)
    want = {b: P.causal_conv(d64(x[b]) + d64(ib), d64(w), d64(ob), {}) for b in x}
    carried = nan(4, taps - 1, D) if taps > 1 else None
    slots, at = [3, 1], [0, 0]
    if taps > 1:
        carried[3].zero_(); carried[1].zero_()
    for lens in ([4, 1], [1, 0], [3, 5], [1, 1], [1, 1], [2, 1]):
        rows, seq, cu, ss = [], [], [0], []
        for b in (0, 1):
            if lens[b]:
                rows.append(x[b][at[b]:at[b] + lens[b]])
                seq += [len(ss)] * lens[b]
                cu.append(cu[-1] + lens[b]); ss.append(slots[b])
        rows.append(torch.zeros(1, D, dtype=dtype)); seq.append(len(ss)); cu.append(cu[-1] + 1); ss.append(-1)
        h = inside(torch.cat(rows).to(DEV), row - D, 0)
        out = nan(h.shape[0], D, dtype=dtype)
        kernels.time_conv(h, f32(w.t()), carried, out, i32(seq), i32(cu), i32(ss), residual=False, one_token_each=max(lens) == 1,
                          in_bias=ib.to(DEV), bias=ob.to(DEV))
        r = 0
        for b in (0, 1):
            close(out[r:r + lens[b]], want[b][at[b]:at[b] + lens[b]], dtype, f32_tol=1e-5, bf16_tol=2e-2)
            r += lens[b]
            at[b] += lens[b]
            if lens[b] and taps > 1:
                kept = (d64(x[b]) + d64(ib))[max(0, at[b] - taps + 1):at[b]]
                close(carried[slots[b], taps - 1 - kept.shape[0]:], kept, torch.float32)
    assert at == [12, 9] and (taps == 1 or bool(torch.isnan(carried[0]).all()))


@pytest.mark.parametrize("softmax,group_max", [(True, True), (True, False), (False, True)])
@pytest.mark.parametrize("E,top,groups,keep,scale", [(14, 5, 2, 1, 1.8), (12, 3, 4, 2, 1.0), (1, 1, 1, 1, 0.5), (6, 2, 6, 3, 1.5), (6, 6, 1, 1, 1.0),
                                                     (64, 8, 8, 4, 2.5), (300, 5, 100, 2, 1.0), (1024, 9, 2, 2, 1.0)])
def test_choice_inside_groups(E, top, groups, keep, scale, softmax, group_max):
    """Corrections from strongly negative to strongly positive (all choice scores negative, all positive, mixed), so that
    a mask of zeros or weights with the correction in them would show."""
    from yalm_amd.ops import kernels
    T = 50
    for shift, seed in ((-3.0, 1), (0.0, 2), (2.0, 3)):
        z, corr = randn(T, E, seed=seed, scale=1.5), randn(E, seed=seed + 10, scale=0.3) + shift
        s = torch.softmax(d64(z), -1) if softmax else torch.sigmoid(d64(z))
        c = (s + d64(corr)).reshape(T, groups, -1)
        best = c.max(-1).values if group_max else torch.topk(c, min(2, c.shape[-1]), dim=-1).values.sum(-1)
        kept = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, torch.topk(best, keep, dim=-1).indices, True)
        masked = c.masked_fill(~kept[..., None], float("-inf")).reshape(T, E)
        order = torch.topk(masked, min(top + 1, E), dim=-1).values
        sure = torch.ones(T, dtype=torch.bool)
        if top < E:
            sure &= order[:, top - 1] - order[:, -1] > 1e-5
        if keep < groups:
            g = torch.topk(best, keep + 1, dim=-1).values
            sure &= g[:, -2] - g[:, -1] > 1e-5
        chosen = torch.topk(masked, top, dim=-1).indices
        weight = torch.gather(s, 1, chosen)
        weight = weight / weight.sum(-1, keepdim=True) * scale
        ids, wts = torch.full((T, top), -7, dtype=torch.int32, device=DEV), nan(T, top)
        kernels.moe_select_groups(z.to(DEV), corr.to(DEV), ids, wts, groups, keep, scale, softmax=softmax, group_max=group_max)
        got_ids, got_w = ids.cpu().long(), d64(wts.cpu())
        assert sure.float().mean() > 0.8
        dense = lambda i, v: torch.zeros(T, E, dtype=F64).scatter_(1, i, v)      # the order among the chosen may differ
        a, b = dense(got_ids, got_w)[sure], dense(chosen, weight)[sure]
        assert torch.allclose(a, b, rtol=1e-5, atol=1e-6), float((a - b).abs().max())


def test_choice_by_softmax_at_the_ends():
    from yalm_amd.ops import kernels
    ids, wts = torch.empty(1, 2, dtype=torch.int32, device=DEV), torch.empty(1, 2, dtype=torch.float32, device=DEV)
    kernels.moe_select_groups(torch.zeros(1, 8, device=DEV), None, ids, wts, 4, 2, 1.0, softmax=True, group_max=True)
    assert ids.tolist() == [[0, 1]] and torch.allclose(wts.cpu(), torch.tensor([[0.5, 0.5]]))
    z = torch.tensor([[500.0, -500.0, -500.0, 400.0, 0.0, 0.0, 0.0, 0.0]], device=DEV)
    kernels.moe_select_groups(z, torch.tensor([-5.0, 1.0, 1.0, -5.0, 0, 0, 0, 0], device=DEV), ids, wts, 1, 1, 1.0, softmax=True)
    assert sorted(ids[0].tolist()) == [1, 2] and bool(torch.isfinite(wts).all())        # chosen experts whose scores vanish


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D,F", [(64, 48), (80, 96), (50, 17), (192, 256), (512, 1024)])
@pytest.mark.parametrize("M", [1, 3, 8, 16, 17, 40, 100, 130, 300, 1100])
def test_clamped_unit_in_the_products_epilogue(M, D, F, dtype):
    """Every product kernel (by rows and sizes) clamps the gate from above only and the up value on both sides."""
    from yalm_amd.ops import kernels
    from yalm_amd.parts.swiglu import interleave_gate_up
    h = randn(M, D, seed=1).to(dtype)
    gate, up = randn(F, D, seed=2, scale=2.0 * D ** -0.5).to(dtype), randn(F, D, seed=3, scale=2.0 * D ** -0.5).to(dtype)
    g, u = (d64(h) @ d64(gate).T), (d64(h) @ d64(up).T)
    for limit, alpha, shift in ((0.9, 1.702, 1.0), (0.0, 1.0, 0.0)):
        gg, uu = (g.clamp(max=limit), u.clamp(-limit, limit)) if limit else (g, u)
        want = gg * torch.sigmoid(alpha * gg) * (uu + shift)
        mid = nan(M, F, dtype=dtype)
        w = interleave_gate_up(gate, up).contiguous().to(DEV)
        n = kernels.gemm_workspace_floats(M, w.shape[0], D) if dtype == torch.bfloat16 else 0
        ws = nan(n) if n else None
        kernels.gemm(h.to(DEV), w, mid, kernels.EPI_GATED, hidden=F, workspace=ws, unit=(limit, alpha, shift))
        close(mid, want, dtype, f32_tol=2e-5, bf16_tol=2e-2)


def scan_texts(H, d, dv, decay, lens, seed, sc=1.5):
    g = gen(seed)
    rn = lambda *s: (torch.randn(*s, generator=g, dtype=F64) * sc).float().to(F64)
    return [rn(n, 2 * H * d + H * dv) for n in lens]


def plain_lightning(pr, H, d, dv, decay, S0=None):
    n = pr.shape[0]
    q, k = (P.silu(pr[:, i * H * d:(i + 1) * H * d]).reshape(n, H, d) for i in (0, 1))
    v = P.silu(pr[:, 2 * H * d:]).reshape(n, H, dv)
    outs, states = zip(*[P.decay_scan(q[:, i], k[:, i], v[:, i], decay[i], torch.zeros(d, dv, dtype=F64) if S0 is None else S0[i])
                         for i in range(H)])
    return torch.stack(outs, dim=1).reshape(n, H * dv), torch.stack(states)


def powers_of(decay):
    return f32(torch.tensor(decay, dtype=F64)[:, None] ** torch.arange(65, dtype=F64))


@pytest.mark.parametrize("n_first", [3, 40])
@pytest.mark.parametrize("d,dv,decay", [(1, 3, [0.5]), (4, 4, [0.0, 1.0]), (32, 48, [0.6, 0.93, 0.999]), (5, 9, [0.3, 0.97, 0.7]),
                                        (64, 40, [0.95, 0.5]), (128, 70, [0.98]), (200, 33, [0.9, 1.0]), (256, 16, [0.99, 0.1]), (44, 200, [0.8])])
def test_lightning_kernel(d, dv, decay, n_first):
    """Two sequences and a padding row, as columns of a wider row: first pieces, then single tokens, against the plain recurrence over
    the whole texts; the state left behind against the plain one (it is kept column by column)."""
    from yalm_amd.ops import kernels
    H = len(decay)
    lens = [n_first + 6, 7]
    texts = scan_texts(H, d, dv, decay, lens, H * 100 + d)
    want = [plain_lightning(t, H, d, dv, decay) for t in texts]
    state = torch.zeros(4, kernels.lightning_state_elements(H, d, dv), dtype=torch.float32, device=DEV)
    state[1].fill_(float("nan"))
    slots, powers = [2, 0], powers_of(decay)

    def step(rows, cu, seq_slot):
        proj = inside(f32(torch.cat(rows)), 4, 3)
        raw = nan(proj.shape[0], H * dv)
        kernels.lightning(proj, powers, state, raw, i32(cu), i32(seq_slot), H, d, dv)
        return d64(raw.cpu())

    first, got = [n_first, 1], [[], []]
    out = step([texts[0][:first[0]], texts[1][:first[1]]], [0, first[0], first[0] + first[1]], slots)
    got[0].append(out[:first[0]]); got[1].append(out[first[0]:])
    for t in range(lens[0] - first[0]):
        rows, ss = [texts[0][first[0] + t:first[0] + t + 1], torch.zeros(1, texts[0].shape[1], dtype=F64)], [slots[0], -1]
        more = first[1] + t < lens[1]
        if more:
            rows.append(texts[1][first[1] + t:first[1] + t + 1]); ss.append(slots[1])
        out = step(rows, list(range(len(rows) + 1)), ss)
        assert float(out[1].abs().max()) == 0.0      # the padding row
        got[0].append(out[0:1])
        if more:
            got[1].append(out[2:3])
    for b in range(2):
        o = torch.cat(got[b])
        assert float((o - want[b][0]).abs().max()) <= 2e-6 * max(1.0, float(want[b][0].abs().max())) * 4
        S = d64(state[slots[b]].cpu()).reshape(H, dv, d).transpose(1, 2)
        assert torch.allclose(S, want[b][1], rtol=1e-5, atol=1e-5)
    assert bool(torch.isnan(state[1]).all()) and float(state[3].abs().sum()) == 0.0


@pytest.mark.parametrize("left", [4, 3])
@pytest.mark.parametrize("d,dv,decay", [(1, 3, [0.5]), (4, 4, [0.0, 1.0, 1e-3]), (32, 48, [0.6, 0.93, 0.999]), (33, 17, [0.3, 0.97]),
                                        (64, 40, [0.95, 0.5]), (128, 128, [0.98, 1.0]), (100, 200, [0.9]), (126, 70, [0.9999])])
def test_lightning_prompts_tile_by_tile(d, dv, decay, left):
    """Prompts of unequal lengths (one token to several tiles, one that ends a tile and one just behind it), from states that
    are not zero: read-outs and states as the recurrence gives them, under decays of nothing to one.  The row's
    columns stand aligned and not."""
    from yalm_amd.ops import kernels
    H = len(decay)
    lens = [1, 64, 65, 200, 17]
    texts = scan_texts(H, d, dv, decay, lens, H * 100 + d)
    slots = [2, 0, 5, 3, 1]
    S0 = (torch.randn(6, H, d, dv, generator=gen(9), dtype=F64) * 0.3).float().to(F64)
    state = f32(S0.transpose(2, 3).reshape(6, -1))
    cu, tile0 = np.concatenate([[0], np.cumsum(lens)]), np.concatenate([[0], np.cumsum([(n + 63) // 64 for n in lens])])
    raw = nan(int(cu[-1]), H * dv)
    proj = inside(f32(torch.cat(texts)), left, (-left - texts[0].shape[1]) % 4)
    kernels.lightning_tiles(proj, powers_of(decay), state, raw, i32(cu), i32(slots), i32(tile0), int(tile0[-1]), H, d, dv, scratch)
    for b, t in enumerate(texts):
        o, S_want = plain_lightning(t, H, d, dv, decay, S0[slots[b]])
        got = d64(raw[cu[b]:cu[b + 1]].cpu())
        assert float((got - o).abs().max()) <= 1e-5 * max(1.0, float(o.abs().max())), (b, float((got - o).abs().max()))
        S = d64(state[slots[b]].cpu()).reshape(H, dv, d).transpose(1, 2)
        assert float((S - S_want).abs().max()) <= 1e-5 * max(1.0, float(S_want.abs().max()))
    assert torch.equal(state[4].cpu(), S0[4].transpose(1, 2).reshape(-1).float())


@pytest.mark.parametrize("n", [300, 2048])
def test_lightning_state_is_carried_in_32_bits(n):
    """Decays of one and close to it, in steps of 1 to 50 tokens: the state stays within 2e-5 of its scale of the float64
    recurrence."""
    from yalm_amd.ops import kernels
    H, d, dv, decay = 3, 16, 24, [1.0, 0.9995, 0.5]
    text = scan_texts(H, d, dv, decay, [n], 5, sc=1.0)[0]
    _, S = plain_lightning(text, H, d, dv, decay)
    state = torch.zeros(1, H * d * dv, dtype=torch.float32, device=DEV)
    at, j = 0, 0
    while at < n:
        m = min(n - at, 1 + (7 * j) % 50)
        kernels.lightning(f32(text[at:at + m]), powers_of(decay), state, nan(m, H * dv), i32([0, m]), i32([0]), H, d, dv)
        at, j = at + m, j + 1
    got = d64(state[0].cpu()).reshape(H, dv, d).transpose(1, 2)
    assert float(S.abs().max()) > 20.0
    assert float((got - S).abs().max()) <= 2e-5 * float(S.abs().max())


def lru_case(W, nb, seed, wdtype, slow):
    """Random gates over W channels in nb blocks; slow: decays close to one in half of the channels, far from it in the rest."""
    n = W // nb
    g = gen(seed)
    rn = lambda *s, sc=1.0: (torch.randn(*s, generator=g, dtype=F64) * sc).float()
    lam = rn(W)
    if slow:
        lam[::2] -= 9.0
    c = {"ra": rn(nb, n, n, sc=n ** -0.5).to(wdtype), "ri": rn(nb, n, n, sc=n ** -0.5).to(wdtype), "ra.b": rn(nb, n), "ri.b": rn(nb, n),
         "lam": lam, "y.b": rn(W), "W": W, "n": n}
    c["w"] = torch.stack([c["ra"], c["ri"]]).contiguous().to(DEV)
    c["bias"] = f32(torch.stack([c["ra.b"].reshape(-1), c["ri.b"].reshape(-1)]))
    c["slope"] = f32(-8.0 * torch.nn.functional.softplus(d64(lam)))
    return c


def plain_lru(c, u, z, S0):
    r, i = (P.block_gate(u, d64(c[k]), d64(c[k + ".b"])) for k in ("ra", "ri"))
    s, S = P.lru_scan(u, r, i, d64(c["lam"]), S0)
    return s * P.gelu_tanh(z + d64(c["y.b"])), S


LRU_SIZES = [(1, 1), (24, 3), (22, 22), (35, 5), (120, 5), (320, 5), (192, 24), (77, 7), (512, 2), (80, 1), (600, 3)]


@pytest.mark.parametrize("slow", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,nb", LRU_SIZES)
def test_gated_recurrence_of_prompts(W, nb, dtype, slow):
    """Prompts of unequal lengths (one token to several tiles, one that ends a tile and one just behind it), from states that
    are not zero."""
    from yalm_amd.ops import kernels
    lens = [1, 64, 65, 200, 17]
    c = lru_case(W, nb, W + nb, dtype, slow)
    T = sum(lens)
    u, z = randn(T, W, seed=2), randn(T, W, seed=3)
    slots = [2, 0, 5, 3, 1]
    S0 = randn(6, W, seed=4)
    state = S0.clone().to(DEV)
    cu, tile0 = np.concatenate([[0], np.cumsum(lens)]), np.concatenate([[0], np.cumsum([(n + 63) // 64 for n in lens])])
    out = nan(T, W, dtype=dtype)
    kernels.lru(u.to(DEV), c["w"], c["bias"], c["slope"], inside(z.to(DEV), 0, W), f32(c["y.b"]), state, out, i32(np.repeat(range(5), lens)),
                i32(cu), i32(slots), scratch, i32(tile0), int(tile0[-1]))
    for b in range(5):
        a, e = int(cu[b]), int(cu[b + 1])
        want, S = plain_lru(c, d64(u[a:e]), d64(z[a:e]), d64(S0[slots[b]]))
        close(out[a:e], want, dtype, f32_tol=2e-5, bf16_tol=2e-2)
        assert torch.allclose(d64(state[slots[b]].cpu()), S, rtol=2e-5, atol=2e-5), float((d64(state[slots[b]].cpu()) - S).abs().max())
    assert torch.equal(state[4].cpu(), S0[4])


@pytest.mark.parametrize("B", [1, 3, 8, 9, 21, 70])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,nb", LRU_SIZES)
def test_gated_recurrence_of_single_tokens(W, nb, dtype, B):
    """Both forms of a step of single tokens, a padding row among them, several steps in a row."""
    from yalm_amd.ops import kernels
    c = lru_case(W, nb, W + nb, dtype, True)
    slots = [int(s) for s in np.random.default_rng(B).permutation(B + 2)[:B]]
    if B > 2:
        slots[B // 2] = -1
    S0 = randn(B + 2, W, seed=4)
    for form in ("step", "tiles"):
        state, S = S0.clone().to(DEV), d64(S0)
        for t in range(3):
            u, z = randn(B, W, seed=10 + t), randn(B, W, seed=20 + t)
            out = nan(B, W, dtype=dtype)
            args = (u.to(DEV), c["w"], c["bias"], c["slope"], inside(z.to(DEV), W, 0), f32(c["y.b"]), state, out)
            if form == "step":
                kernels.lru_step(*args, i32(slots))
            else:
                kernels.lru(*args, i32(range(B)), i32(range(B + 1)), i32(slots), scratch)
            for b, s in enumerate(slots):
                if s < 0:
                    assert float(out[b].abs().max()) == 0.0
                    continue
                want, S[s] = plain_lru(c, d64(u[b:b + 1]), d64(z[b:b + 1]), S[s])
                close(out[b:b + 1], want, dtype, f32_tol=2e-5, bf16_tol=2e-2)
        assert torch.allclose(d64(state.cpu()), S, rtol=2e-5, atol=2e-5)


def test_gated_recurrence_is_carried_in_32_bits():
    """2,048 tokens under decays from 0.9999 to next to nothing, in steps of 1 to 150 tokens through both forms, from inputs far
    larger than what a token adds: the state stays within 2e-5 of its scale of the float64 recurrence."""
    from yalm_amd.ops import kernels
    n, W = 2048, 16
    c = lru_case(W, 2, 3, torch.float32, True)
    c["lam"][0], c["lam"][1] = -12.0, 30.0
    c["slope"] = f32(-8.0 * torch.nn.functional.softplus(d64(c["lam"])))
    u, z = randn(n, W, seed=1, scale=5.0) + 3.0, randn(n, W, seed=2)
    _, S = plain_lru(c, d64(u), d64(z), torch.zeros(W, dtype=F64))
    state = torch.zeros(1, W, dtype=torch.float32, device=DEV)
    at, j = 0, 0
    while at < n:
        m = 1 if j % 3 else min(n - at, 1 + (37 * j) % 150)
        args = (u[at:at + m].contiguous().to(DEV), c["w"], c["bias"], c["slope"], z[at:at + m].contiguous().to(DEV), f32(c["y.b"]), state, nan(m, W))
        if m == 1:
            kernels.lru_step(*args, i32([0]))
        else:
            kernels.lru(*args, i32([0] * m), i32([0, m]), i32([0]), scratch, i32([0, (m + 63) // 64]), (m + 63) // 64)
        at, j = at + m, j + 1
    assert float((d64(state[0].cpu()) - S).abs().max()) <= 2e-5 * float(S.abs().max())


def test_operands_that_do_not_fit_are_errors():
    from yalm_amd.ops import kernels
    with pytest.raises(ValueError):
        kernels.lru_step(nan(2, 12), nan(2, 3, 5, 5), nan(2, 12), nan(12), nan(2, 12), nan(12), nan(4, 12), nan(2, 12), i32([0, 1]))
    with pytest.raises(ValueError):
        kernels.lightning(nan(2, 30), nan(1, 65), nan(4, 64), nan(2, 8), i32([0, 1, 2]), i32([0, 1]), 1, 8, 8)
    with pytest.raises(ValueError):
        kernels.lightning(nan(2, 2000), nan(1, 65), nan(4, 8000), nan(2, 8), i32([0, 1, 2]), i32([0, 1]), 1, 996, 8)
    with pytest.raises(ValueError):
        kernels.head_gate(nan(2, 30), nan(2, 4), 4)


# ------------------------------------------------------------------------------------------ whole models
def make_folder(tmp, name, cfg, seed, stored, change=None):
    """A folder with random weights; the channels' rates are moved down, so that the recurrences remember (they forget in a
    few tokens otherwise); change(name, tensor) may replace tensors."""
    from yalm_amd.weights import TensorSource, write_file, write_random_model
    folder = os.path.join(str(tmp), "%s_%d_%s" % (name, seed, str(stored).split(".")[-1]))
    if os.path.exists(os.path.join(folder, "model.safetensors")):
        return folder
    write_random_model(folder, cfg, seed=seed, dtype=torch.float32)
    src = TensorSource(folder)
    t = {n: src.get(n).clone() for n in src.names()}
    for n in t:
        if n.endswith(".lam"):
            t[n] = t[n] * 2.0 - 5.0
        if change is not None:
            t[n] = change(n, t[n])
    write_file(os.path.join(folder, "model.safetensors"), {n: v.to(stored).contiguous() for n, v in t.items()})
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("zebivik")
    return {(name, dt): make_folder(tmp, name, cfg, 5, helpers.torch_dtype(dt))
            for name, cfg in ZC.ALL.items() for dt in ("float32", "bfloat16")}


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
FAINT = 0.1                # a linear attention whose read-out is this small beside the layer's median: its norm divides by it


def check_request(got, folder, dtype, toks, what):
    """float32: every position within the tolerance.  bfloat16: the same, except that a position may differ more if a
    router choice at or before it in its request was a close call (the other expert is then as good an answer, and later
    positions read that token's keys and states) or a linear attention read next to nothing from its state.  Returns the
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
    """Between batches, when no sequence is alive, pages and states are filled with NaN, which must not reach a new sequence's
    logits: pages behind its length are never read, its states are cleared."""
    def before(step):
        if not engine.cache.slots.held:
            for g in engine.cache.kv_groups:
                g.k_pages.fill_(float("nan"))
                g.v_pages.fill_(float("nan"))
            for g in engine.cache.state_groups:
                g.data.fill_(float("nan"))
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


LENGTHS = {"mixed": [1, 2, 23, 64, 65, 150, 230], "medium": [300, 70, 131], "wide": [2, 100, 250], "odd": [1, 9, 10, 70, 129],
           "only_lru": [1, 2, 17, 140], "only_parallel": [3, 64, 65, 130], "only_state": [1, 2, 70], "one_side": [1, 2, 70]}
GROUPS = {"mixed": [([0, 2, 4, 5], [1, 23, 60, 100]), ([6, 1, 3], [221, 2, 64]), ([5, 4], [2, 1])],
          "medium": [([0, 1, 2], [250, 3, 100]), ([2, 1], [1, 64])],
          "wide": [([0, 1, 2], [2, 60, 222]), ([2, 1], [1, 99])],
          "odd": [([0, 1, 2, 3], [1, 3, 10, 64]), ([4, 3], [100, 1])],
          "only_lru": [([0, 1, 2, 3], [1, 1, 9, 100]), ([3, 2], [1, 16])],
          "only_parallel": [([0, 1, 2], [2, 63, 64]), ([3, 1], [100, 1])], "only_state": [([0, 1, 2], [1, 1, 40]), ([2, 1], [69, 1])],
          "one_side": [([0, 1, 2], [1, 1, 40]), ([2, 1], [69, 1])]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LENGTHS))
def test_whole_prompts(folders, name, dtype):
    requests = requests_for(ZC.ALL[name], LENGTHS[name])
    compare(folders, name, dtype, schedules.whole(requests), requests, engine_for(folders, name, dtype), "whole prompts")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(LENGTHS))
def test_last_tokens_one_by_one(folders, name, dtype):
    requests = requests_for(ZC.ALL[name], LENGTHS[name], seed=1)
    compare(folders, name, dtype, schedules.tail_one_by_one(requests, tail=80), requests, engine_for(folders, name, dtype),
            "last 80 tokens one by one")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["mixed", "medium", "odd", "only_lru"])
def test_token_by_token_from_the_first(folders, name, dtype):
    requests = requests_for(ZC.ALL[name], [150], seed=2)
    compare(folders, name, dtype, schedules.tail_one_by_one(requests, tail=10 ** 6), requests, engine_for(folders, name, dtype),
            "token by token")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(GROUPS))
def test_unequal_batches_with_reuse(folders, name, dtype):
    """Batches of unequal requests one after another and overlapping in time, in a cache with room for little more than
    one batch: slots, pages, recurrent states and convolution inputs are given back and taken again."""
    base = requests_for(ZC.ALL[name], LENGTHS[name], seed=3)
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
    """Decode batches beyond 16, 64 and 128 rows take other product kernels, another form of the recurrence and other graph
    buckets."""
    g = np.random.default_rng(n_requests)
    lengths = [int(n) for n in g.integers(1, 14, size=n_requests)]
    lengths[0], lengths[1] = 30, 26
    requests = requests_for(ZC.ALL[name], lengths, seed=6)
    firsts = {rid: max(1, len(t) - int(g.integers(0, 6))) for rid, t in requests.items()}
    steps = schedules.batches(requests, [list(requests)], firsts)
    compare(folders, name, dtype, steps, requests, engine_for(folders, name, dtype, max_tokens=n_requests * 64 + 64), "many requests")


@pytest.mark.parametrize("name", ["mixed", "medium"])
def test_without_graphs_and_on_the_float32_arithmetic_kernels(folders, name, monkeypatch):
    """The same logits from decode steps launched kernel by kernel, and from the kernels of the 32-bit path on bfloat16
    storage."""
    from yalm_amd.ops import kernels
    requests = requests_for(ZC.ALL[name], [90, 20], seed=7)
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
    folder = make_folder(tmp_path, name + "_changed", ZC.ALL[name], 7, helpers.torch_dtype(dtype), change=change)
    return folder, Engine(Model.from_folder(folder, dtype=helpers.torch_dtype(dtype), device=DEV), max_tokens=1024)


@pytest.mark.parametrize("name,n", [("only_parallel", 449), ("wide", 300), ("mixed", 300)])
def test_sharp_attention_over_hundreds_of_keys(tmp_path, name, n):
    """The queries scaled up: attention is nearly one-hot on single keys among hundreds, so that a key lost far back, at a page's
    border or among the first tokens shows in float32's tolerance."""
    folder, engine = changed_engine(tmp_path, name, "float32", lambda k, v: v * 9.0 if ".left.q" in k else v)
    toks = requests_for(ZC.ALL[name], [n], seed=9)["r0"]
    want, _ = plain_result(folder, toks)
    for decode_from in (None, n - 160):
        err = np.abs(logits_of(engine, toks, decode_from) - want).max(axis=1)
        bad = np.nonzero(err > 3 * helpers.F32_TOL * max(1.0, np.abs(want).max()))[0]
        assert not len(bad), "first wrong position %d (error %.3g)" % (bad[0], err[bad[0]])


@pytest.mark.parametrize("decode_from", [None, 20, 66])
def test_every_earlier_key_is_seen_and_no_later_one(tmp_path, decode_from):
    """One mixer whose linear attention gives nothing: changing ONE token changes the logits of every position from it on, and of none
    before it."""
    def change(k, v):
        return torch.zeros_like(v) if k.endswith(".right.o") else v
    _, engine = changed_engine(tmp_path, "one_side", "float32", change)
    toks = requests_for(ZC.ONE_SIDE, [70], seed=8)["r0"]
    base = logits_of(engine, toks, decode_from)
    for j in (0, 1, 19, 63, 64, 65, 69):
        other = list(toks)
        other[j] = (other[j] + 1) % ZC.ONE_SIDE["vocab"]
        moved = np.abs(logits_of(engine, other, decode_from) - base).max(axis=1) > 1e-7
        assert not moved[:j].any() and moved[j:].mean() > 0.95, (j, np.nonzero(moved)[0].tolist())


@pytest.mark.parametrize("decode_from", [None, 2, 150])
@pytest.mark.parametrize("name", ["only_state", "one_side"])
def test_the_recurrent_states_carry_the_first_token(tmp_path, name, decode_from):
    """One recurrence under decays close to one and nothing else that reaches back: the engine agrees with the plain recurrence over
    300 positions, through a prompt, through decoding and through both, and another first token moves the last logits as it
    does there."""
    def change(k, v):
        if k.endswith(".left.o"):
            return torch.zeros_like(v)
        if k.endswith(".lam"):
            return torch.full_like(v, -9.5)
        return v * 30.0 if k.endswith(".mix.o") or k.endswith(".right.o") else v
    folder, engine = changed_engine(tmp_path, name, "float32", change)
    toks = requests_for(ZC.ALL[name], [300], seed=10)["r0"]
    other = [(toks[0] + 1) % ZC.ALL[name]["vocab"]] + toks[1:]
    got, want = ([f(t) for t in (toks, other)] for f in (lambda t: logits_of(engine, t, decode_from), lambda t: plain_result(folder, t)[0]))
    assert np.abs(got[0] - want[0]).max() <= helpers.F32_TOL * max(1.0, np.abs(want[0]).max())
    moved, should = got[1][299] - got[0][299], want[1][299] - want[0][299]
    assert np.abs(should).max() > 3e-5 and np.abs(moved - should).max() <= 0.1 * np.abs(should).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decode_from", [None, 1, 2, 3, 12])
def test_the_convolution_sees_the_token_before_across_a_step(tmp_path, decode_from, dtype):
    """A recurrent block that forgets at once (rates of thousands): a token sees its predecessor through the convolution's two taps
    alone.  Changing token j moves the logits of j and j + 1 and of no other position, wherever the prompt ended."""
    folder, engine = changed_engine(tmp_path, "only_state", dtype, lambda k, v: torch.full_like(v, 3000.0) if k.endswith(".lam") else v)
    toks = requests_for(ZC.ONLY_STATE, [20], seed=15)["r0"]
    base = logits_of(engine, toks, decode_from)
    want, _ = plain_result(folder, toks)
    tol = helpers.F32_TOL if dtype == "float32" else helpers.BF16_MAX_TOL
    assert np.abs(base - want).max() <= tol * max(1.0, np.abs(want).max())
    for j in (0, 1, 2, 3, 11, 12, 19):
        other = list(toks)
        other[j] = (other[j] + 1) % ZC.ONLY_STATE["vocab"]
        moved = np.abs(logits_of(engine, other, decode_from) - base).max(axis=1) > 1e-6
        assert (moved == np.array([j <= i <= j + 1 for i in range(20)])).all(), (j, np.nonzero(moved)[0].tolist())


@pytest.mark.parametrize("part", [".left.g", ".left.o.b", ".left.v.b", ".right.g", ".right.norm", ".conv.b", ".x.b", ".y.b", ".ra.b", ".ri.b",
                                  ".norm1b.alpha", ".norm2.b", ".mlp.correction"])
def test_small_tensors_count(tmp_path, part):
    """Each scaled up to where leaving it out would show: the engine still agrees with the plain implementation."""
    folder, engine = changed_engine(tmp_path, "mixed", "float32", lambda k, v: v * 4.0 if k.endswith(part) else v)
    toks = requests_for(ZC.MIXED, [70], seed=16)["r0"]
    want, _ = plain_result(folder, toks)
    cfg, w = R.read_folder(folder)
    less = {k: (v * 0.25 if k.endswith(part) else v) for k, v in w.items()}
    assert np.abs(P.forward(cfg, less, toks).float().numpy() - want).max() > 10 * helpers.F32_TOL
    for decode_from in (None, 40):
        assert np.abs(logits_of(engine, toks, decode_from) - want).max() <= helpers.F32_TOL * max(1.0, np.abs(want).max())


def test_long_decoding(folders):
    """400 tokens one by one after a short prompt: the recurrent states are read and written 400 times, seven pages fill."""
    requests = requests_for(ZC.MIXED, [410], seed=11)
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
    toks = requests_for(ZC.ODD, [50], seed=13)["r0"]
    want, _ = plain_result(folders[("odd", "float32")], toks)
    s = engine.start(1)
    probs = engine.step(s, [toks[:-1]], [list(range(49))], targets=[toks[1:]]).cpu().numpy()
    engine.release(s)
    ref = torch.softmax(torch.tensor(want[:-1], dtype=F64), dim=-1).numpy()[np.arange(49), toks[1:]]
    assert np.allclose(probs, ref, rtol=2e-3, atol=1e-6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_runner(folders, tmp_path, dtype):
    requests = requests_for(ZC.MIXED, [1, 30, 90], seed=14)
    steps = schedules.batches(requests, [list(requests)], {"r0": 1, "r1": 12, "r2": 70})
    out = schedules.replay_trace_run(folders[("mixed", dtype)], dtype, steps, str(tmp_path / "out"),
                                     schedules.max_tokens_needed(steps))
    got = schedules.per_request(steps, out, requests)
    differ = sum(check_request(got[rid], folders[("mixed", dtype)], dtype, toks, "trace_run %s %s" % (dtype, rid))
                 for rid, toks in requests.items())
    assert differ <= 12


# ------------------------------------------------------------------------------------------ configurations drawn at random
def random_config(seed):
    """A Zebivik configuration whose every size, count, constant and the order of its layers are drawn from `seed`."""
    g = np.random.default_rng(seed)
    pick = lambda lo, hi: int(g.integers(lo, hi + 1))
    width = pick(17, 150)
    layers = []
    for i in range(pick(2, 6)):
        if g.random() < 0.5:
            nb = pick(1, 6)
            mixer = ZC.rglru(nb * pick(1, 40), nb, pick(1, 6))
        else:
            kv, dim = pick(1, 3), pick(2, 80)
            scaling = (float(g.uniform(1.5, 10)), float(g.uniform(0.5, 2)), float(g.uniform(2.5, 6)), pick(16, 400)) if g.random() < 0.6 else None
            left = ZC.attention(kv * pick(1, 4), kv, dim, pick(2, 140), float(g.uniform(0.05, 0.4)), dims=2 * pick(0, dim // 2),
                                base=float(10.0 ** g.uniform(1, 6)), scaling=scaling)
            right = ZC.lightning(pick(1, 140), pick(1, 90), *[float(1.0 - 10.0 ** g.uniform(-4, 0)) for _ in range(pick(1, 5))])
            mixer = ZC.side(left, right, float(g.uniform(0.5, 1.5)), float(g.uniform(0.5, 1.5)))
        groups = pick(1, 4)
        per = pick(1, 5)
        keep = pick(1, groups)
        kind = g.random()
        mlp = None if kind < 0.15 else ZC.dense(pick(3, 150), float(g.uniform(0.3, 4.0))) if kind < 0.45 else ZC.moe(
            groups * per, pick(1, keep * per), pick(3, 100), float(g.uniform(0.5, 3.0)), (groups, keep) if g.random() < 0.8 else None,
            shared=pick(3, 100) if g.random() < 0.7 else None)
        if mlp is not None and mlp["kind"] == "moe" and "groups" not in mlp["router"]:
            mlp["router"]["top"] = pick(1, groups * per)
        layers.append(ZC.layer(mixer, mlp))
    return ZC.model(pick(30, 400), width, float(10.0 ** g.uniform(-7, -4)), float(g.uniform(0.2, 1.5)), layers,
                    float(g.uniform(5.0, 50.0)) if g.random() < 0.8 else None)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [31, 32, 33, 34, 35, 36, 37, 38, 39, 40])
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
