"""The ops behind the Daberax blocks, each alone, against the float64 oracle in
daberax_oracle.py.  CPU parametrisation: the torch execution path; `gpu`: the
HIP kernels in fp32 and bf16 storage.

Where random inputs would hide a fault they are constructed: one score that
stands out just inside and just outside a window, at page borders, at the
query itself and one past it; a key that comes back so that its write must
correct the held value; decays that shut in the middle of a chunk; stale
content in reused slots and cache rows.
"""

import math

import pytest
import torch

from llm_instance_gateway_amd import ops
from llm_instance_gateway_amd.models.hybrid_blocks import (
    GatedDeltaMixer, GatedMLP, LatentAttention, NormedRotaryAttention, TokenTableGate,
)

import daberax_oracle as O

F64 = torch.float64
DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
CASES = [("cpu", torch.float32), pytest.param("cuda:0", torch.float32, marks=pytest.mark.gpu),
         pytest.param("cuda:0", torch.bfloat16, marks=pytest.mark.gpu)]


def rnd(g, *shape, s=1.0):
    return torch.randn(*shape, generator=g) * s


def close(got, want, dtype, scale=None, tol32=2e-5, tol16=2e-2):
    want = want.to(F64)
    ref = max(want.abs().max().item(), 1e-30) if scale is None else scale
    err = (got.detach().double().cpu() - want).abs().max().item() / ref
    assert err < (tol32 if dtype == torch.float32 else tol16), err


def i32(v, dev):
    return torch.tensor(v, dtype=torch.int32, device=dev)


# -- residual step, activations, frequencies ----------------------------------------------

@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("H", [7, 40, 50, 1032, 4096])
def test_normed_output_joins_the_residual(device, dtype, H):
    """x += rms(y) * w in fp32, and the sum rounded to the storage type: not a
    norm of the sum, and not a sum of rounded terms."""
    g = torch.Generator().manual_seed(H)
    R, eps = 5, 1e-2
    x, y = rnd(g, R, H, s=40.0), rnd(g, R, H, s=0.3).to(dtype)
    w = (1 + 0.3 * rnd(g, H)).to(dtype)
    xs = x.clone().to(device)
    h = ops.post_add_pre_norm(xs, y.to(device), w.to(device), None, eps, 1, rounded=True)
    want = x.to(F64) + O.unit_rms(y.to(F64), eps) * w.to(F64)
    assert h.dtype == dtype and xs.dtype == torch.float32
    close(xs, want, torch.float32, tol32=1e-6)
    assert torch.equal(h.float(), xs.to(dtype).float())
    wf = (1 + 0.3 * rnd(g, H)).to(dtype)
    hn = ops.post_add_pre_norm(xs, y.to(device), w.to(device), wf.to(device), eps, 1)
    want = want + O.unit_rms(y.to(F64), eps) * w.to(F64)
    close(hn, O.unit_rms(want, eps) * wf.to(F64), dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("F_", [12, 7])
def test_gated_gelu_feed_forward(device, dtype, F_):
    g = torch.Generator().manual_seed(F_)
    x = rnd(g, 9, 2 * F_, s=3.0).to(dtype)
    xd = x.to(F64)
    close(ops.glu_act(x.to(device), "gelu_tanh"), O.gelu_tanh(xd[:, :F_]) * xd[:, F_:], dtype, tol32=1e-6)
    mlp = GatedMLP(16, F_, "gelu_tanh", device=device, dtype=dtype)
    W = {"gate": rnd(g, F_, 16, s=0.5), "up": rnd(g, F_, 16, s=0.5), "down": rnd(g, 16, F_, s=0.5)}
    W = {k: v.to(dtype) for k, v in W.items()}
    mlp.load(lambda n: W[n].to(device), "")
    h = rnd(g, 5, 16, s=2.0).to(dtype)
    close(mlp(h.to(device)), O.gated_ff(h.to(F64), {k: v.to(F64) for k, v in W.items()}, ""), dtype)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("dim", [8, 3])
def test_token_table_gate(device, dtype, dim):
    """The layer's own columns of the table, the tanh form of gelu."""
    g = torch.Generator().manual_seed(dim)
    H, V, L, eps = 24, 11, 3, 1e-4
    W = {"side.embed": rnd(g, V, dim * L)}
    for i in range(L):
        W.update({f"l{i}.side.gate": rnd(g, dim, H, s=0.5), f"l{i}.side.proj": rnd(g, H, dim), f"l{i}.side.norm": 1 + 0.2 * rnd(g, H)})
    W = {k: v.to(dtype) for k, v in W.items()}
    x, toks = rnd(g, 6, H, s=2.0).to(dtype), torch.tensor([4, 0, 10, 4, 7, 1])
    Wd = {k: v.to(F64) for k, v in W.items()}
    table = W["side.embed"].to(device)
    for i in range(L):
        side = TokenTableGate(H, dim, device, dtype)
        side.load(lambda n: W[n].to(device), f"l{i}.side.")
        y = side(x.to(device), table[:, i * dim : (i + 1) * dim], toks.to(device))
        res = torch.zeros(6, H, device=device)
        ops.post_add_pre_norm(res, y.contiguous(), side.norm, None, eps, 1)
        close(res, O.token_side(x.to(F64), toks, Wd, i, dim, eps), dtype, tol16=4e-2)


def test_banded_frequency_scaling_has_three_bands():
    rot = {"base": 10000.0, "dims": 32, "scaling": {"factor": 6.0, "low": 1.5, "high": 5.0, "original": 700.0}}
    got = ops.rotary_inv_freq(rot["base"], rot["dims"], "cpu", scaling=rot["scaling"])
    want = torch.tensor(O.frequencies(rot), dtype=F64)
    plain = torch.tensor(O.frequencies(dict(rot, scaling=None)), dtype=F64)
    kept, slowed = want == plain, (want - plain / 6.0).abs() < 1e-15
    assert kept.sum() >= 3 and slowed.sum() >= 3 and (~kept & ~slowed).sum() >= 2
    assert ((got.double() - want) / want).abs().max() < 1e-7


# -- batches over scattered pages and slots ----------------------------------------------------

def batch(device, bs, tables, parts, slots=None, tiles=True):
    """parts: [(sequence, tokens before, tokens now)], prompt portions first."""
    pos, slot, tok_seq, start, qsl, ts, tq = [], [], [], [], [0], [], []
    pre = [p for p in parts if p[2] > 1]
    assert parts[: len(pre)] == pre, "portions come before single tokens"
    for i, (s, done, n) in enumerate(parts):
        start.append(len(pos))
        for p in range(done, done + n):
            pos.append(p)
            slot.append(tables[s][p // bs] * bs + p % bs)
            tok_seq.append(i)
        if n > 1:
            qsl.append(qsl[-1] + n)
            for qb in range(0, n, 64):
                ts.append(i)
                tq.append(qb)
    width = max(len(t) for t in tables.values())
    bt = i32([tables[s] + [0] * (width - len(tables[s])) for s, _, _ in parts], device)

    class Meta:
        num_prefill_tokens, num_decode_tokens = qsl[-1], len(parts) - len(pre)
        slot_mapping = torch.tensor(slot, device=device)
        seq_block_tables = bt
        seg_start, seg_len = i32(start, device), i32([n for _, _, n in parts], device)
        seg_ctx = i32([d + n for _, d, n in parts], device)
        seg_fresh = i32([int(d == 0) for _, d, _ in parts], device)
        seg_slot = i32([(slots or {s: s for s, _, _ in parts})[s] for s, _, _ in parts], device)
        max_seg_len = max(n for _, _, n in parts)
        prefill_block_tables = bt[: len(pre)].contiguous()
        prefill_query_start_locs = i32(qsl, device)
        prefill_context_lens = i32([d + n for _, d, n in pre], device)
        prefill_tile_seq = i32(ts, device) if tiles and pre else None
        prefill_tile_qstart = i32(tq, device) if tiles and pre else None

    Meta.tok_seq = i32(tok_seq, device)
    return Meta, torch.tensor(pos, device=device)


def in_steps(layer, h, caches, device, bs, tables, steps, slots=None):
    """Feed the sequences h {s: [T, hidden]} through `layer` step by step;
    steps: lists of (sequence, tokens).  Returns {s: outputs}."""
    at = {s: 0 for s in h}
    got = {s: [] for s in h}
    for step in steps:
        parts = [(s, at[s], n) for s, n in step]
        meta, pos = batch(device, bs, tables, parts, slots)
        x = torch.cat([h[s][d : d + n] for s, d, n in parts]).to(device)
        y = layer(x, pos, caches, meta).float().cpu()
        r = 0
        for s, d, n in parts:
            got[s].append(y[r : r + n])
            r += n
            at[s] += n
    return {s: torch.cat(v) for s, v in got.items() if v}


# -- short convolution ----------------------------------------------------------------------------

CUTS = [[147], [20, 2, 1, 64, 60], [2] * 10 + [127], [1] * 60 + [87], [64, 64, 19], [130, 17], [3, 2, 2, 140]]


def plans_for(cuts, other):
    """Sequence 0 in `cuts`; sequence 1 joins with portions of two tokens."""
    return [[(0, n)] + ([(1, 2)] if i * 2 < other else []) for i, n in enumerate(cuts)]


def run_plans(device, plans, slots, step):
    """step(rows, segments) -> [R, *] for rows [(sequence, t)]; collects per sequence."""
    at, got = {}, {}
    for plan in plans:
        start, ln, fresh, rows = [], [], [], []
        for s, n in plan:
            start.append(sum(ln)); ln.append(n); fresh.append(int(at.get(s, 0) == 0))
            rows += [(s, t) for t in range(at.get(s, 0), at.get(s, 0) + n)]
            at[s] = at.get(s, 0) + n
        seg = (i32(start, device), i32(ln, device), i32([slots[s] for s, _ in plan], device), i32(fresh, device))
        o = step(rows, seg, max(ln)).cpu()
        for (s, n), r0 in zip(plan, start):
            got.setdefault(s, []).append(o[r0 : r0 + n])
    return {s: torch.cat(v) for s, v in got.items()}


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("taps,C", [(4, 24), (4, 13), (2, 8), (3, 2056), (1, 16), (7, 40), (20, 9)])
def test_short_convolution(device, dtype, taps, C):
    """Portions shorter than the filter, slots full of another sequence's
    inputs, a column block of wider rows, two sequences per launch."""
    g = torch.Generator().manual_seed(taps * 100 + C)
    T = {0: 147, 1: 12}
    w = rnd(g, C, taps).to(dtype)
    x = {s: rnd(g, n, C + 8).to(dtype) for s, n in T.items()}
    want = {s: O.silu(O.causal_conv(x[s][:, :C].to(F64), w.to(F64))) for s in T}
    wd = w.t().contiguous().to(device)
    for cuts in CUTS:
        state = torch.full((4, (taps - 1) * C), 9.0, device=device)

        def step(rows, seg, longest):
            fused = torch.stack([x[s][t] for s, t in rows]).to(device)
            return ops.short_conv_silu(fused[:, :C], wd, state, *seg, longest)

        got = run_plans(device, plans_for(cuts, 12), {0: 2, 1: 0}, step)
        for s in got:
            close(got[s], want[s][: got[s].shape[0]], dtype, scale=want[s].abs().max().item(), tol16=1e-2)
        if taps > 1:  # the slots hold the last inputs, oldest first; others are untouched
            n = got[1].shape[0]
            last = torch.cat([torch.zeros(taps, C), x[1][:n, :C].float()])[-(taps - 1):]
            assert torch.equal(state[0].view(taps - 1, C).cpu(), last)
            assert torch.all(state[1] == 9.0) and torch.all(state[3] == 9.0)


# -- gated delta rule --------------------------------------------------------------------------------

def delta_case(kind, g, n, heads, kv, dim, vdim):
    """(q | k | v rows, write logits, decay logits) of one sequence."""
    q, k, v = rnd(g, n, kv * dim), rnd(g, n, kv * dim), rnd(g, n, heads * vdim)
    b, a = rnd(g, n, heads), rnd(g, n, heads)
    if kind == "again":     # few keys that come back: every write must correct
        base = rnd(g, 3, kv * dim)
        k = base[torch.arange(n) % 3] + 0.02 * k
        b, a = b + 4.0, a - 9.0
    elif kind == "shut":    # now and then nearly everything is forgotten, in mid-chunk
        a = a - 6.0
        a[::7] = 60.0
        a[40:45] = 300.0
    elif kind == "far":     # one early token dominates what follows
        a, b = a - 11.0, b - 3.0
        v[3] *= 60.0
        b[3] = 8.0
        k[30::11] = k[3] + 0.3 * k[30::11]
    elif kind == "tiny":    # rows near zero: the unit norm's epsilon rules
        q, k = q * 3e-4, k * 3e-4
        k[::5] = 0.0
    return torch.cat([q, k, v], dim=1), b, a


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("kind", ["plain", "again", "shut", "far", "tiny"])
@pytest.mark.parametrize("heads,kv,dim,vdim", [(4, 2, 16, 24), (3, 1, 40, 72), (2, 2, 64, 128), (1, 1, 128, 40),
                                                (3, 3, 5, 7), (2, 1, 136, 200), (2, 1, 256, 8), (1, 1, 1, 1)])
def test_gated_delta_scan(device, dtype, kind, heads, kv, dim, vdim):
    g = torch.Generator().manual_seed(heads * 1000 + dim)
    T, nq = {0: 147, 1: 12}, kv * dim
    rate, bias = (rnd(g, heads) * 0.5), rnd(g, heads)
    data, gates, want = {}, {}, {}
    eye = torch.eye(heads, dtype=F64)
    for s, n in T.items():
        x, b, a = delta_case(kind, g, n, heads, kv, dim, vdim)
        data[s], gates[s] = x.to(dtype), torch.cat([b, a], dim=1)
        xd = data[s].to(F64)
        q, k = (O.unit_length(t.reshape(n, kv, dim)).repeat_interleave(heads // kv, dim=1)
                for t in (xd[:, :nq], xd[:, nq : 2 * nq]))
        W = {"b": eye, "a": eye, "A_log": rate.to(F64), "dt_bias": bias.to(F64)}
        dec, _ = O.delta_gates(a.to(F64), W, "")
        _, beta = O.delta_gates(b.to(F64), W, "")
        want[s] = O.delta_recurrence(q * dim ** -0.5, k, xd[:, 2 * nq :].reshape(n, heads, vdim), dec, beta)[0].reshape(n, -1)
    if kind == "again":  # without the correction the state would pile up
        assert want[0].abs().max() < 0.5 * data[0].abs().max().double() * math.sqrt(T[0])
    for cuts in CUTS:
        state = torch.full((3, ops.matrix_state_width(heads, dim, vdim)), 5.0, device=device)

        def step(rows, seg, longest):
            fused = torch.stack([data[s][t] for s, t in rows]).to(device)
            z = torch.stack([torch.cat([torch.zeros(3), gates[s][t]]) for s, t in rows]).to(device)
            o = ops.gated_delta_scan(
                fused[:, :nq], fused[:, nq : 2 * nq], fused[:, 2 * nq :], (z[:, 3 : 3 + heads], z[:, 3 + heads :]),
                rate.to(device), bias.to(device), state, *seg, heads, kv, dim, vdim, q_scale=dim ** -0.5,
                max_seg_len=longest)
            assert o.dtype == torch.float32
            return o

        got = run_plans(device, plans_for(cuts, 12), {0: 2, 1: 0}, step)
        assert torch.all(state[1] == 5.0)
        for s in got:
            # bf16 storage: products of exact bf16 numbers and fp32 split in two halves
            close(got[s], want[s][: got[s].shape[0]], dtype, scale=want[s].abs().max().item(), tol32=3e-5, tol16=3e-4)


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("heads,kv,dim,vdim,taps", [(4, 2, 16, 24, 4), (3, 3, 10, 6, 2), (2, 1, 64, 64, 1)])
def test_delta_mixer(device, dtype, heads, kv, dim, vdim, taps):
    g = torch.Generator().manual_seed(dim)
    hidden, eps = 40, 1e-3
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps}
    mix = GatedDeltaMixer(hidden, heads, kv, dim, vdim, taps, eps, device=device, dtype=dtype)
    W = {"A_log": 0.5 * rnd(g, heads), "dt_bias": rnd(g, heads) - 3, "norm": 1 + 0.2 * rnd(g, vdim),
         "o": rnd(g, hidden, heads * vdim, s=0.2)}
    for n, r in (("q", kv * dim), ("k", kv * dim), ("v", heads * vdim)):
        W[n], W[n + ".conv"] = rnd(g, r, hidden, s=hidden ** -0.5), rnd(g, r, taps, s=0.7)
    W["g"], W["b"], W["a"] = rnd(g, heads * vdim, hidden, s=0.2), rnd(g, heads, hidden, s=0.2), rnd(g, heads, hidden, s=0.2)
    W = {k: v.to(dtype) for k, v in W.items()}
    mix.load(lambda n: W[n].to(device), "")
    Wd = {k: v.to(F64) for k, v in W.items()}
    h = {0: rnd(g, 90, hidden).to(dtype), 1: rnd(g, 23, hidden).to(dtype)}
    want = {s: O.delta(h[s].to(F64), Wd, "", m, eps) for s in h}
    caches = tuple(torch.full((4, c["width"]), 7.0, device=device) for c in mix.cache_spec())
    steps = [[(0, 33), (1, 2)], [(1, 17), (0, 1)], [(0, 2), (1, 3)], [(0, 53), (1, 1)], [(0, 1)]]
    got = in_steps(mix, h, caches, device, 16, {0: [0] * 8, 1: [0] * 8}, steps, slots={0: 3, 1: 1})
    for s in h:
        close(got[s], want[s], dtype, tol32=1e-4, tol16=4e-2)


# -- soft-capped windowed attention -------------------------------------------------------------------

def paged(k, v, bs, table, kc, vc):
    for t in range(k.shape[0]):
        kc[table[t // bs], :, t % bs] = k[t].to(kc.dtype)
        vc[table[t // bs], :, t % bs] = v[t].to(vc.dtype)


def planted(g, T, H, G, D, Dv, dtype, plant, boost):
    """Random q, k, v with, for every (query, key) in `plant`, both pushed
    along one axis so that their score stands out."""
    q, k, v = rnd(g, T, H, D, s=0.3), rnd(g, T, G, D, s=0.3), rnd(g, T, G, Dv)
    for qi, kj in plant:
        if 0 <= kj < T:
            q[qi, :, (qi + kj) % D] += boost
            k[kj, :, (qi + kj) % D] += boost
    return q.to(dtype), k.to(dtype), v.to(dtype)


def edges(rows, w):
    """Oldest key a window keeps, the one just outside, the query, one past it."""
    return [(r, j) for r in rows for j in (r - w + 1, r - w, r, r + 1)]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("window,cap", [(1, 3.0), (7, 5.0), (16, 2.0), (50, 20.0), (64, 4.0), (65, 0.0), (0, 3.0), (1000, 6.0)])
def test_softcapped_attention_rows(device, dtype, window, cap):
    g = torch.Generator().manual_seed(3)
    T, H, G, D, Dv, bs, scale = 150, 4, 2, 12, 6, 16, 0.5
    rows = [149, 148, 130, 128, 127, 112, 100, 80, 65, 64, 63, 49, 48, 16, 15, 7, 6, 1, 0]
    q, k, v = planted(g, T, H, G, D, Dv, dtype, edges(rows, window) + [(149, 2), (130, 0), (100, 17)], 4.0)
    kc = torch.full((12, G, bs, D), 7.0, dtype=dtype, device=device)
    vc = torch.full((12, G, bs, Dv), -7.0, dtype=dtype, device=device)
    table = [9, 2, 7, 0, 5, 11, 3, 8, 1, 10]
    paged(k, v, bs, table, kc, vc)
    gate = rnd(g, T, H, s=2.0).to(dtype)
    want = O.window_attention(q.to(F64), k.to(F64), v.to(F64), scale, window, cap)
    if cap:  # the cap must matter here
        bare = O.window_attention(q.to(F64), k.to(F64), v.to(F64), scale, window)
        assert window == 1 or (bare - want).abs().max() > 0.02
    want = want * torch.sigmoid(gate.to(F64))[:, :, None]
    got = ops.paged_attention_general(
        q[rows].reshape(len(rows), H * D).to(device), kc, vc, i32([[0] * 10, table], device),
        i32([1] * (len(rows) - 1) + [-1], device), torch.tensor(rows, device=device), scale, H, window=window,
        softcap=cap, gate=gate[rows].to(device), gate_per_head=True)
    close(got[:-1], want[rows[:-1]].reshape(len(rows) - 1, H * Dv), dtype, scale=want.abs().max().item())
    assert torch.all(got[-1] == 0)  # a row of no sequence


@pytest.mark.gpu
@pytest.mark.parametrize("window,cap,D,Dv", [(1, 4.0, 32, 16), (50, 20.0, 32, 16), (64, 3.0, 96, 32), (33, 8.0, 24, 40),
                                             (200, 2.0, 64, 64), (0, 5.0, 128, 128)])
def test_softcapped_attention_prompt_tiles(window, cap, D, Dv):
    """The MFMA prompt kernel: a whole prompt, a portion that starts inside a
    sequence and a short one in one launch."""
    dev, dtype = "cuda:0", torch.bfloat16
    g = torch.Generator().manual_seed(4)
    H, G, bs, scale = 4, 2, 16, 0.4
    ctx, done = {0: 230, 1: 200, 2: 40}, {0: 0, 1: 90, 2: 37}
    kc = torch.full((40, G, bs, D), 7.0, dtype=dtype, device=dev)
    vc = torch.full((40, G, bs, Dv), -7.0, dtype=dtype, device=dev)
    tables, qs, gs, wants, at = {}, [], [], [], 0
    for s, n in ctx.items():
        d0 = done[s]
        rows = [n - 1, d0, d0 + 1, min(d0 + 63, n - 1), min(d0 + 64, n - 1), (d0 + n) // 2]
        q, k, v = planted(g, n, H, G, D, Dv, dtype, edges(rows, window) + [(n - 1, 1), (n - 1, d0)], 4.0)
        nb = (n + bs - 1) // bs
        tables[s] = list(range(at, at + nb))[::-1]
        at += nb
        paged(k, v, bs, tables[s], kc, vc)
        gate = rnd(g, n, H, s=2.0).to(dtype)
        want = O.window_attention(q.to(F64), k.to(F64), v.to(F64), scale, window, cap) * torch.sigmoid(gate.to(F64))[:, :, None]
        qs.append(q[d0:].reshape(n - d0, H * D)); gs.append(gate[d0:]); wants.append(want[d0:].reshape(n - d0, H * Dv))
    meta, _ = batch(dev, bs, tables, [(s, done[s], ctx[s] - done[s]) for s in ctx])
    got = ops.paged_attention_prefill_tiles(
        torch.cat(qs).to(dev), kc, vc, meta.prefill_block_tables, meta.prefill_query_start_locs,
        meta.prefill_context_lens, meta.prefill_tile_seq, meta.prefill_tile_qstart, scale, H, window=window,
        softcap=cap, gate=torch.cat(gs).to(dev), gate_per_head=True)
    close(got, torch.cat(wants), dtype)


STEPS = [[(0, 60), (1, 20)], [(1, 7), (0, 1)], [(0, 2)], [(0, 1), (1, 1)], [(0, 70), (1, 1)], [(0, 16)]]


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("heads,kv,dim,vdim,rot,window", [(6, 2, 12, 10, 8, 9), (4, 4, 32, 16, 32, 48), (2, 1, 16, 16, 0, 1),
                                                          (3, 1, 64, 64, 20, 500)])
def test_attention_block(device, dtype, heads, kv, dim, vdim, rot, window):
    """Biases, norms over the whole projection, banded rotation, cap, window
    and head gates together, over scattered pages of a used cache."""
    g = torch.Generator().manual_seed(dim)
    hidden, eps, bs = 40, 1e-3, 8
    rc = {"base": 300.0, "dims": rot, "scaling": {"factor": 3.0, "low": 1.0, "high": 4.0, "original": 60.0}}
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": 1.3 * dim ** -0.5, "softcap": 2.5,
         "mask": {"size": window}, "rot": rc}
    blk = NormedRotaryAttention(
        hidden, heads, kv, dim, vdim, m["scale"], eps, qk_norm="row", rot_base=rc["base"], rot_dims=rot,
        rot_layout="interleaved", rot_scaling=rc["scaling"], window=window, bias=True, head_gate=True, softcap=2.5,
        device=device, dtype=dtype)
    W = {}
    for n, r in (("q", heads * dim), ("k", kv * dim), ("v", kv * vdim)):
        W[n], W[n + ".b"] = rnd(g, r, hidden, s=0.3), rnd(g, r)
    W["q.norm"], W["k.norm"] = 1 + 0.3 * rnd(g, heads * dim), 1 + 0.3 * rnd(g, kv * dim)
    W["g"], W["o"], W["o.b"] = rnd(g, heads, hidden, s=0.5), rnd(g, hidden, heads * vdim, s=0.3), rnd(g, hidden)
    W = {k: v.to(dtype) for k, v in W.items()}
    blk.load(lambda n: W[n].to(device), "")
    h = {0: rnd(g, 150, hidden).to(dtype), 1: rnd(g, 29, hidden).to(dtype)}
    Wd = {k: v.to(F64) for k, v in W.items()}
    want = {s: O.attention(h[s].to(F64), Wd, "", m, eps) for s in h}
    caches = (torch.full((24, kv, bs, dim), 3.0, dtype=dtype, device=device),
              torch.full((24, kv, bs, vdim), -3.0, dtype=dtype, device=device))
    perm = torch.randperm(24, generator=g).tolist()
    got = in_steps(blk, h, caches, device, bs, {0: perm[:19], 1: perm[19:23]}, STEPS)
    for s in h:
        close(got[s], want[s], dtype, tol32=5e-5, tol16=4e-2)


# -- windowed latent attention ---------------------------------------------------------------------------

@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("heads,dim,rot,vdim,rank,window", [(3, 16, 8, 24, 40, 9), (2, 5, 4, 3, 7, 1), (5, 32, 16, 32, 96, 64),
                                                            (1, 8, 8, 8, 64, 33), (4, 8, 8, 16, 24, 1000)])
def test_windowed_latent_attention(device, dtype, heads, dim, rot, vdim, rank, window):
    g = torch.Generator().manual_seed(rank)
    hidden, eps, bs = 40, 1e-4, 8
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": 0.3,
         "rot": {"base": 30.0, "dims": rot}, "mask": {"size": window}}
    blk = LatentAttention(hidden, heads, dim, rot, vdim, 0, rank, 0.3, 30.0, rot, eps, sink=False, out_gate=False,
                          window=window, device=device, dtype=dtype)
    W = {"q": rnd(g, heads * (dim + rot), hidden, s=0.3), "dkv": rnd(g, rank + rot, hidden, s=0.3),
         "dkv.norm": 1 + 0.2 * rnd(g, rank), "uk": rnd(g, heads * dim, rank, s=0.3),
         "uv": rnd(g, heads * vdim, rank, s=0.3), "o": rnd(g, hidden, heads * vdim, s=0.3)}
    W = {k: v.to(dtype) for k, v in W.items()}
    blk.load(lambda n: W[n].to(device), "")
    h = {0: rnd(g, 150, hidden).to(dtype), 1: rnd(g, 29, hidden).to(dtype)}
    Wd = {k: v.to(F64) for k, v in W.items()}
    want = {s: O.latent_attention(h[s].to(F64), Wd, "", m, eps) for s in h}
    cache = (torch.full((24, 1, bs, rank + rot), 3.0, dtype=dtype, device=device),)
    perm = torch.randperm(24, generator=g).tolist()
    got = in_steps(blk, h, cache, device, bs, {0: perm[:19], 1: perm[19:23]}, STEPS)
    for s in h:
        close(got[s], want[s], dtype, tol32=5e-5, tol16=4e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("nsplit", [1, 3, 0])
@pytest.mark.parametrize("window", [1, 16, 31, 32, 100, 0])
@pytest.mark.parametrize("H,row,Dv", [(3, 80, 64), (20, 40, 24), (16, 576, 512)])
def test_windowed_latent_rows_kernel(H, row, Dv, window, nsplit):
    """The MFMA row kernel alone: single tokens, portions that start inside a
    sequence, one shorter than its tile; for every edge row a key just inside
    and one just outside its window dominates."""
    g = torch.Generator().manual_seed(9)
    bs, dev, dtype = 16, "cuda:0", torch.bfloat16
    ctx, now = {0: 70, 1: 150, 2: 90, 3: 600}, {0: 70, 1: 33, 2: 1, 3: 1}
    qs, wants, tables, at = [], [], {}, 0
    cache = torch.full((64, 1, bs, row), 3.0, dtype=dtype, device=dev)
    for s, n in ctx.items():
        d0 = n - now[s]
        edge_rows = sorted({n - 1, d0, (d0 + n) // 2})
        q, k = rnd(g, n, H, row, s=0.2), rnd(g, n, row, s=0.5)
        for r, j in edges(edge_rows, window) + [(n - 1, 1)]:
            if 0 <= j < n:
                q[r, :, (r + j) % row] += 5.0
                k[j, (r + j) % row] += 5.0
        q, k = q.to(dtype), k.to(dtype)
        nb = (n + bs - 1) // bs
        tables[s] = list(range(at, at + nb))[::-1]
        at += nb
        for t in range(n):
            cache[tables[s][t // bs], 0, t % bs] = k[t].to(dev)
        kd = k.to(F64)[:, None, :]
        w = torch.zeros(now[s], H, Dv, dtype=F64)
        for i, p in enumerate(range(d0, n)):
            lo = max(0, p - window + 1) if window else 0
            sc = torch.einsum("hd,jd->hj", q[p].to(F64), kd[lo : p + 1, 0]) * 0.4
            w[i] = torch.softmax(sc, dim=-1) @ kd[lo : p + 1, 0, :Dv]
        qs.append(q[d0:].reshape(now[s], H * row))
        wants.append(w.reshape(now[s], H * Dv))
    meta, _ = batch(dev, bs, tables, [(s, ctx[s] - now[s], now[s]) for s in ctx])
    got = ops.latent_attention_rows(
        torch.cat(qs).to(dev), cache, Dv, meta.seq_block_tables, meta.seg_start, meta.seg_len, meta.seg_ctx, 70, 0.4, H,
        nsplit=nsplit, window=window)
    close(got, torch.cat(wants), dtype)
