"""Daberax through the engine (scheduler, block/state pools, model runner,
kernels) against the slow float64 oracle in daberax_oracle.py.

Every test builds its own small configuration and random bf16 checkpoint in a
temp folder, so the config reader and the safetensors loader are on the path
too.  The CPU parametrisation runs the engine's torch execution path; the
`gpu` one runs the HIP kernels (fp32 storage for sharp comparisons, bf16 for
the serving precision).
"""

import json
import math
import struct

import pytest
import torch

from llm_instance_gateway_amd.engine import EngineConfig, LLMEngine, SamplingParams
from llm_instance_gateway_amd.models.config import get_model_config

import daberax_oracle as O

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
CASES = [("cpu", torch.float32), pytest.param("cuda:0", torch.float32, marks=pytest.mark.gpu),
         pytest.param("cuda:0", torch.bfloat16, marks=pytest.mark.gpu)]


def dense(ff):
    return {"kind": "dense", "ff": ff}


def lat(heads, dim, rot_dim, vdim, rank, window, mlp=None, base=500.0, scale=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {
        "heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "mask": {"size": window},
        "rot": {"base": base, "dims": rot_dim}, "scale": scale if scale is not None else 1.2 / math.sqrt(dim + rot_dim)}}


def att(heads, kv, dim, vdim, window, cap, mlp=None, rot=None, base=3000.0, scale=None, bands=(4.0, 1.0, 4.0, 128)):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "mask": {"size": window}, "softcap": cap,
         "rot": {"base": base, "dims": dim if rot is None else rot},
         "scale": scale if scale is not None else 1.1 / math.sqrt(dim)}
    if bands:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), bands))
    return {"type": "attention", "mixer": m, "mlp": mlp}


def dlt(heads, kv, dim, vdim, taps, mlp=None):
    return {"type": "delta", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps}}


def config(vocab, width, layers, eps=1e-5, scale=0.7, side=8):
    return {"architecture": "Daberax", "vocab": vocab, "width": width, "layers": layers,
            "norm": {"eps": eps}, "logit_scale": scale, "token_side": {"dim": side}}


# sizes unlike one another; windows that are no multiple of a page; a layer
# without feed-forward; partly rotated heads; filters of other lengths
CFG_A = config(61, 48, [
    dlt(6, 2, 10, 14, 3, dense(40)),
    att(6, 3, 12, 20, 21, 6.0, dense(56), rot=8),
    lat(3, 8, 6, 12, 18, 33, dense(24)),
    dlt(2, 1, 24, 8, 5, None),
    att(4, 1, 8, 8, 7, 2.5, None, bands=None),
    lat(5, 16, 4, 8, 10, 50, dense(40), base=20.0, scale=0.4),
    dlt(3, 3, 6, 70, 2, dense(32)),
])
# degenerate values: one head, windows of one and of more than any prompt,
# sizes that are multiples of nothing, a filter of one tap (no inputs to
# carry), scales of exactly one, a side table of one entry
CFG_B = config(31, 18, [
    dlt(1, 1, 5, 3, 1, dense(7)), att(1, 1, 6, 5, 1, 1.0, dense(1), rot=2, scale=1.0, bands=(1.0, 1.0, 2.0, 10)),
    lat(1, 5, 2, 3, 7, 1000, None), lat(2, 3, 2, 1, 1, 1, dense(3), scale=1.0), dlt(2, 1, 1, 1, 2, None),
], eps=1e-2, scale=1.0, side=1)
# head sizes and cache rows of the MFMA kernels
CFG_C = config(40, 64, [
    dlt(4, 2, 32, 48, 4, dense(96)), att(4, 2, 32, 24, 40, 12.0, dense(64)), lat(4, 32, 16, 32, 48, 65, dense(48)),
    dlt(2, 2, 64, 136, 3, dense(96)),
], side=16)
# no recurrent layer, no side table
CFG_D = config(33, 32, [att(2, 2, 8, 16, 9, 4.0, dense(24)), lat(2, 8, 8, 8, 24, 12, None)], side=0)
del CFG_D["token_side"]


def make_checkpoint(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    H, V, dim = cfg["width"], cfg["vocab"], cfg.get("token_side", {}).get("dim", 0)

    def r(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(torch.bfloat16)

    def near1(n):
        return (1 + 0.2 * torch.randn(n, generator=g)).to(torch.bfloat16)

    W = {"embed": r(V, H), "final.norm": near1(H), "head": r(V, H, s=H ** -0.5)}
    if dim:
        W["side.embed"] = r(V, dim * len(cfg["layers"]))
    for i, layer in enumerate(cfg["layers"]):
        p, m = "l%d." % i, layer["mixer"]
        hd, D, Dv = m["heads"], m["dim"], m["vdim"]
        W[p + "norm1"] = near1(H)
        if layer["type"] == "latent_attention":
            R, Rk = m["rot_dim"], m["kv_rank"]
            W[p + "mix.q"] = r(hd * (D + R), H, s=H ** -0.5)
            W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = r(Rk + R, H, s=H ** -0.5), near1(Rk)
            W[p + "mix.uk"], W[p + "mix.uv"] = r(hd * D, Rk, s=Rk ** -0.5), r(hd * Dv, Rk, s=Rk ** -0.5)
        elif layer["type"] == "attention":
            G = m["kv_heads"]
            for n, rows in (("q", hd * D), ("k", G * D), ("v", G * Dv)):
                W[p + "mix." + n], W[p + "mix." + n + ".b"] = r(rows, H, s=H ** -0.5), r(rows, s=0.3)
            W[p + "mix.q.norm"], W[p + "mix.k.norm"] = 1.5 * near1(hd * D), 1.5 * near1(G * D)
            W[p + "mix.g"], W[p + "mix.o.b"] = r(hd, H, s=H ** -0.5), r(H, s=0.3)
        else:
            G = m["kv_heads"]
            for n, rows in (("q", G * D), ("k", G * D), ("v", hd * Dv)):
                W[p + "mix." + n], W[p + "mix." + n + ".conv"] = r(rows, H, s=H ** -0.5), r(rows, m["conv"], s=0.7)
            W[p + "mix.g"], W[p + "mix.norm"] = r(hd * Dv, H, s=H ** -0.5), near1(Dv)
            W[p + "mix.b"], W[p + "mix.a"] = r(hd, H, s=H ** -0.5), r(hd, H, s=H ** -0.5)
            W[p + "mix.A_log"], W[p + "mix.dt_bias"] = r(hd, s=0.5), (r(hd) - 3).to(torch.bfloat16)
        W[p + "mix.o"] = r(H, hd * Dv, s=(hd * Dv) ** -0.5)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            W[p + "norm2"] = near1(H)
            W[p + "mlp.gate"], W[p + "mlp.up"] = r(ff, H, s=H ** -0.5), r(ff, H, s=H ** -0.5)
            W[p + "mlp.down"] = r(H, ff, s=ff ** -0.5)
        if dim:
            W[p + "side.gate"], W[p + "side.proj"], W[p + "side.norm"] = r(dim, H, s=H ** -0.5), r(H, dim), near1(H)
    return {k: v.to(torch.bfloat16) for k, v in W.items()}


def write_model(folder, cfg, W):
    folder.mkdir(parents=True, exist_ok=True)
    (folder / "config.json").write_text(json.dumps(cfg))
    header, blobs, at = {}, [], 0
    for name, t in W.items():
        raw = t.contiguous().view(torch.uint8).numpy().tobytes()
        header[name] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    hj = json.dumps(header).encode()
    with open(folder / "model.safetensors", "wb") as f:
        f.write(struct.pack("<Q", len(hj)) + hj + b"".join(blobs))
    return str(folder)


def make_engine(path, device, dtype=torch.float32, blocks=64, block_size=16, seqs=4, budget=4096, **kw):
    kw.setdefault("enforce_eager", True)
    cfg = EngineConfig(
        model=get_model_config(path), block_size=block_size, num_kv_blocks=blocks, max_num_seqs=seqs,
        num_state_slots=seqs, max_num_batched_tokens=budget, max_model_len=blocks * block_size,
        watermark_blocks=0, **kw,
    )
    return LLMEngine(cfg, device=device, dtype=dtype)


def row_errs(got, want):
    """Per-row RMS of the mean-free difference over the RMS of the oracle's logits."""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def assert_logits(got, want, dtype):
    """fp32: every row within rounding.  bf16: the norm on a small sub-layer
    output magnifies that output's rounding; plain torch operations in bf16
    bring single rows of these models to 0.1 - 0.3, with a median below 0.03."""
    e = row_errs(got, want)
    if dtype == torch.float32:
        assert e.max().item() < 3e-4, (e.max().item(), e.argmax().item())
    else:
        assert (e < 0.1).double().mean().item() >= 0.9 and e.median().item() < 4e-2, e


def tokens_for(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def replay_all(eng, rid, toks, cuts):
    """Feed toks in portions `cuts`, wanting every position; returns [T, V]."""
    rows, at = [], 0
    for i, n in enumerate(cuts):
        last = i == len(cuts) - 1
        res = eng.replay_step([(rid, toks[at : at + n], list(range(n)))], end=[rid] if last else [])
        rows.append(res[rid].float().cpu())
        at += n
    assert at == len(toks)
    return torch.cat(rows)


def _model(tmp_path_factory, cfg, seed, name):
    W = make_checkpoint(cfg, seed)
    return write_model(tmp_path_factory.mktemp("dbx") / name, cfg, W), W


@pytest.fixture(scope="module")
def model_a(tmp_path_factory):
    return _model(tmp_path_factory, CFG_A, 11, "a")


@pytest.fixture(scope="module")
def model_c(tmp_path_factory):
    return _model(tmp_path_factory, CFG_C, 13, "c")


@pytest.fixture(scope="module")
def oracle_a(model_a):
    toks = tokens_for(CFG_A, 90, 5)
    res = []
    return toks, O.forward(CFG_A, model_a[1], toks, residuals=res), res


def test_config_reader_and_cache_accounting(model_a):
    mc = get_model_config(model_a[0])
    assert mc.architecture == "daberax" and mc.logit_scale == 0.7 and mc.token_side_dim == 8 and not mc.is_moe
    assert mc.kv_elems_per_token() == 3 * (12 + 20) + (18 + 6) + (8 + 8) + (10 + 4)
    assert mc.state_elems_per_seq() == (
        6 * 10 * 14 + 2 * (2 * 20 + 84) + 2 * 24 * 8 + 4 * (2 * 24 + 16) + 3 * 6 * 70 + (2 * 18 + 210))
    eng = make_engine(model_a[0], "cpu")
    assert [len(c) for c in eng.runner.kv_caches] == [2, 2, 1, 2, 2, 1, 2]
    assert eng.runner.kv_caches[0][0].dtype == torch.float32 and eng.runner.kv_caches[0][0].shape == (5, 2 * 124)
    from llm_instance_gateway_amd.models.daberax import config_from_json
    for path, bad in ((("type",), "retention"), (("mlp", "kind"), "moe")):
        cfg = json.loads(json.dumps(CFG_A))
        at = cfg["layers"][0]
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = bad
        with pytest.raises(ValueError):
            config_from_json(cfg)


def test_checkpoint_with_missing_or_unknown_tensors(tmp_path):
    W = make_checkpoint(CFG_D, 3)
    for name, change in (("missing", lambda d: d.pop("l0.mix.g")), ("unknown", lambda d: d.update(extra=d["head"]))):
        broken = dict(W)
        change(broken)
        with pytest.raises((KeyError, ValueError)):
            make_engine(write_model(tmp_path / name, CFG_D, broken), "cpu")


@pytest.mark.parametrize("device,dtype", CASES)
def test_whole_prompt_and_every_layer(model_a, oracle_a, device, dtype):
    toks, want, want_res = oracle_a
    eng = make_engine(model_a[0], device, dtype)
    captured = eng.runner.model.capture_residuals = []
    assert_logits(replay_all(eng, "w", toks, [len(toks)]), want, dtype)
    assert len(captured) == len(CFG_A["layers"])
    for i, (x, xo) in enumerate(zip(captured, want_res)):
        assert x.dtype == torch.float32, "the residual stream stays fp32"
        e = (x[: len(toks)].double().cpu() - xo).abs().max(-1).values / xo.abs().max().item()
        assert e.max().item() < (1e-4 if dtype == torch.float32 else 8e-2), f"layer {i}: {e.max().item()}"


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("which", ["b", "d"])
def test_degenerate_sizes_and_padded_batches(tmp_path, device, which):
    cfg = CFG_B if which == "b" else CFG_D
    W = make_checkpoint(cfg, 14)
    path = write_model(tmp_path / which, cfg, W)
    toks = tokens_for(cfg, 40, 6)
    want = O.forward(cfg, W, toks)
    eng = make_engine(path, device, block_size=8)
    assert get_model_config(path).has_recurrent_state == (which == "b")
    assert row_errs(replay_all(eng, "d", toks, [17, 1, 1, 2, 19]), want).max().item() < 3e-4
    if which == "d":  # bf16 with padded batches, two requests side by side
        eng = make_engine(path, device, torch.bfloat16 if device != "cpu" else torch.float32)
        t2 = tokens_for(cfg, 21, 7)
        r1 = eng.replay_step([("x", toks[:30], list(range(30))), ("y", t2[:20], list(range(20)))])
        r2 = eng.replay_step([("x", toks[30:], list(range(10))), ("y", t2[20:], [0])], end=["x", "y"])
        assert row_errs(torch.cat([r1["x"], r2["x"]]).float(), want).max().item() < 8e-2
        assert row_errs(torch.cat([r1["y"], r2["y"]]).float(), O.forward(cfg, W, t2)).max().item() < 8e-2


@pytest.mark.parametrize("device", DEVICES)
def test_prefill_against_token_by_token(model_a, oracle_a, device):
    toks, want, _ = oracle_a
    for cuts, n in (([30] + [1] * 60, 90), ([1] * 40, 40), ([1], 1)):  # the last: the first token alone
        eng = make_engine(model_a[0], device)
        assert row_errs(replay_all(eng, "p", toks[:n], cuts), want[:n]).max().item() < 3e-4


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("cuts", [[2] * 45, [3, 13, 16, 17, 2, 31, 8], [15, 1, 16, 1, 32, 25], [64, 2, 24], [65, 25]])
def test_portions(model_a, oracle_a, device, cuts):
    toks, want, _ = oracle_a
    eng = make_engine(model_a[0], device)
    assert row_errs(replay_all(eng, "c", toks, cuts), want).max().item() < 3e-4


@pytest.mark.parametrize("device,dtype", CASES)
def test_mixed_batch_equals_each_alone_and_pools_are_reused(model_a, device, dtype):
    """Unequal requests share steps (portions beside single tokens), with a
    pool so small that pages and state slots of finished requests are handed
    to later ones; every logit row matches the request run alone."""
    lens = {"a": 37, "b": 5, "c": 50, "d": 1, "e": 23, "f": 33}
    toks = {k: tokens_for(CFG_A, n, 100 + i) for i, (k, n) in enumerate(lens.items())}
    want = {k: O.forward(CFG_A, model_a[1], t) for k, t in toks.items()}
    plan = [
        [("a", 20), ("b", 3)],
        [("a", 1), ("b", 2), ("c", 30), ("d", 1)],           # b, d end: slots free
        [("a", 16), ("e", 7)],                                # c sits this step out; e reuses a freed slot + pages
        [("c", 20), ("e", 1), ("f", 2)],                      # a ended; c comes back and ends
        [("e", 15), ("f", 30)],
        [("f", 1)],
    ]
    eng = make_engine(model_a[0], device, dtype, blocks=9, block_size=16, seqs=4)
    at = {k: 0 for k in toks}
    got = {k: [] for k in toks}
    for step in plan:
        entries, end = [], []
        for rid, n in step:
            entries.append((rid, toks[rid][at[rid] : at[rid] + n], list(range(n))))
            at[rid] += n
            if at[rid] == lens[rid]:
                end.append(rid)
        res = eng.replay_step(entries, end)
        for rid, _ in step:
            got[rid].append(res[rid].float().cpu())
    assert all(at[k] == lens[k] for k in lens)
    bm = eng.scheduler.block_manager
    assert bm.num_free_blocks == 9 and bm.num_free_state_slots == 4
    for k in toks:
        assert_logits(torch.cat(got[k]), want[k], dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_far_token_over_dirty_pages_and_slots(tmp_path, device):
    """An early token lies far outside every window, yet the delta layers'
    states carry it to the end of a 300-token prompt and 16 decoded tokens,
    after another request has dirtied every page and slot.  The model is made
    so that it shows: slow decays, and the oracle's logits without that token
    differ by far more than the bound."""
    cfg = config(61, 40, [
        dlt(2, 1, 16, 16, 4, None), lat(2, 16, 8, 16, 24, 30, dense(32), scale=0.6), dlt(2, 2, 16, 24, 3, dense(24)),
        att(2, 1, 16, 16, 18, 8.0, None),
    ])
    W = make_checkpoint(cfg, 31)
    for i in (0, 2):
        W[f"l{i}.mix.dt_bias"] -= 8.0   # nearly nothing is forgotten
        W[f"l{i}.mix.b"] *= 3.0
        W[f"l{i}.norm1"] *= 2.0
    key = 7
    toks = [t if t != key else 8 for t in tokens_for(cfg, 300, 31)]
    toks[4] = key
    W["embed"][key] *= 4.0
    path = write_model(tmp_path / "far", cfg, W)
    want = O.forward(cfg, W, toks)
    other = O.forward(cfg, W, toks[:4] + [9] + toks[5:])
    assert row_errs(other[-20:], want[-20:]).min().item() > 5e-3
    eng = make_engine(path, device, blocks=19, block_size=16, seqs=1)
    eng.replay_step([("junk", tokens_for(cfg, 304, 32), [])], end=["junk"])
    got = replay_all(eng, "x", toks, [250, 1, 1, 30, 2] + [1] * 16)
    assert row_errs(got, want).max().item() < 3e-4


@pytest.mark.parametrize("device,dtype", CASES)
@pytest.mark.parametrize("layer", ["attention", "latent"])
def test_window_edges_in_prompts_and_decoding(tmp_path, device, dtype, layer):
    """One layer with a window of 24 whose queries all look for one token; the
    rows where it stands just inside, and just outside, the window are checked
    in a prompt portion and decoded alone, and they differ by much more than
    the bound from what a window one token off would give."""
    w = 24
    one = att(2, 1, 16, 16, w, 10.0, None, scale=0.9) if layer == "attention" else lat(2, 16, 8, 16, 24, w, None, scale=0.9)
    cfg = config(61, 40, [one], side=0)
    del cfg["token_side"]
    W = make_checkpoint(cfg, 17)
    key = 7
    if layer == "attention":
        W["l0.mix.q.b"] += 4.0 * torch.sign(W["l0.mix.q.b"].float()).to(torch.bfloat16)
        bias = W["l0.mix.q.b"].float().view(2, 16).mean(0)  # what every query carries
        W["l0.mix.k"] = (W["l0.mix.k"].float() + torch.outer(bias, W["embed"][key].float()) * 0.05).to(torch.bfloat16)
    else:
        W["l0.mix.q"] *= 2.0
    W["embed"][key] *= 3.0
    W["l0.norm1"] *= 3.0
    path = write_model(tmp_path / "edge", cfg, W)
    toks = [t if t != key else 8 for t in tokens_for(cfg, 120, 5)]
    for at in (10, 47, 80):
        toks[at] = key
    want = O.forward(cfg, W, toks)
    for off in (-1, 1):
        moved = json.loads(json.dumps(cfg))
        moved["layers"][0]["mixer"]["mask"]["size"] = w + off
        d = row_errs(O.forward(moved, W, toks), want)
        at = w - 1 if off < 0 else w  # rows where only one of the two windows holds the token
        assert max(d[a + at].item() for a in (10, 47, 80)) > (2e-2 if dtype == torch.float32 else 0.12)
    for cuts in ([120], [30] + [1] * 90, [50, 20, 2, 1, 31, 2, 2, 12]):
        eng = make_engine(path, device, dtype, blocks=8)
        e = row_errs(replay_all(eng, "e", toks, cuts), want)
        assert e.max().item() < (3e-4 if dtype == torch.float32 else 5e-2), (cuts, e.max().item(), e.argmax().item())


def assert_greedy_follows_oracle(cfg, W, prompt, outputs, margin):
    """Teacher-forced on the engine's own outputs: every chosen token's
    oracle logit is within `margin` (in units of the logits' spread) of the
    oracle's best."""
    toks = list(prompt) + list(outputs)
    logits = O.forward(cfg, W, toks)
    for step, tok in enumerate(outputs):
        z = logits[len(prompt) + step - 1]
        gap = float(z.max() - z[tok]) / float(z.std())
        assert gap <= margin, (step, tok, gap)


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_scheduler(model_a, device):
    """add_request + generate_all: chunked prefill under a tiny token budget,
    continuous batching of three requests, one of them long."""
    prompts = [tokens_for(CFG_A, n, 200 + n) for n in (19, 7, 26)]
    eng = make_engine(model_a[0], device, budget=8, blocks=32)
    seqs = [eng.add_request(p, SamplingParams(max_new_tokens=n)) for p, n in zip(prompts, (6, 60, 6))]
    assert len(eng.generate_all(max_steps=300)) == 3
    for seq, prompt, n in zip(seqs, prompts, (6, 60, 6)):
        assert len(seq.output_token_ids) == n
        assert_greedy_follows_oracle(CFG_A, model_a[1], prompt, seq.output_token_ids, 2e-3)
    bm = eng.scheduler.block_manager
    assert bm.num_free_blocks == 32 and bm.num_free_state_slots == 4


@pytest.mark.parametrize("device", DEVICES)
def test_preempted_sequence_recomputes_its_state(model_a, device):
    prompt = tokens_for(CFG_A, 21, 77)
    ref = make_engine(model_a[0], device)
    s0 = ref.add_request(prompt, SamplingParams(max_new_tokens=8))
    ref.generate_all(max_steps=50)
    eng = make_engine(model_a[0], device)
    s1 = eng.add_request(prompt, SamplingParams(max_new_tokens=8))
    for _ in range(4):
        eng.step()
    sch = eng.scheduler
    sch.running.remove(s1)
    sch.block_manager.free(s1)
    s1.preempt()
    sch.waiting.appendleft(s1)
    assert s1.state_slot == -1
    eng.generate_all(max_steps=50)
    assert s1.output_token_ids == s0.output_token_ids


@pytest.mark.parametrize("device,dtype", CASES)
def test_sizes_of_the_mfma_kernels(model_c, device, dtype):
    ta, tb = tokens_for(CFG_C, 150, 41), tokens_for(CFG_C, 70, 42)
    wa, wb = O.forward(CFG_C, model_c[1], ta), O.forward(CFG_C, model_c[1], tb)
    eng = make_engine(model_c[0], device, dtype)
    if device != "cpu" and dtype == torch.bfloat16:
        model = eng.runner.model
        assert model.needs_prefill_tiles and model.layers[2].mixer.mfma_rows(dtype, True)
    got = {"a": [], "b": []}
    # a: 100-token portion (two 64-row tiles, the second partial), then single
    # tokens; b joins with portions beside a's single tokens
    plan = [[("a", 100)], [("a", 1), ("b", 65)], [("a", 30), ("b", 1)], [("a", 1), ("b", 4)], [("a", 18)]]
    at, toks = {"a": 0, "b": 0}, {"a": ta, "b": tb}
    for step in plan:
        entries = []
        for rid, n in step:
            entries.append((rid, toks[rid][at[rid] : at[rid] + n], list(range(n))))
            at[rid] += n
        res = eng.replay_step(entries, [r for r, _ in step if at[r] == len(toks[r])])
        for rid, _ in step:
            got[rid].append(res[rid].float().cpu())
    assert_logits(torch.cat(got["a"]), wa, dtype)
    assert_logits(torch.cat(got["b"]), wb, dtype)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("which", ["a", "c"])
def test_decode_graphs_replay_like_eager(model_a, model_c, dtype, which):
    """Decode-only steps replay captured hipGraphs (static per-sequence
    tables, state slots filled per step).  Many replays with eager prefill
    steps of later requests in between; every generated token is checked."""
    path, W = model_a if which == "a" else model_c
    cfg = CFG_A if which == "a" else CFG_C
    eng = make_engine(path, "cuda:0", dtype, budget=32, enforce_eager=False)
    prompts = [tokens_for(cfg, n, 300 + n) for n in (9, 40, 17)]
    seqs = [eng.add_request(prompts[0], SamplingParams(max_new_tokens=14))]
    for _ in range(5):
        eng.step()                      # prefill, then graph replays at batch 1
    seqs.append(eng.add_request(prompts[1], SamplingParams(max_new_tokens=9)))
    for _ in range(4):
        eng.step()                      # chunked eager prefill beside the decode
    seqs.append(eng.add_request(prompts[2], SamplingParams(max_new_tokens=11)))
    eng.generate_all(max_steps=100)
    assert eng.runner.graph_runner is not None and eng.runner.graph_runner.graphs
    margin = 1e-3 if dtype == torch.float32 else 0.4
    for seq, prompt in zip(seqs, prompts):
        assert seq.is_finished()
        assert_greedy_follows_oracle(cfg, W, prompt, seq.output_token_ids, margin)


@pytest.mark.gpu
def test_an_engine_captures_while_a_dropped_one_awaits_collection(model_c):
    """Graphs of a dropped engine must not be destroyed inside another
    engine's capture, however eagerly the collector runs."""
    import gc

    path, _ = model_c
    prompt = tokens_for(CFG_C, 9, 1)
    outs = []
    before = gc.get_threshold()
    gc.set_threshold(5, 1, 1)
    try:
        for _ in range(2):
            gc.disable()  # the dropped engine's cycles stay until the next capture
            eng = make_engine(path, "cuda:0", torch.bfloat16, enforce_eager=False)
            gc.enable()
            seq = eng.add_request(prompt, SamplingParams(max_new_tokens=4))
            eng.generate_all(max_steps=20)
            assert eng.runner.graph_runner.graphs and gc.isenabled()
            outs.append(seq.output_token_ids)
            gc.disable()
            del eng, seq
    finally:
        gc.enable()
        gc.set_threshold(*before)
    assert outs[0] == outs[1]


def test_served_through_the_pool_and_front_door(tmp_path):
    """A model folder as the pool's base model: worker process, router, HTTP
    front door, greedy completion from prompt token ids."""
    from starlette.testclient import TestClient

    from llm_instance_gateway_amd.api.types import InferenceModel
    from llm_instance_gateway_amd.serving import EnginePool, build_app

    cfg = dict(CFG_A, vocab=300)
    W = make_checkpoint(cfg, 21)
    path = write_model(tmp_path / "served", cfg, W)
    pool = EnginePool(
        path, devices=["cpu"],
        engine_kwargs=dict(num_kv_blocks=64, max_num_seqs=4, max_num_batched_tokens=64, max_model_len=256),
    )
    pool.start()
    try:
        pool.datastore.store_model(InferenceModel(model_name="delta"))
        client = TestClient(build_app(pool))
        prompt = tokens_for(cfg, 23, 8)
        r = client.post("/v1/completions", json={"model": "delta", "prompt": prompt, "max_tokens": 5})
        assert r.status_code == 200, r.text
        out = r.json()["choices"][0]["token_ids"]
        assert len(out) == 5
        assert_greedy_follows_oracle(cfg, W, prompt, out, margin=0.3)  # workers run bf16
    finally:
        pool.stop()
