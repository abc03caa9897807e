#!/usr/bin/env python3
"""Daberax beside Garesun and Potatar at equal size: prefill and decode
throughput through the engine, and the new kernels beside the like kernels of
those paths against the roofline.

    python bench.py --delta                 # both parts, JSON lines
    python benchmarks/bench_delta.py --part engine|kernels|profile [--sizes s,m]

The closest existing family is Garesun: matrix recurrences and latent
attention in one stack, with a token table per layer.  Its feed-forward is
routed; Potatar has a dense one, matrix recurrences (wkv) and chunked softmax
attention, so both stand beside Daberax.

Engine part, per size: a Daberax stack (latent attention, two delta layers,
soft-capped attention; twice), a Garesun stack as in bench_recurrent.py and a
Potatar stack (attention, three wkv layers; twice) with the same width, depth
and active feed-forward parameters.  The same workload goes through
LLMEngine.step(): N prompts of L tokens in budget-sized steps, then K decode
steps (hipGraph replay) at batch N.  Random weights, synthetic tokens.

Kernel part: each new kernel or kernel mode and its counterpart, timed with
events at the layer shapes of the sizes above; bytes that must move / time
against 8 TB/s, attention in useful TFLOP/s.
"""

from __future__ import annotations

import argparse
import json
import math
import os
import sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))

from llm_instance_gateway_amd import ops
from llm_instance_gateway_amd.models.config import ModelConfig
from llm_instance_gateway_amd.models.daberax import make_config
from llm_instance_gateway_amd.models.potatar import make_config as potatar_make

import bench_recurrent
from bench_hybrid import HBM_BYTES_PER_S, engine_run, timeit

# delta heads (value, query/key) x key/value sizes; attention heads, key/value
# heads, size; latent attention and side table as in bench_recurrent.SIZES
SIZES = {
    "s": dict(width=2048, layers=8, delta=(32, 16, 128, 128), conv=4, att=(16, 4, 128), window=512, cap=30.0,
              heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, ff=4096, side=128, vocab=32000),
    "m": dict(width=4096, layers=8, delta=(64, 32, 128, 128), conv=4, att=(32, 8, 128), window=512, cap=30.0,
              heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, ff=7168, side=256, vocab=32000),
}


def daberax_config(name: str, z: dict) -> ModelConfig:
    mlp = {"kind": "dense", "ff": z["ff"]}
    hv, hk, dk, dv = z["delta"]
    ha, ga, da = z["att"]
    layers = []
    for i in range(z["layers"]):
        if i % 4 == 0:
            layers.append({"type": "latent_attention", "mlp": mlp, "mixer": {
                "heads": z["heads"], "dim": z["dim"], "rot_dim": z["rot_dim"], "vdim": z["vdim"],
                "kv_rank": z["kv_rank"], "mask": {"size": z["window"]},
                "rot": {"base": 500000.0, "dims": z["rot_dim"]}, "scale": 1.0 / math.sqrt(z["dim"] + z["rot_dim"])}})
        elif i % 4 == 3:
            layers.append({"type": "attention", "mlp": mlp, "mixer": {
                "heads": ha, "kv_heads": ga, "dim": da, "vdim": da, "mask": {"size": z["window"]}, "softcap": z["cap"],
                "rot": {"base": 500000.0, "dims": da,
                        "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}},
                "scale": 1.0 / math.sqrt(da)}})
        else:
            layers.append({"type": "delta", "mlp": mlp, "mixer": {
                "heads": hv, "kv_heads": hk, "dim": dk, "vdim": dv, "conv": z["conv"]}})
    return make_config(f"daberax-{name}", z["vocab"], z["width"], layers, logit_scale=0.5, side_dim=z["side"])


def potatar_config(name: str, z: dict) -> ModelConfig:
    ha, ga, da = z["att"]
    mlp = {"ff": 3 * z["ff"] // 2, "kind": "dense"}
    att = {"type": "attention", "mlp": mlp, "mixer": {
        "heads": ha, "kv_heads": ga, "dim": da, "vdim": da, "mask": {"size": z["window"]}, "scale": 1.0 / math.sqrt(da),
        "rot": {"base": 500000.0, "dims": da}}}
    wkv = {"type": "wkv", "mlp": mlp, "mixer": {"heads": z["width"] // 64, "dim": 64, "decay_rank": 64}}
    return potatar_make(f"potatar-{name}", z["vocab"], z["width"],
                        [dict(att if i % 4 == 0 else wkv) for i in range(z["layers"])], alpha=2.0)


def part_engine(sizes) -> None:
    for name in sizes:
        z = SIZES[name]
        zg = bench_recurrent.SIZES[name]
        for n_seqs, plen in ((16, 1024), (64, 512)):
            row = {"bench": "engine", "size": name, **z, "seqs": n_seqs, "prompt_len": plen, "decode_steps": 64}
            row["daberax"] = engine_run(daberax_config(name, z), n_seqs, plen, 64)
            row["garesun"] = engine_run(bench_recurrent.garesun_config(name, zg), n_seqs, plen, 64)
            row["potatar"] = engine_run(potatar_config(name, z), n_seqs, plen, 64)
            for k in ("prefill_tok_per_s", "decode_tok_per_s"):
                for other in ("garesun", "potatar"):
                    row[f"vs_{other}_{k}"] = round(row["daberax"][k] / row[other][k], 3)
            print(json.dumps(row), flush=True)


def part_kernels(sizes) -> None:
    dev, bf = "cuda:0", torch.bfloat16
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)
    for name in sizes:
        z, zg = SIZES[name], bench_recurrent.SIZES[name]
        W, FF = z["width"], z["ff"]
        for T in (8192, 256):  # a prefill step's rows / a decode batch
            rows = []

            def add(kernel, like, t, nbytes):
                rows.append({"kernel": kernel, "like": like, "us": round(t * 1e6, 2),
                             "GB_per_s": round(nbytes / t / 1e9, 1),
                             "of_roofline": round(nbytes / t / HBM_BYTES_PER_S, 3)})

            # -- residual step, activations ------------------------------------------------------
            x32 = torch.randn(T, W, device=dev)
            y = torch.randn(T, W, device=dev, dtype=bf)
            w = torch.ones(W, device=dev, dtype=bf)
            add("post_add_pre_norm, rounded sum", "",
                timeit(lambda: ops.post_add_pre_norm(x32, y, w, None, 1e-5, 1, rounded=True)), T * W * 12)
            add("add_layer_norm (Garesun)", "residual step",
                timeit(lambda: ops.add_layer_norm(x32, w, 1e-5, y, w)), T * W * 12)
            add("scaled_add_rms_norm (Potatar)", "residual step",
                timeit(lambda: ops.scaled_add_rms_norm(x32, 2.0, w, 1e-6, y)), T * W * 12)
            gu = torch.randn(T, 2 * FF, device=dev, dtype=bf)
            add("glu_act, gelu_tanh", "", timeit(lambda: ops.glu_act(gu, "gelu_tanh")), T * FF * 6)
            add("glu_act, relu (Vemenex)", "gelu_tanh", timeit(lambda: ops.glu_act(gu, "relu")), T * FF * 6)
            del gu
            # -- segments: prompts of 1024 / single tokens ----------------------------------------
            seg = 1024 if T >= 1024 else 1
            S = T // seg
            segs = (i32([i * seg for i in range(S)]), i32([seg] * S), i32(list(range(S))), i32([0] * S))
            hv, hk, dk, dv = z["delta"]
            nk, nv = hk * dk, hv * dv
            C = 2 * nk + nv
            proj = torch.randn(T, C + nv, device=dev, dtype=bf)
            wc = torch.randn(z["conv"], C, device=dev, dtype=bf) * 0.5
            st = torch.zeros(S + 1, (z["conv"] - 1) * C, device=dev)
            state_io = S * (z["conv"] - 1) * C * 8
            add(f"short_conv_silu ({z['conv']} taps, {C} channels)", "",
                timeit(lambda: ops.short_conv_silu(proj[:, :C], wc, st, *segs, seg)), T * C * 4 + state_io)
            del st
            tok_seq = i32([i // seg for i in range(T)])
            mu = torch.rand(5, W, device=dev).to(bf)
            sh = torch.zeros(S + 1, W, device=dev)
            add("token_shift_mix (Potatar, 5 blends)", "short_conv_silu",
                timeit(lambda: ops.token_shift_mix(x32, mu, sh, tok_seq, *segs)), T * W * (4 + 10) + S * W * 8)

            # -- matrix recurrences: q, k, v in (2B), output (4B); the state both ways ----------------
            def scan_bytes(h, hq, d, v, ones=0):
                return T * (2 * hq * d * 2 + h * v * 6) + 2 * S * h * d * (v + ones) * 4

            qkv = torch.randn(T, C, device=dev, dtype=bf)
            q, k, v = qkv[:, :nk], qkv[:, nk : 2 * nk], qkv[:, 2 * nk :]
            ba = torch.randn(T, 2 * hv, device=dev)
            rate, bias = torch.zeros(hv, device=dev), torch.full((hv,), -4.0, device=dev)
            state = torch.zeros(S + 1, ops.matrix_state_width(hv, dk, dv), device=dev)
            add(f"gated_delta_scan ({hv} heads {dk} x {dv}, {hk} q/k heads)", "",
                timeit(lambda: ops.gated_delta_scan(q, k, v, (ba[:, :hv], ba[:, hv:]), rate, bias, state, *segs, hv, hk,
                                                    dk, dv, q_scale=dk ** -0.5, max_seg_len=seg), 10),
                scan_bytes(hv, hk, dk, dv))
            qq = torch.randn(T, 2 * hv * dk + nv, device=dev, dtype=bf)
            dec = torch.full((hv,), 0.99, device=dev)
            add("matrix_state_scan, constant decay, the same heads", "gated_delta_scan",
                timeit(lambda: ops.matrix_state_scan(qq[:, : hv * dk], qq[:, hv * dk : 2 * hv * dk], qq[:, 2 * hv * dk :],
                                                     state, *segs, hv, dk, dv, head_decay=dec, max_seg_len=seg), 10),
                scan_bytes(hv, hv, dk, dv))
            del qq, state
            hr, dr, vr = zg["ret"]
            pos = torch.arange(T, device=dev, dtype=torch.int64) % 1024
            cs = ops.rotary_table(pos, ops.rotary_inv_freq(10000.0, dr, dev))
            decr = torch.full((hr,), 0.99, device=dev)
            pr = torch.randn(T, hr * (2 * dr + vr), device=dev, dtype=bf)
            state = torch.zeros(S + 1, ops.matrix_state_width(hr, dr, vr), device=dev)
            add(f"matrix_state_scan, retention (Garesun, {hr} heads {dr} x {vr}, rotated)", "gated_delta_scan",
                timeit(lambda: ops.matrix_state_scan(pr[:, : hr * dr], pr[:, hr * dr : 2 * hr * dr], pr[:, 2 * hr * dr :],
                                                     state, *segs, hr, dr, vr, head_decay=decr, rot=cs, k_scale=0.1,
                                                     max_seg_len=seg), 10), scan_bytes(hr, hr, dr, vr))
            del pr, state
            hm, dm, vm = zg["mls"]
            pm = torch.randn(T, hm * (2 * dm + vm), device=dev, dtype=bf)
            zz = torch.randn(T, 2 * hm, device=dev)
            bi, bfg = torch.full((hm,), -1.0, device=dev), torch.full((hm,), 4.0, device=dev)
            state = torch.zeros(S + 1, ops.matrix_state_width(hm, dm, vm, True), device=dev)
            add(f"matrix_state_scan, mLSTM (Garesun, {hm} heads {dm} x {vm})", "gated_delta_scan",
                timeit(lambda: ops.matrix_state_scan(pm[:, : hm * dm], pm[:, hm * dm : 2 * hm * dm], pm[:, 2 * hm * dm :],
                                                     state, *segs, hm, dm, vm, gates=(zz[:, :hm], zz[:, hm:]),
                                                     gate_bias=(bi, bfg), gate_cap=15.0, q_scale=0.1, max_seg_len=seg), 10),
                scan_bytes(hm, hm, dm, vm, 1))
            del pm, state
            o = torch.randn(T, nv, device=dev)
            wn = torch.ones(nv, device=dev, dtype=bf)
            add(f"group_rms_norm_gate (groups of {dv})", "",
                timeit(lambda: ops.group_rms_norm_gate(o, proj[:, C:], wn, dv, "silu", 1e-5)), T * nv * 8)
            add(f"group_rms_norm_gate (Garesun, groups of {vr})", "groups of " + str(dv),
                timeit(lambda: ops.group_rms_norm_gate(o, proj[:, C:], None, vr, "silu", 1e-5)), T * nv * 8)
            del o, proj, qkv

            # -- attention: 1024 tokens per sequence, window of the model ------------------------------
            bs, L, win = 16, 1024, z["window"]
            nb = L // bs
            ha, ga, da = z["att"]
            SQ = S
            tables = torch.arange(SQ * nb, dtype=torch.int32, device=dev).view(SQ, nb)
            kc = torch.randn(SQ * nb + 1, ga, bs, da, device=dev, dtype=bf)
            vc = torch.randn_like(kc)
            pa = torch.randn(T, (ha + 2 * ga) * da + ha, device=dev, dtype=bf)
            wq, wk = torch.ones(ha * da, device=dev, dtype=bf), torch.ones(ga * da, device=dev, dtype=bf)
            inv = ops.rotary_inv_freq(500000.0, da, dev)
            slots = torch.randperm(SQ * L, device=dev)[:T].to(torch.int64)
            qkv_b = T * (ha + 2 * ga) * da * 4
            for lay in ("interleaved", "half"):
                add(f"qkv_norm_rope_cache (row norms, {lay})", "" if lay == "interleaved" else "the same, Potatar's layout",
                    timeit(lambda: ops.qkv_norm_rope_cache(pa, ha, ga, da, da, "row", wq, wk, 1e-5, inv, pos, kc, vc, slots,
                                                           rot_layout=lay)), qkv_b)
            qa = torch.randn(T, ha * da, device=dev, dtype=bf)
            gate = pa[:, -ha:]
            sc = 1.0 / math.sqrt(da)
            kw = dict(window=win, gate=gate, gate_per_head=True)
            seen = min(win, L)
            if T >= 1024:
                ts = i32([s for s in range(S) for _ in range(L // 64)])
                tq = i32([qb for _ in range(S) for qb in range(0, L, 64)])
                args = (qa, kc, vc, tables, i32([i * L for i in range(S + 1)]), i32([L] * S), ts, tq, sc, ha)
                pairs = S * ha * (seen * (seen + 1) / 2 + (L - seen) * seen)
                for what, extra in (("soft cap", dict(softcap=z["cap"])), ("no cap", {})):
                    t = timeit(lambda: ops.paged_attention_prefill_tiles(*args, **kw, **extra), 10)
                    rows.append({"kernel": f"paged_attention_prefill_tiles (window, {what})", "like": "",
                                 "us": round(t * 1e6, 1), "TFLOP_per_s": round(4 * da * pairs / t / 1e12, 1)})
            else:
                ts, ps = i32(list(range(T))), torch.full((T,), L - 1, device=dev, dtype=torch.int64)
                args = (qa, kc, vc, tables, ts, ps, sc, ha)
                for what, extra in (("soft cap", dict(softcap=z["cap"])), ("no cap", {})):
                    add(f"paged_attention_general (single tokens, window, {what})", "",
                        timeit(lambda: ops.paged_attention_general(*args, **kw, **extra), 10), T * seen * ga * da * 4)
            del kc, vc, pa, qa
            # -- latent attention ---------------------------------------------------------------------------
            hq, Rk, row = z["heads"], z["kv_rank"], z["kv_rank"] + z["rot_dim"]
            lc = torch.randn(SQ * nb + 1, 1, bs, row, device=dev, dtype=bf)
            ql = torch.randn(T, hq * row, device=dev, dtype=bf)
            n1 = L if T >= 1024 else 1
            args = (ql, lc, Rk, tables, segs[0], segs[1], i32([L] * S), n1, sc, hq)
            for what, wn_ in (("window", win), ("causal, Garesun", 0)):
                s_ = min(wn_, L) if wn_ else L
                if T >= 1024:
                    t = timeit(lambda: ops.latent_attention_rows(*args, window=wn_), 5)
                    pairs = S * hq * (s_ * (s_ + 1) / 2 + (L - s_) * s_)
                    rows.append({"kernel": f"latent_attention_rows ({what})", "like": "", "us": round(t * 1e6, 1),
                                 "TFLOP_per_s": round(2 * (row + Rk) * pairs / t / 1e12, 1)})
                else:
                    add(f"latent_attention_rows (single tokens, {what})", "",
                        timeit(lambda: ops.latent_attention_rows(*args, window=wn_), 10), T * s_ * row * 2)
            del lc, ql
            torch.cuda.empty_cache()
            print(json.dumps({"bench": "kernels", "size": name, "rows": T, "kernels": rows}), flush=True)


def main(argv=None) -> None:
    ap = argparse.ArgumentParser(description=__doc__.splitlines()[0])
    ap.add_argument("--part", default="engine,kernels")
    ap.add_argument("--sizes", default="s,m")
    args = ap.parse_args(argv)
    assert torch.cuda.is_available(), "this benchmark needs the GPU"
    sizes = [s for s in args.sizes.split(",") if s]
    if "kernels" in args.part:
        part_kernels(sizes)
    if "engine" in args.part:
        part_engine(sizes)
    if "profile" in args.part:
        # Daberax only: the run to put under a profiler
        for name in sizes:
            print(json.dumps({"bench": "profile", "size": name,
                              "daberax": engine_run(daberax_config(name, SIZES[name]), 16, 1024, 64)}), flush=True)


if __name__ == "__main__":
    main()
