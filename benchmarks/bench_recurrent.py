#!/usr/bin/env python3
"""Garesun beside routed Lopovik and Potatar at equal size: prefill and decode
throughput through the engine, and the new kernels beside the like kernels of
those paths against the roofline.

    python bench.py --recurrent                 # both parts, JSON lines
    python benchmarks/bench_recurrent.py --part engine|kernels|profile [--sizes s,m]

The closest existing family is Lopovik with routed experts in every layer:
parallel layers over the same latent rows and the same attention kernel.  Its
mixers are all latent attention, two of four of Garesun's layers are matrix
recurrences; so Potatar's matrix-state layers (wkv in every layer, dense
feed-forward) stand beside it as well.

Engine part, per size: a Garesun stack (latent, retention, mLSTM, latent on
the first one's rows; twice), a routed Lopovik stack with the same width,
depth, latent sizes and as many active feed-forward parameters (three-matrix
experts against two-matrix experts beside a shared one), and a Potatar stack
of wkv layers with as many active feed-forward parameters.  The same workload
goes through LLMEngine.step(): N prompts of L tokens in budget-sized steps,
then K decode steps (hipGraph replay) at batch N.  Random weights, synthetic
tokens.

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
from llm_instance_gateway_amd.models.garesun import make_config
from llm_instance_gateway_amd.models.lopovik import make_config as lopovik_make
from llm_instance_gateway_amd.models.potatar import make_config as potatar_make

from bench_hybrid import HBM_BYTES_PER_S, engine_run, timeit

# latent attention, retention (heads x key/value sizes) and mLSTM sizes, expert
# width, side table entries per layer
SIZES = {
    "s": dict(width=2048, layers=8, heads=16, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=768,
              ret=(8, 128, 256), mls=(4, 256, 512), experts=8, top=2, ff=2048, side=128, vocab=32000),
    "m": dict(width=4096, layers=8, heads=32, dim=128, rot_dim=64, vdim=128, kv_rank=512, q_rank=1536,
              ret=(16, 128, 256), mls=(8, 256, 512), experts=8, top=2, ff=3584, side=256, vocab=32000),
}


def garesun_config(name: str, z: dict) -> ModelConfig:
    mlp = {"kind": "moe", "expert": {"ff": z["ff"]}, "router": {"experts": z["experts"], "top": z["top"]},
           "shared": {"ff": z["ff"]}}
    hr, dr, vr = z["ret"]
    hm, dm, vm = z["mls"]
    layers = []
    for i in range(z["layers"]):
        if i % 4 in (0, 3):
            m = {"heads": z["heads"], "dim": z["dim"], "rot_dim": z["rot_dim"], "vdim": z["vdim"],
                 "kv_rank": z["kv_rank"], "rot": {"base": 500000.0, "dims": z["rot_dim"]},
                 "scale": 1.0 / math.sqrt(z["dim"] + z["rot_dim"])}
            if i % 4 == 3:
                m["kv_from"] = i - 3
            layers.append({"type": "latent_attention", "mixer": m, "mlp": mlp})
        elif i % 4 == 1:
            decay = [1.0 - 2.0 ** (-5 - 7 * h / max(hr - 1, 1)) for h in range(hr)]
            layers.append({"type": "retention", "mixer": {"heads": hr, "dim": dr, "vdim": vr, "decay": decay,
                                                          "rot": {"base": 10000.0, "dims": dr}}, "mlp": mlp})
        else:
            layers.append({"type": "mlstm", "mixer": {"heads": hm, "dim": dm, "vdim": vm, "gate_cap": 15.0}, "mlp": mlp})
    return make_config(f"garesun-{name}", z["vocab"], z["width"], layers, embed_scale=1.0, side_dim=z["side"])


def lopovik_config(name: str, z: dict) -> ModelConfig:
    mixer = {"heads": z["heads"], "dim": z["dim"], "rot_dim": z["rot_dim"], "vdim": z["vdim"],
             "q_rank": z["q_rank"], "kv_rank": z["kv_rank"], "rot": {"base": 10000.0, "dims": z["rot_dim"]},
             "scale": 1.0 / math.sqrt(z["dim"] + z["rot_dim"])}
    mlp = {"kind": "moe", "expert": {"ff": z["ff"]}, "router": {"experts": z["experts"], "top": z["top"]}}
    return lopovik_make(f"lopovik-routed-{name}", z["vocab"], z["width"],
                        [{"type": "latent_attention", "mixer": dict(mixer), "mlp": mlp} for _ in range(z["layers"])])


def potatar_config(name: str, z: dict) -> ModelConfig:
    layer = {"type": "wkv", "mixer": {"heads": z["width"] // 64, "dim": 64, "decay_rank": 64},
             "mlp": {"ff": 3 * z["ff"], "kind": "dense"}}
    return potatar_make(f"potatar-wkv-{name}", z["vocab"], z["width"], [dict(layer) for _ in range(z["layers"])],
                        alpha=2.0)


def part_engine(sizes) -> None:
    for name in sizes:
        z = SIZES[name]
        for n_seqs, plen in ((16, 1024), (64, 512)):
            row = {"bench": "engine", "size": name, **z, "seqs": n_seqs, "prompt_len": plen, "decode_steps": 64}
            row["garesun"] = engine_run(garesun_config(name, z), n_seqs, plen, 64)
            row["lopovik_routed"] = engine_run(lopovik_config(name, z), n_seqs, plen, 64)
            row["potatar_wkv"] = engine_run(potatar_config(name, z), n_seqs, plen, 64)
            for k in ("prefill_tok_per_s", "decode_tok_per_s"):
                for other in ("lopovik_routed", "potatar_wkv"):
                    row[f"vs_{other}_{k}"] = round(row["garesun"][k] / row[other][k], 3)
            print(json.dumps(row), flush=True)


def part_kernels(sizes) -> None:
    dev, bf = "cuda:0", torch.bfloat16
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)
    for name in sizes:
        z = SIZES[name]
        W, FF = z["width"], z["ff"]
        hq, D, Rr, Rk = z["heads"], z["dim"], z["rot_dim"], z["kv_rank"]
        row = Rk + Rr
        for T in (8192, 256):  # a prefill step's rows / a decode batch
            rows = []

            def add(kernel, like, t, nbytes):
                rows.append({"kernel": kernel, "like": like, "us": round(t * 1e6, 2),
                             "GB_per_s": round(nbytes / t / 1e9, 1),
                             "of_roofline": round(nbytes / t / HBM_BYTES_PER_S, 3)})

            x32 = torch.randn(T, W, device=dev)
            y = torch.randn(T, W, device=dev, dtype=bf)
            w = torch.ones(W, device=dev, dtype=bf)
            toks = torch.randint(0, z["vocab"], (T,), device=dev)
            table = torch.randn(z["vocab"], W, device=dev, dtype=bf)
            # residual in and out (4B each), branch in, GEMM input out (2B each)
            add("add_layer_norm (normed add + layer norm)", "",
                timeit(lambda: ops.add_layer_norm(x32, w, 1e-5, y, w)), T * W * 12)
            add("scaled_add_rms_norm", "add_layer_norm",
                timeit(lambda: ops.scaled_add_rms_norm(x32, 2.0, w, 1e-6, y)), T * W * 12)
            add("embed_layer_norm", "", timeit(lambda: ops.embed_layer_norm(toks, table, 12.0, w, 1e-5)), T * W * 8)
            add("embed_group_norm", "embed_layer_norm",
                timeit(lambda: ops.embed_group_norm(toks, table, w, 1e-5, 1)), T * W * 6)
            ye = torch.randn(T * z["top"], W, device=dev, dtype=bf)
            rws = torch.randperm(T * z["top"], device=dev).view(T, z["top"])
            cw = torch.rand(T, z["top"], device=dev)
            add("residual_routed_add (+ rounding for the next GEMM)", "",
                timeit(lambda: ops.residual_routed_add(x32, y, ye, cw, rws)), T * W * (12 + 2 * z["top"]))
            add("routed_combine", "residual_routed_add",
                timeit(lambda: ops.routed_combine(ye, y, rws, cw)), T * W * 2 * (z["top"] + 1))
            add("residual_add (two branches)", "residual_routed_add",
                timeit(lambda: ops.residual_add(x32, y, y)), T * W * 12)
            # router + gate columns in fp32
            n_small = z["experts"] + 2 * z["mls"][0]
            ws = torch.randn(n_small, W, device=dev, dtype=bf)
            wr = torch.randn(z["experts"], W, device=dev)
            add(f"small_projection ({n_small} fp32 columns)", "",
                timeit(lambda: ops.small_projection(y, ws)), T * (W * 2 + n_small * 4))
            add("fp32 copy + library GEMM (Lopovik's router)", "small_projection",
                timeit(lambda: torch.nn.functional.linear(y.float(), wr)), T * (W * 2 + z["experts"] * 4))
            up = torch.randn(T, W + FF, device=dev, dtype=bf)
            o2 = torch.empty(T, W + FF, device=dev, dtype=bf)
            add("relu_squared between column blocks", "",
                timeit(lambda: ops.relu_squared(up[:, W:], out=o2[:, W:])), T * FF * 4)
            up1 = up[:, W:].contiguous()
            add("relu_squared", "the same map, contiguous", timeit(lambda: ops.relu_squared(up1)), T * FF * 4)
            zg = torch.randn(T, z["side"], device=dev, dtype=bf)
            st = torch.randn(z["vocab"], z["side"] * z["layers"], device=dev, dtype=bf)
            add("gelu_tanh_table_mul", "",
                timeit(lambda: ops.gelu_tanh_table_mul(zg, st[:, : z["side"]], toks)), T * z["side"] * 6)
            add("gelu_erf", "gelu_tanh_table_mul", timeit(lambda: ops.gelu_erf(zg)), T * z["side"] * 4)
            pos = torch.arange(T, device=dev, dtype=torch.int64) % 1024
            hr, dr, vr = z["ret"]
            inv = ops.rotary_inv_freq(10000.0, dr, dev)
            add("rotary_table (once per step)", "", timeit(lambda: ops.rotary_table(pos, inv)), T * dr * 4)
            # matrix recurrences: q, k, v in (2B), output (4B); single tokens also move the state both ways
            seg = 1024 if T >= 1024 else 1
            S = T // seg
            segs = (i32([i * seg for i in range(S)]), i32([seg] * S), i32(list(range(S))), i32([0] * S))

            def scan_bytes(h, d, v, ones=0):
                return T * h * (2 * d * 2 + v * 6) + 2 * S * h * d * (v + ones) * 4

            cs = ops.rotary_table(pos, inv)
            dec = torch.full((hr,), 0.99, device=dev)
            proj = torch.randn(T, hr * (2 * dr + 2 * vr), device=dev, dtype=bf)
            q, k, v = proj[:, : hr * dr], proj[:, hr * dr : 2 * hr * dr], proj[:, 2 * hr * dr : hr * (2 * dr + vr)]
            state = torch.zeros(S + 1, ops.matrix_state_width(hr, dr, vr), device=dev)
            add(f"matrix_state_scan, retention ({hr} heads {dr} x {vr}, rotated)", "",
                timeit(lambda: ops.matrix_state_scan(q, k, v, state, *segs, hr, dr, vr, head_decay=dec, rot=cs,
                                                     k_scale=0.1, max_seg_len=seg), 10), scan_bytes(hr, dr, vr))
            add("matrix_state_scan, constant decay + silu, the same sizes", "retention",
                timeit(lambda: ops.matrix_state_scan(q, k, v, state, *segs, hr, dr, vr, head_decay=dec,
                                                     act_silu=True), 10), scan_bytes(hr, dr, vr))
            del state
            hm, dm, vm = z["mls"]
            projm = torch.randn(T, hm * (2 * dm + 2 * vm), device=dev, dtype=bf)
            qm, km, vmv = (projm[:, : hm * dm], projm[:, hm * dm : 2 * hm * dm],
                           projm[:, 2 * hm * dm : hm * (2 * dm + vm)])
            zz = torch.randn(T, 2 * hm, device=dev)
            bi, bfg = torch.full((hm,), -1.0, device=dev), torch.full((hm,), 4.0, device=dev)
            state = torch.zeros(S + 1, ops.matrix_state_width(hm, dm, vm, True), device=dev)
            add(f"matrix_state_scan, mLSTM ({hm} heads {dm} x {vm}, gated)", "",
                timeit(lambda: ops.matrix_state_scan(qm, km, vmv, state, *segs, hm, dm, vm,
                                                     gates=(zz[:, :hm], zz[:, hm:]), gate_bias=(bi, bfg),
                                                     gate_cap=15.0, q_scale=0.1, max_seg_len=seg), 10), scan_bytes(hm, dm, vm, 1))
            del state
            decm = torch.full((hm,), 0.99, device=dev)
            state = torch.zeros(S + 1, ops.matrix_state_width(hm, dm, vm), device=dev)
            add("matrix_state_scan, constant decay + silu, the same sizes", "mLSTM",
                timeit(lambda: ops.matrix_state_scan(qm, km, vmv, state, *segs, hm, dm, vm, head_decay=decm,
                                                     act_silu=True), 10), scan_bytes(hm, dm, vm))
            del state
            hw = W // 64
            r64 = torch.randn(T, W, device=dev, dtype=bf)
            pre = torch.randn(T, W, device=dev) - 2.0
            bonus = torch.zeros(W, device=dev)
            state = torch.zeros(S + 1, ops.matrix_state_width(hw, 64, 64), device=dev)
            add(f"matrix_state_scan, bonus form ({hw} heads 64 x 64, Potatar)", "retention, mLSTM",
                timeit(lambda: ops.matrix_state_scan(r64, r64, r64, state, *segs, hw, 64, 64, decay_pre=pre,
                                                     bonus=bonus), 10), scan_bytes(hw, 64, 64) + T * W * 4)
            del state
            for h_, v_, act, wt in ((hr, vr, "silu", False), (hm, vm, "sigmoid", True), (hw, 64, "silu", True)):
                o = torch.randn(T, h_ * v_, device=dev)
                gt = torch.randn(T, h_ * v_, device=dev, dtype=bf)
                wn = torch.ones(h_ * v_, device=dev, dtype=bf) if wt else None
                add(f"group_rms_norm_gate (groups of {v_}, {act})", "" if v_ != 64 else "groups of retention, mLSTM",
                    timeit(lambda: ops.group_rms_norm_gate(o, gt, wn, v_, act, 1e-5)), T * h_ * v_ * 8)
            # latent attention: direct queries, gate per head
            bs, L = 16, 1024
            nb_seq = L // bs
            nblk = T // 16 + 1
            cache = torch.zeros(nblk, 1, bs, row, device=dev, dtype=bf)
            slots = torch.randperm(T, device=dev).to(torch.int64)
            nq = hq * (D + Rr)
            proj = torch.randn(T, nq + row + hq, device=dev, dtype=bf)
            wk = torch.ones(Rk, device=dev, dtype=bf)
            wq = torch.ones(z["q_rank"], device=dev, dtype=bf)
            inv = ops.rotary_inv_freq(10000.0, Rr, dev)
            add("latent_kv_prep without a query latent", "",
                timeit(lambda: ops.latent_kv_prep(proj[:, nq:], 0, Rk, Rr, None, wk, 1e-5, inv, pos, slots, cache)),
                T * row * 4)
            add("latent_kv_prep (Lopovik)", "the same kernel with a query latent",
                timeit(lambda: ops.latent_kv_prep(proj, z["q_rank"], Rk, Rr, wq, wk, 1e-5, inv, pos, slots, cache)),
                T * (row + z["q_rank"]) * 4)
            qa = torch.zeros(T, hq, row, device=dev, dtype=bf)
            qc = proj[:, :nq].contiguous()
            add("rotate_pack_queries from the fused projection", "",
                timeit(lambda: ops.rotate_pack_queries(proj[:, :nq], hq, D, Rr, inv, pos, qa, Rk)), T * hq * Rr * 4)
            add("rotate_pack_queries (Lopovik)", "the same kernel, contiguous",
                timeit(lambda: ops.rotate_pack_queries(qc, hq, D, Rr, inv, pos, qa, Rk)), T * hq * Rr * 4)
            sink = torch.zeros(hq, device=dev)
            gate = proj[:, nq + row :]
            sc = 1.0 / math.sqrt(D + Rr)
            qlat = torch.randn(T, hq * row, device=dev, dtype=bf)
            if T >= 1024:
                lcache = torch.randn(S * nb_seq + 1, 1, bs, row, device=dev, dtype=bf)
                tables = torch.arange(S * nb_seq, dtype=torch.int32, device=dev).view(S, nb_seq)
                args = (qlat, lcache, Rk, tables, i32([i * L for i in range(S)]), i32([L] * S), i32([L] * S), L, sc, hq)
                pairs = S * (L * (L + 1) / 2) * hq
                for what, kw in (("gate per head", dict(gate=gate)), ("sink, Lopovik", dict(sink=sink))):
                    t = timeit(lambda: ops.latent_attention_rows(*args, **kw), 5)
                    rows.append({"kernel": f"latent_attention_rows ({what})", "like": "", "us": round(t * 1e6, 1),
                                 "TFLOP_per_s": round(2 * (row + Rk) * pairs / t / 1e12, 1)})
            else:
                lcache = torch.randn(T * nb_seq + 1, 1, bs, row, device=dev, dtype=bf)
                tables = torch.arange(T * nb_seq, dtype=torch.int32, device=dev).view(T, nb_seq)
                args = (qlat, lcache, Rk, tables, i32(list(range(T))), i32([1] * T), i32([L] * T), 1, sc, hq)
                for what, kw in (("gate per head", dict(gate=gate)), ("sink, Lopovik", dict(sink=sink))):
                    add(f"latent_attention_rows (single tokens, {what})", "",
                        timeit(lambda: ops.latent_attention_rows(*args, **kw), 10), T * L * row * 2)
            print(json.dumps({"bench": "kernels", "size": name, "rows": T, "kernels": rows}), flush=True)
            del lcache, tables, qlat, qa, proj
            torch.cuda.empty_cache()


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
        # Garesun only: the run to put under a profiler
        for name in sizes:
            print(json.dumps({"bench": "profile", "size": name,
                              "garesun": engine_run(garesun_config(name, SIZES[name]), 16, 1024, 64)}), flush=True)


if __name__ == "__main__":
    main()
