"""Garesun: a decoder-only stack of parallel layers over recurrent and latent
mixers, with a per-layer token table beside the residual.

config.json lists the layers; both sub-layers read ONE layer norm (centred,
weight, no bias) and are added at once, then the token table joins:

    h = LN(x) * w;   x <- x + mixer(h) + ff(h)
    y = W_proj (gelu_tanh(W_gate x) * side[token, layer]);  x <- x + rms(y) * w_side

The embedding rows are multiplied by a constant.  Mixers:
  * "retention": linear attention with one fixed decay per head, rotate-half
    positions on q and k, unit-RMS heads, silu gate.
  * "mlstm": matrix memory with capped exponential input and sigmoid forget
    gates, a normaliser and a running maximum; normed heads, sigmoid gate.
  * "latent_attention": queries projected directly, keys and values from a
    normed low-rank latent plus one rotated key part shared by the heads,
    softmax, one sigmoid gate per head.  A layer with "kv_from" caches
    nothing: it reads the rows another layer cached for the same tokens.

Feed-forward: routed squared-ReLU experts (softmax over the chosen logits)
beside a shared expert; a layer may have none.  The residual stream is fp32
in every mode.

Execution on the engine's flat batch, per layer: one input GEMM (the mixer's
projections and the shared expert's up-projection), one fp32 product for the
router's and the recurrence gates' columns, the mixer's kernels, one output
GEMM over [gated heads | shared activation], the routed experts, one kernel
that adds everything to the residual, the token-table GEMMs, and one kernel
for their norm, the add and the NEXT layer's norm.
"""

from __future__ import annotations

import os
from typing import List, Optional

import torch
import torch.nn as nn
import torch.nn.functional as F

from .. import ops
from .config import LayerSpec, ModelConfig
from .hybrid_blocks import (
    LatentAttention, ReluSquaredExpertsMLP, ScalarDecayMixer, TokenTableGate, _param,
)

MIXERS = ("retention", "mlstm", "latent_attention")


def config_from_json(raw: dict, path: str = "") -> ModelConfig:
    specs: List[LayerSpec] = []
    for i, entry in enumerate(raw["layers"]):
        t, m = entry["type"], dict(entry["mixer"])
        if t not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer type {t!r}")
        mlp = entry.get("mlp")
        if mlp is not None and mlp.get("kind") != "moe":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
        src = m.get("kv_from")
        if src is not None:
            if not 0 <= src < i or specs[src].type != "latent_attention":
                raise ValueError(f"layer {i}: kv_from {src} is no earlier latent-attention layer")
            own = specs[src].mixer
            if own.get("kv_from") is not None or any(
                own[k] != m[k] for k in ("kv_rank", "rot_dim", "rot")
            ):
                raise ValueError(f"layer {i}: kv_from {src} caches no rows this layer can read")
        specs.append(LayerSpec(type=t, mixer=m, mlp=None if mlp is None else dict(mlp)))
    return ModelConfig(
        name=os.path.basename(os.path.normpath(path)) or "garesun",
        architecture="garesun",
        vocab_size=int(raw["vocab"]),
        hidden_size=int(raw["width"]),
        num_layers=len(specs),
        rms_norm_eps=float(raw["norm"]["eps"]),
        layer_specs=specs,
        weights_path=path,
        embed_scale=float((raw.get("embedding") or {}).get("scale", 1.0)),
        token_side_dim=int((raw.get("token_side") or {}).get("dim", 0)),
        # angles are computed from the position itself: no table bounds the
        # context
        max_position_embeddings=1 << 30,
    )


def make_config(
    name: str, vocab: int, width: int, layers: List[dict], eps: float = 1e-5,
    embed_scale: float = 1.0, side_dim: int = 0,
) -> ModelConfig:
    """A random-init config from the same fields config.json carries."""
    cfg = config_from_json(
        {"vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
         "embedding": {"scale": embed_scale}, "token_side": {"dim": side_dim}}
    )
    cfg.name = name
    return cfg


def _mixer(kind: str, hidden: int, m: dict, eps: float, device, dtype):
    rot = m.get("rot") or {}
    base, dims = float(rot.get("base", 10000.0)), int(rot.get("dims", 0))
    if kind == "latent_attention":
        return LatentAttention(
            hidden, m["heads"], m["dim"], m["rot_dim"], m["vdim"], 0, m["kv_rank"], m["scale"],
            base, dims, eps, sink=False, out_gate=False, head_gate=True,
            own_rows=m.get("kv_from") is None, device=device, dtype=dtype,
        )
    return ScalarDecayMixer(
        hidden, kind, m["heads"], m["dim"], m["vdim"], eps, decay=m.get("decay"),
        rot_base=base, rot_dims=dims, gate_cap=float(m.get("gate_cap", 1.0)),
        device=device, dtype=dtype,
    )


class GaresunLayer(nn.Module):
    def __init__(self, spec: LayerSpec, hidden: int, eps: float, side_dim: int, device, dtype) -> None:
        super().__init__()
        self.type = spec.type
        self.kv_from = spec.mixer.get("kv_from")
        self.mixer = _mixer(spec.type, hidden, spec.mixer, eps, device, dtype)
        self.norm1 = _param((hidden,), device, dtype, None)
        with torch.no_grad():
            self.norm1.fill_(1.0)
        self.mlp: Optional[ReluSquaredExpertsMLP] = None
        if spec.mlp is not None:
            r = spec.mlp["router"]
            self.mlp = ReluSquaredExpertsMLP(
                hidden, int(spec.mlp["expert"]["ff"]), int(r["experts"]), int(r["top"]),
                shared_ff=int((spec.mlp.get("shared") or {}).get("ff", 0)),
                device=device, dtype=dtype,
            )
        self.side = TokenTableGate(hidden, side_dim, device, dtype) if side_dim > 0 else None
        self.w_in = self.w_out = self.w_small = None
        self.fuse()

    def fuse(self) -> None:
        """One weight per GEMM: [mixer rows | shared expert's up] in, [mixer's
        output | shared expert's down] out, [router | mixer gates] for the
        fp32 columns.  The blocks' own weights become views of the fused
        ones.  The mixer's rows are padded so that the shared expert's columns
        stay 16-byte aligned."""
        mix = self.mixer
        shared = self.mlp.shared if self.mlp is not None else None
        n = mix.w_in.shape[0]
        self.shared_col = (n + 7) // 8 * 8
        rows = [mix.w_in.data]
        if shared is not None:
            rows += [mix.w_in.data.new_zeros(self.shared_col - n, mix.w_in.shape[1]), shared.w_up.data]
        self.w_in = torch.cat(rows, dim=0).contiguous()
        mix.w_in.data = self.w_in[:n]
        cols = [mix.w_o.data]
        if shared is not None:
            shared.w_up.data = self.w_in[self.shared_col :]
            cols.append(shared.w_down.data)
        self.w_out = torch.cat(cols, dim=1).contiguous()
        mix.w_o.data = self.w_out[:, : mix.n_out]
        if shared is not None:
            shared.w_down.data = self.w_out[:, mix.n_out :]
        small = ([self.mlp] if self.mlp is not None else []) + (
            [mix] if getattr(mix, "w_small", None) is not None else []
        )
        self.n_experts = self.mlp.experts if self.mlp is not None else 0
        if small:
            self.w_small = torch.cat([b.w_small.data for b in small], dim=0).contiguous()
            at = 0
            for b in small:
                n = b.w_small.shape[0]
                b.w_small.data = self.w_small[at : at + n]
                at += n

    def forward(self, x, h, positions, cache, meta, tables):
        """Adds mixer(h) + ff(h) to the fp32 residual x in place; returns x
        rounded to the activation dtype."""
        mix, rows = self.mixer, h.shape[0]
        proj = F.linear(h, self.w_in)
        small = ops.small_projection(h, self.w_small) if self.w_small is not None else None
        buf = torch.empty(rows, self.w_out.shape[1], dtype=h.dtype, device=h.device)
        heads = buf[:, : mix.n_out]
        if self.type == "latent_attention":
            mix.mix(proj, positions, cache, meta, out=heads)
        else:
            gates = small[:, self.n_experts :] if self.type == "mlstm" else None
            mix.mix(proj, gates, positions, cache, meta, out=heads, tables=tables)
        if heads.shape[1] < buf.shape[1]:
            ops.relu_squared(proj[:, self.shared_col :], out=buf[:, mix.n_out :])
        y = F.linear(buf, self.w_out)
        routed = {}
        if self.mlp is not None:
            routed = self.mlp.experts_of(h, small[:, : self.n_experts], meta)
        return ops.residual_routed_add(x, y, **routed)


class GaresunForCausalLM(nn.Module):
    # the runner builds per-token sequence tables and per-sequence segments
    needs_seq_tables = True
    # no adapter hooks in the mixers: base model only
    supports_lora = False
    # single-token steps have static shapes and no host round trip
    supports_decode_graphs = True

    def __init__(self, cfg: ModelConfig, device="cpu", dtype=torch.bfloat16, tp=None) -> None:
        super().__init__()
        if tp is not None and tp.world_size > 1:
            raise NotImplementedError("Garesun runs on one GPU per engine (no tensor parallelism)")
        assert cfg.layer_specs, "Garesun needs per-layer specs"
        self.cfg = cfg
        self.device_ = torch.device(device)
        self.dtype_ = dtype
        H, V, L = cfg.hidden_size, cfg.vocab_size, len(cfg.layer_specs)
        self.embed = _param((V, H), device, dtype, 1.0)
        self.side_embed = (
            _param((V, L * cfg.token_side_dim), device, dtype, 1.0) if cfg.token_side_dim > 0 else None
        )
        self.final_norm = _param((H,), device, dtype, None)
        with torch.no_grad():
            self.final_norm.fill_(1.0)
        self.head = _param((V, H), device, dtype, 1.0 / (H ** 0.5))
        self.layers = nn.ModuleList(
            [
                GaresunLayer(s, H, cfg.rms_norm_eps, cfg.token_side_dim, device, dtype)
                for s in cfg.layer_specs
            ]
        )
        # attention addresses the batch per segment: no per-head query tiles
        self.needs_prefill_tiles = False
        # test/debug hook: when a list, forward() appends the fp32 residual
        # stream after every layer
        self.capture_residuals: Optional[list] = None

    def decode_attention_shape(self):
        return None  # no layer uses the split paged-decode kernel

    def cache_specs(self) -> List:
        return [layer.mixer.cache_spec() for layer in self.layers]

    def load_weights(self, tensors) -> None:
        used = set()

        def get(name: str) -> torch.Tensor:
            if name not in tensors:
                raise KeyError(f"checkpoint has no tensor {name!r}")
            used.add(name)
            return tensors[name].to(device=self.device_, dtype=self.dtype_)

        with torch.no_grad():
            self.embed.copy_(get("embed"))
            if self.side_embed is not None:
                self.side_embed.copy_(get("side.embed"))
            self.final_norm.copy_(get("final.norm"))
            self.head.copy_(get("head"))
            for i, layer in enumerate(self.layers):
                p = f"l{i}."
                layer.norm1.copy_(get(p + "norm1"))
                layer.mixer.load(get, p + "mix.")
                if layer.mlp is not None:
                    layer.mlp.load(get, p + "mlp.")
                if layer.side is not None:
                    layer.side.load(get, p + "side.")
        extra = sorted(set(tensors) - used)
        if extra:
            raise ValueError(f"checkpoint tensors the model does not know: {extra[:8]}")

    def forward(self, input_ids, positions, kv_caches, meta) -> torch.Tensor:
        cfg = self.cfg
        eps, dim = cfg.rms_norm_eps, cfg.token_side_dim
        tables: dict = {}  # rotation tables, shared by the layers of this step
        norms = [layer.norm1 for layer in self.layers[1:]] + [self.final_norm]
        x, h = ops.embed_layer_norm(input_ids, self.embed, cfg.embed_scale, self.layers[0].norm1, eps)
        for i, layer in enumerate(self.layers):
            cache = kv_caches[i if layer.kv_from is None else layer.kv_from]
            xt = layer(x, h, positions, cache, meta, tables)
            if layer.side is not None:
                y = layer.side(xt, self.side_embed[:, i * dim : (i + 1) * dim], input_ids)
                h = ops.add_layer_norm(x, norms[i], eps, y, layer.side.norm)
            else:
                h = ops.add_layer_norm(x, norms[i], eps)
            if self.capture_residuals is not None:
                self.capture_residuals.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor, indices: torch.Tensor) -> torch.Tensor:
        return (hidden[indices] @ self.head.t()).float()
