"""Daberax: a decoder-only stack whose norms sit on the sub-layers' outputs,
over delta-rule, latent and soft-capped attention mixers, with a per-layer
token table.

config.json lists the layers.  A sub-layer reads the residual itself; only
its output is normed on the way in:

    x <- x + rms(mixer(x)) * w1;   x <- x + rms(ff(x)) * w2
    y = W_proj (gelu_tanh(W_gate x) * side[token, layer]);  x <- x + rms(y) * w_side

Mixers:
  * "delta": the gated delta rule behind short convolutions, unit-length q
    and k, silu gate on normed heads.
  * "attention": grouped-query softmax attention with biases, q and k normed
    over the whole projection, interleaved rotation with banded frequency
    scaling, soft-capped scores, a sliding window, one sigmoid gate per head.
  * "latent_attention": queries projected directly, keys and values from a
    normed low-rank latent plus one rotated key part shared by the heads, a
    sliding window.

The feed-forward is down(gelu_tanh(gate x) * up x); a layer may have none.
The logits are multiplied by a constant.  The residual stream is fp32 in
every mode.

Execution on the engine's flat batch: every sub-layer is its input GEMM, the
mixer's kernels (or the activation), its output GEMM, and one kernel that
norms the output, adds it to the residual and writes the sum rounded for the
next GEMM; the last one writes the final norm instead.
"""

from __future__ import annotations

import os
from typing import List, Optional

import torch
import torch.nn as nn

from .. import ops
from .config import LayerSpec, ModelConfig
from .hybrid_blocks import (
    GatedDeltaMixer, GatedMLP, LatentAttention, NormedRotaryAttention, TokenTableGate, _param,
)

MIXERS = ("delta", "attention", "latent_attention")


def config_from_json(raw: dict, path: str = "") -> ModelConfig:
    specs: List[LayerSpec] = []
    for i, entry in enumerate(raw["layers"]):
        t = entry["type"]
        if t not in MIXERS:
            raise ValueError(f"layer {i}: unknown mixer type {t!r}")
        mlp = entry.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
        specs.append(
            LayerSpec(type=t, mixer=dict(entry["mixer"]), mlp=None if mlp is None else dict(mlp))
        )
    return ModelConfig(
        name=os.path.basename(os.path.normpath(path)) or "daberax",
        architecture="daberax",
        vocab_size=int(raw["vocab"]),
        hidden_size=int(raw["width"]),
        num_layers=len(specs),
        rms_norm_eps=float(raw["norm"]["eps"]),
        layer_specs=specs,
        weights_path=path,
        logit_scale=float(raw.get("logit_scale", 1.0)),
        token_side_dim=int((raw.get("token_side") or {}).get("dim", 0)),
        # angles are computed from the position itself: no table bounds the
        # context
        max_position_embeddings=1 << 30,
    )


def make_config(
    name: str, vocab: int, width: int, layers: List[dict], eps: float = 1e-5,
    logit_scale: float = 1.0, side_dim: int = 0,
) -> ModelConfig:
    """A random-init config from the same fields config.json carries."""
    cfg = config_from_json(
        {"vocab": vocab, "width": width, "layers": layers, "norm": {"eps": eps},
         "logit_scale": logit_scale, "token_side": {"dim": side_dim}}
    )
    cfg.name = name
    return cfg


def _mixer(kind: str, hidden: int, m: dict, eps: float, device, dtype):
    if kind == "delta":
        return GatedDeltaMixer(
            hidden, m["heads"], m["kv_heads"], m["dim"], m["vdim"], int(m["conv"]), eps,
            device=device, dtype=dtype,
        )
    rot = m.get("rot") or {}
    base, dims, scaling = float(rot.get("base", 10000.0)), int(rot.get("dims", 0)), rot.get("scaling")
    window = int((m.get("mask") or {}).get("size", 0))
    if kind == "attention":
        return NormedRotaryAttention(
            hidden, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], eps,
            qk_norm="row", rot_base=base, rot_dims=dims, rot_layout="interleaved",
            rot_scaling=scaling, window=window, bias=True, head_gate=True,
            softcap=float(m.get("softcap") or 0.0), device=device, dtype=dtype,
        )
    return LatentAttention(
        hidden, m["heads"], m["dim"], m["rot_dim"], m["vdim"], 0, m["kv_rank"], m["scale"], base,
        dims, eps, sink=False, out_gate=False, window=window, rot_scaling=scaling,
        device=device, dtype=dtype,
    )


class DaberaxLayer(nn.Module):
    def __init__(self, spec: LayerSpec, hidden: int, eps: float, side_dim: int, device, dtype) -> None:
        super().__init__()
        self.mixer = _mixer(spec.type, hidden, spec.mixer, eps, device, dtype)
        self.norm1 = _param((hidden,), device, dtype, None)
        self.mlp: Optional[GatedMLP] = None
        self.norm2 = None
        if spec.mlp is not None:
            self.mlp = GatedMLP(hidden, int(spec.mlp["ff"]), "gelu_tanh", device=device, dtype=dtype)
            self.norm2 = _param((hidden,), device, dtype, None)
        with torch.no_grad():
            self.norm1.fill_(1.0)
            if self.norm2 is not None:
                self.norm2.fill_(1.0)
        self.side = TokenTableGate(hidden, side_dim, device, dtype) if side_dim > 0 else None


class DaberaxForCausalLM(nn.Module):
    # the runner builds per-token sequence tables and per-sequence segments
    needs_seq_tables = True
    # no adapter hooks in the mixers: base model only
    supports_lora = False
    # single-token steps have static shapes and no host round trip
    supports_decode_graphs = True

    def __init__(self, cfg: ModelConfig, device="cpu", dtype=torch.bfloat16, tp=None) -> None:
        super().__init__()
        if tp is not None and tp.world_size > 1:
            raise NotImplementedError("Daberax runs on one GPU per engine (no tensor parallelism)")
        assert cfg.layer_specs, "Daberax needs per-layer specs"
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
                DaberaxLayer(s, H, cfg.rms_norm_eps, cfg.token_side_dim, device, dtype)
                for s in cfg.layer_specs
            ]
        )
        # prompt rows of the attention layers run the MFMA tile kernel where
        # the head sizes allow: the runner then builds 64-row tiles
        on_gpu = self.device_.type == "cuda"
        self.needs_prefill_tiles = any(
            s.type == "attention"
            and ops.tiled_prefill_supported(dtype, s.mixer["dim"], s.mixer["vdim"], on_gpu)
            for s in cfg.layer_specs
        )
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
                    layer.norm2.copy_(get(p + "norm2"))
                    layer.mlp.load(get, p + "mlp.")
                else:
                    used.add(p + "norm2")  # a layer without feed-forward has no use for it
                if layer.side is not None:
                    layer.side.load(get, p + "side.")
        extra = sorted(set(tensors) - used)
        if extra:
            raise ValueError(f"checkpoint tensors the model does not know: {extra[:8]}")

    def forward(self, input_ids, positions, kv_caches, meta) -> torch.Tensor:
        eps, dim, last = self.cfg.rms_norm_eps, self.cfg.token_side_dim, len(self.layers) - 1
        h = self.embed.index_select(0, input_ids)  # activation dtype
        x = h.float()                              # the residual, fp32

        def join(y, w, ends: bool):
            """x += rms(y) * w; the rounded sum, or the final norm of it."""
            if ends:
                return ops.post_add_pre_norm(x, y, w, self.final_norm, eps, 1)
            return ops.post_add_pre_norm(x, y, w, None, eps, 1, rounded=True)

        for i, layer in enumerate(self.layers):
            y = layer.mixer(h, positions, kv_caches[i], meta)
            h = join(y, layer.norm1, i == last and layer.mlp is None and layer.side is None)
            if layer.mlp is not None:
                h = join(layer.mlp(h), layer.norm2, i == last and layer.side is None)
            if layer.side is not None:
                y = layer.side(h, self.side_embed[:, i * dim : (i + 1) * dim], input_ids)
                h = join(y, layer.side.norm, i == last)
            if self.capture_residuals is not None:
                self.capture_residuals.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor, indices: torch.Tensor) -> torch.Tensor:
        z = (hidden[indices] @ self.head.t()).float()
        if self.cfg.logit_scale != 1.0:
            z.mul_(self.cfg.logit_scale)
        return z
