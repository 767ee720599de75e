"""Senavik: a pre-norm decoder whose softmaxes have a sink,

    x <- x + mixer(norm1(x)) ;  x <- x + ff(norm2(x)) ,

where norm is an RMS norm whose weight is stored as what it adds to 1, and x
starts as the normed embedding row. Layers pick one of two mixers: `attention`
(grouped-query, partial rotary positions in the banded frequency scaling, a
sliding window that keeps the first tokens) or `latent_attention` (queries
through a latent of their own, one low-rank cache row per token, YaRN-scaled
rotary part); both have a learned score per head that takes part in the
softmax without a value. The feed-forward is a dense squared-relu layer or a
mixture of silu-gated experts chosen by sigmoid scores plus a learned
correction, within the best groups of neighbours; a layer may have none.

Everything a checkpoint's config.json states (sizes, the order of layers,
constants) is read from it. All memory sits in the paged cache (key and value
rows per kv head, or one latent row per token); there is no carried state.

Tensor parallelism is not implemented for this family (tp_size must be 1).
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from kukeon_amd import ops
from kukeon_amd import parallel
from kukeon_amd.models.feedforward import FFCfg, RoutedMoE, SquaredReluFF
from kukeon_amd.models.mixers import (LatentAttention, LatentAttnCfg,
                                      RotaryAttention, RotaryAttnCfg)
from kukeon_amd.models.rotary import attach_tables, scaling_key

_DTYPES = {"bf16": torch.bfloat16, "bfloat16": torch.bfloat16,
           "fp32": torch.float32, "float32": torch.float32}

MIXERS = {"attention": RotaryAttention, "latent_attention": LatentAttention}
FEED_FORWARDS = {"dense": SquaredReluFF, "moe": RoutedMoE}


@dataclass
class SenavikLayerCfg:
    type: str                # "attention" | "latent_attention"
    mixer: object
    mlp: Optional[FFCfg]


@dataclass
class SenavikConfig:
    family = "senavik"
    name: str = "senavik"
    width: int = 1024
    vocab_size: int = 32000
    norm_eps: float = 1e-5
    layers: List[SenavikLayerCfg] = field(default_factory=list)

    @property
    def hidden_size(self) -> int:
        return self.width

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def is_moe(self) -> bool:
        return False

    @staticmethod
    def from_json(c: dict, name: str = "senavik") -> "SenavikConfig":
        layers = []
        for i, L in enumerate(c["layers"]):
            kind = L.get("type")
            m = L["mixer"]
            if kind == "attention":
                r, mask = m.get("rot") or {}, m.get("mask") or {}
                mix = RotaryAttnCfg(
                    heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                    dim=int(m["dim"]), vdim=int(m["vdim"]),
                    scale=float(m["scale"]),
                    rot_dims=int(r.get("dims") or 0),
                    rot_base=float(r.get("base") or 1.0),
                    rot_scaling=scaling_key(r.get("scaling")),
                    window=int(mask.get("size") or 0),
                    keep_first=int(mask.get("keep_first") or 0), sink=True)
            elif kind == "latent_attention":
                r = m["rot"]
                mix = LatentAttnCfg(
                    heads=int(m["heads"]), dim=int(m["dim"]),
                    rot_dim=int(m["rot_dim"]), vdim=int(m["vdim"]),
                    q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]),
                    scale=float(m["scale"]), window=0,
                    rot_dims=int(r["dims"]), rot_base=float(r["base"]),
                    rot_scaling=scaling_key(r.get("scaling")),
                    rot_layout="half", gate="none", sink=True)
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            mlp = None
            if L.get("mlp"):
                f = L["mlp"]
                fk = f.get("kind")
                if fk == "dense":
                    mlp = FFCfg("dense", int(f["ff"]))
                elif fk == "moe":
                    r = f["router"]
                    g = r.get("groups") or {}
                    mlp = expert_cfg(int(f["expert"]["ff"]),
                                     int(r["experts"]), int(r["top"]),
                                     int(g.get("count") or 0),
                                     int(g.get("keep") or 0))
                else:
                    raise ValueError(f"layer {i}: unknown feed-forward kind "
                                     f"{fk!r}")
            layers.append(SenavikLayerCfg(kind, mix, mlp))
        return SenavikConfig(
            name=name, width=int(c["width"]), vocab_size=int(c["vocab"]),
            norm_eps=float(c["norm"]["eps"]), layers=layers)


def expert_cfg(ff: int, experts: int, top: int, groups: int = 0,
               keep: int = 0) -> FFCfg:
    """Silu-gated experts; the choice by corrected sigmoid scores, a group
    of experts standing for the sum of its two best."""
    return FFCfg("moe", ff, experts=experts, top=top, act="silu",
                 score="corrected", groups=groups, keep=keep, group_best=2)


def senavik_bench(width=4096, layers=8, heads=32, kv_heads=8, ff=14336,
                  vocab=128256, window=1024, keep_first=4, experts=16, top=2,
                  name="senavik-8b-like") -> SenavikConfig:
    """A layer stack at real-model sizes (random weights) for throughput
    runs, in periods of four layers (a shorter stack ends like one): three of
    windowed attention (heads of 128, half of a head rotated) and one of
    latent attention (heads of 128 + 64, a 512-wide latent, a query latent of
    3/8 of the width);
    feed-forwards alternate between dense and routed experts of the same
    active size, the experts in four groups of which two are kept."""
    hd = 128 if width >= 1024 else 32
    ls = []
    for i in range(layers):
        if i % 4 == 3 or (layers < 4 and i == layers - 1 > 0):
            kind = "latent_attention"
            mix = LatentAttnCfg(
                heads=heads, dim=128, rot_dim=64, vdim=128,
                q_rank=max(64, width * 3 // 8), kv_rank=512,
                scale=192 ** -0.5, window=0, rot_dims=64, rot_base=10000.0,
                rot_scaling=scaling_key(dict(factor=4.0, original=4096,
                                             fast=32.0, slow=1.0)),
                rot_layout="half", gate="none", sink=True)
        else:
            kind = "attention"
            mix = RotaryAttnCfg(
                heads=heads, kv_heads=kv_heads, dim=hd, vdim=hd,
                scale=hd ** -0.5, rot_dims=hd // 2, rot_base=500000.0,
                rot_scaling=scaling_key(dict(factor=8.0, low=1.0, high=4.0,
                                             original=8192)),
                window=window, keep_first=keep_first, sink=True)
        if i % 2:
            mlp = expert_cfg(max(8, ff // top // 8 * 8), experts, top,
                             4 if experts % 4 == 0 else 0, 2)
        else:
            mlp = FFCfg("dense", ff)
        ls.append(SenavikLayerCfg(kind, mix, mlp))
    return SenavikConfig(name=name, width=width, vocab_size=vocab,
                         norm_eps=1e-5, layers=ls)


def tensor_shapes(cfg: SenavikConfig) -> Dict[str, tuple]:
    """Names and shapes of a checkpoint of this configuration."""
    W = cfg.width
    out = {"embed": (cfg.vocab_size, W), "embed.norm": (W,)}
    for i, L in enumerate(cfg.layers):
        p = f"l{i}."
        out[p + "norm1"] = (W,)
        for n, s in MIXERS[L.type].tensor_shapes(L.mixer, W).items():
            out[p + "mix." + n] = s
        if L.mlp is not None:
            out[p + "norm2"] = (W,)
            shapes = FEED_FORWARDS[L.mlp.kind].tensor_shapes(
                L.mlp, W, cfg.vocab_size)
            for n, s in shapes.items():
                out[p + "mlp." + n] = s
    out["final.norm"] = (W,)
    out["head"] = (cfg.vocab_size, W)
    return out


def random_tensors(cfg: SenavikConfig, seed: int = 0,
                   device="cpu") -> Dict[str, torch.Tensor]:
    """Random bf16 weights at a scale that keeps activations O(1)."""
    on_gpu = torch.device(device).type == "cuda"
    gdev = device if on_gpu else "cpu"
    g = torch.Generator(device=gdev).manual_seed(seed)
    out = {}
    for name, shp in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        t = torch.randn(shp, generator=g, device=gdev)
        if len(shp) == 2:
            std = shp[1] ** -0.5 if name != "embed" else 1.0
            t = t * (2.0 * std if leaf == "router" else std)
        elif name.endswith(("dq.norm", "dkv.norm")):
            t = 1.0 + 0.1 * t                  # plain weights
        elif leaf == "sink":
            pass
        else:                                  # added to 1, or to a score
            t = 0.1 * t
        out[name] = t.to(torch.bfloat16).to(device)
    return out


class SenavikLayer(nn.Module):
    def __init__(self, cfg: SenavikConfig, idx: int,
                 t: Dict[str, torch.Tensor], device, dtype):
        super().__init__()
        L = cfg.layers[idx]
        p = f"l{idx}."
        W = cfg.width
        f32 = dict(device=device, dtype=torch.float32)
        self.norm1 = t[p + "norm1"].to(**f32).contiguous()
        self.mixer = MIXERS[L.type](L.mixer, W, cfg.norm_eps, t, p + "mix.",
                                    device, dtype)
        self.ff = None
        if L.mlp is not None:
            self.norm2 = t[p + "norm2"].to(**f32).contiguous()
            self.ff = FEED_FORWARDS[L.mlp.kind](L.mlp, W, t, p + "mlp.",
                                                device, dtype)


class SenavikModel(nn.Module):
    family = "senavik"
    op_groups = ("sink",)       # kernel groups the forward pass needs

    def __init__(self, cfg: SenavikConfig, device="cuda", dtype="bf16",
                 tensors: Optional[Dict[str, torch.Tensor]] = None,
                 max_position: int = 4096, seed: int = 0):
        super().__init__()
        if parallel.tp_size() != 1:
            raise NotImplementedError("Senavik runs with tp_size == 1 only")
        self.cfg = cfg
        self.device_ = torch.device(device)
        self.dtype = _DTYPES[dtype] if isinstance(dtype, str) else dtype
        if tensors is None:
            tensors = random_tensors(cfg, seed, device=self.device_)
        for name, shp in tensor_shapes(cfg).items():
            if name not in tensors:
                raise KeyError(f"checkpoint lacks tensor {name}")
            if tuple(tensors[name].shape) != tuple(shp):
                raise ValueError(f"{name}: shape {tuple(tensors[name].shape)}"
                                 f", configuration says {tuple(shp)}")
        dev, dt = self.device_, self.dtype
        self.embed = nn.Parameter(tensors["embed"].to(dev).to(dt)
                                  .contiguous(), requires_grad=False)
        self.head = nn.Parameter(tensors["head"].to(dev).to(dt).contiguous(),
                                 requires_grad=False)
        self.embed_norm = tensors["embed.norm"].to(dev).float().contiguous()
        self.final_norm = tensors["final.norm"].to(dev).float().contiguous()
        self.layers = nn.ModuleList(
            [SenavikLayer(cfg, i, tensors, dev, dt)
             for i in range(cfg.num_layers)])
        self.set_max_position(max_position)

    @classmethod
    def from_checkpoint(cls, model_dir: str, device="cuda", dtype="bf16",
                        max_position: int = 4096):
        from kukeon_amd.models.weights import read_checkpoint
        config, tensors = read_checkpoint(model_dir)
        cfg = SenavikConfig.from_json(config)
        return cfg, cls(cfg, device=device, dtype=dtype, tensors=tensors,
                        max_position=max_position)

    def set_max_position(self, n: int) -> None:
        """(Re)build the angle tables for positions 0 .. n-1."""
        self.max_position = n
        attach_tables([L.mixer for L in self.layers], n, self.device_)

    # ---- what the engine asks of a model with its own cache layout ----
    def kv_specs(self):
        return [L.mixer.kv_spec() for L in self.layers]

    def activation_dtype(self) -> torch.dtype:
        return self.dtype

    # ---- forward ----
    def forward(self, input_ids: torch.Tensor, kv_k, kv_v, meta,
                taps: Optional[list] = None) -> torch.Tensor:
        """-> final-normed hidden [T, W]. `taps`, if a list, receives the
        fp32 residual stream after every layer."""
        cfg = self.cfg
        T, eps = input_ids.shape[0], cfg.norm_eps
        x = torch.empty(T, cfg.width, dtype=torch.float32,
                        device=input_ids.device)
        h = torch.empty(T, cfg.width, dtype=self.dtype, device=x.device)
        # the norm that follows layer i
        after = [L.norm1 for L in self.layers][1:] + [self.final_norm]
        first = self.layers[0].norm1 if len(self.layers) else self.final_norm
        ops.embed_rmsnorm(x, h, input_ids, self.embed, self.embed_norm, first,
                          1.0, eps)
        for i, layer in enumerate(self.layers):
            y = layer.mixer(h, kv_k[i], None, meta, kv_v[i])
            h = torch.empty_like(h)
            if layer.ff is not None:
                ops.residual_add_rmsnorm(x, y, None, layer.norm2, 1.0, eps, h)
                y = layer.ff(h, input_ids, meta)
                h = torch.empty_like(h)
            ops.residual_add_rmsnorm(x, y, None, after[i], 1.0, eps, h)
            if taps is not None:
                taps.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear_f32(hidden, self.head)
