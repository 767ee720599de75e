"""Noridra: a decoder that norms AFTER the residual sum,

    x <- norm1(alpha x + ls1 * mixer(in1(x)))
    x <- norm2(alpha x + ls2 * ff(in2(x))) ,

where norm is an RMS norm in equal runs of the row, ls a factor per entry of
the sublayer's output, and in(x) = x + conv(x) a short causal convolution of
the fp32 residual stream itself over time. Layers pick one of three mixers:
`delta` (gated delta rule), `attention` (chunk-local softmax attention whose
values are its unnormed keys, with capped scores, a logarithmic distance bias
and a sink) or `mamba1` (selective scan); the feed-forward is a mixture of
silu-gated experts chosen by sigmoid scores that multiply the experts' inputs;
a layer may have none. A learned position row is added to the embedding.

Everything a checkpoint's config.json states (sizes, the order of layers,
constants) is read from it. The attention layers keep one key row per token in
the paged cache; the recurrences, the convolution tails of the mixers and of
both sublayers' inputs live in the engine's state slots (fp32).

Tensor parallelism is not implemented for this family (tp_size must be 1).
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional

import torch
import torch.nn as nn

from kukeon_amd import ops
from kukeon_amd import parallel
from kukeon_amd.models.feedforward import FFCfg, RoutedMoE
from kukeon_amd.models.mixers import (DeltaCfg, DeltaMixer, SelectiveCfg,
                                      SelectiveMixer, SinkAttention,
                                      SinkAttnCfg)

_DTYPES = {"bf16": torch.bfloat16, "bfloat16": torch.bfloat16,
           "fp32": torch.float32, "float32": torch.float32}

MIXERS = {"delta": DeltaMixer, "attention": SinkAttention,
          "mamba1": SelectiveMixer}


@dataclass
class NoridraLayerCfg:
    type: str                # "delta" | "attention" | "mamba1"
    mixer: object
    mlp: Optional[FFCfg]


@dataclass
class NoridraConfig:
    family = "noridra"
    name: str = "noridra"
    width: int = 1024
    vocab_size: int = 32000
    norm_eps: float = 1e-6
    norm_groups: int = 1
    alpha: float = 1.0       # factor of the residual stream in every sum
    canon_taps: int = 4      # taps of the sublayers' input convolution
    max_positions: int = 0   # rows of the learned position table
    layers: List[NoridraLayerCfg] = field(default_factory=list)

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
    def from_json(c: dict, name: str = "noridra") -> "NoridraConfig":
        layers = []
        for i, L in enumerate(c["layers"]):
            kind = L.get("type")
            m = L["mixer"]
            if kind == "delta":
                mix = DeltaCfg(heads=int(m["heads"]),
                               kv_heads=int(m["kv_heads"]),
                               dim=int(m["dim"]), vdim=int(m["vdim"]),
                               conv=int(m.get("conv") or 0))
            elif kind == "attention":
                mix = SinkAttnCfg(
                    heads=int(m["heads"]), kv_heads=int(m["kv_heads"]),
                    dim=int(m["dim"]), scale=float(m["scale"]),
                    softcap=float(m.get("softcap") or 0.0),
                    chunk=int((m.get("mask") or {}).get("size") or 0))
                if m.get("vdim") is not None and int(m["vdim"]) != mix.dim:
                    raise ValueError(f"layer {i}: values are the keys, so "
                                     "vdim must equal dim")
            elif kind == "mamba1":
                mix = SelectiveCfg(inner=int(m["inner"]),
                                   state=int(m["state"]),
                                   dt_rank=int(m["dt_rank"]),
                                   conv=int(m.get("conv") or 0))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            mlp = None
            if L.get("mlp"):
                f = L["mlp"]
                if f.get("kind", "moe") != "moe":
                    raise ValueError(f"layer {i}: unknown feed-forward kind "
                                     f"{f.get('kind')!r}")
                mlp = expert_cfg(int(f["expert"]["ff"]),
                                 int(f["router"]["experts"]),
                                 int(f["router"]["top"]))
            layers.append(NoridraLayerCfg(kind, mix, mlp))
        n = c["norm"]
        return NoridraConfig(
            name=name, width=int(c["width"]), vocab_size=int(c["vocab"]),
            norm_eps=float(n["eps"]), norm_groups=int(n.get("groups") or 1),
            alpha=float(c.get("postln_alpha", 1.0)),
            canon_taps=int((c.get("canon") or {}).get("taps") or 0),
            max_positions=int(c.get("max_positions") or 0), layers=layers)


def expert_cfg(ff: int, experts: int, top: int) -> FFCfg:
    """Silu-gated experts, sigmoid scores as they are, on the inputs."""
    return FFCfg("moe", ff, experts=experts, top=top, act="silu",
                 score="sigmoid", weigh_input=True)


def noridra_bench(width=4096, layers=8, heads=32, kv_heads=8, ff=14336,
                  vocab=128256, chunk=8192, experts=16, top=2,
                  max_positions=8192, name="noridra-8b-like"
                  ) -> NoridraConfig:
    """A layer stack at real-model sizes (random weights) for throughput
    runs: periods of delta rule (heads of 128, two value heads per key head),
    attention (heads of 128), selective scan (twice the width, 16 states) and
    delta rule. Every feed-forward has `ff` active rows in `top` routed
    experts, chosen among `experts` in every second layer and among `top`
    (all chosen: a dense layer in effect) in the others."""
    hd = 128 if width >= 1024 else 32
    vh = max(2, width // hd)
    ls = []
    for i in range(layers):
        kind = ("delta", "attention", "mamba1", "delta")[i % 4]
        if kind == "delta":
            mix = DeltaCfg(heads=vh, kv_heads=vh // 2, dim=hd, vdim=hd,
                           conv=4)
        elif kind == "attention":
            mix = SinkAttnCfg(heads=heads, kv_heads=kv_heads, dim=hd,
                              scale=hd ** -0.5, softcap=50.0, chunk=chunk)
        else:
            mix = SelectiveCfg(inner=2 * width, state=16,
                               dt_rank=max(1, width // 16), conv=4)
        ls.append(NoridraLayerCfg(kind, mix, expert_cfg(
            max(8, ff // top // 8 * 8), experts if i % 2 else top, top)))
    return NoridraConfig(name=name, width=width, vocab_size=vocab,
                         norm_eps=1e-6, norm_groups=4, alpha=2.0,
                         canon_taps=4, max_positions=max_positions, layers=ls)


def tensor_shapes(cfg: NoridraConfig) -> Dict[str, tuple]:
    """Names and shapes of a checkpoint of this configuration."""
    W = cfg.width
    out = {"embed": (cfg.vocab_size, W)}
    if cfg.max_positions:
        out["pos"] = (cfg.max_positions, W)
    for i, L in enumerate(cfg.layers):
        p = f"l{i}."
        for q in ("1", "2") if L.mlp is not None else ("1",):
            out[p + "norm" + q] = (W,)
            out[p + "ls" + q] = (W,)
            if cfg.canon_taps:
                out[p + "canon" + q] = (W, cfg.canon_taps)
        for n, s in MIXERS[L.type].tensor_shapes(L.mixer, W).items():
            out[p + "mix." + n] = s
        if L.mlp is not None:
            for n, s in RoutedMoE.tensor_shapes(L.mlp, W,
                                                cfg.vocab_size).items():
                out[p + "mlp." + n] = s
    out["final.norm"] = (W,)
    out["head"] = (cfg.vocab_size, W)
    return out


def random_tensors(cfg: NoridraConfig, seed: int = 0,
                   device="cpu") -> Dict[str, torch.Tensor]:
    """Random bf16 weights at a scale that keeps activations O(1)."""
    on_gpu = torch.device(device).type == "cuda"
    gdev = device if on_gpu else "cpu"
    g = torch.Generator(device=gdev).manual_seed(seed)
    out = {}

    def rn(shp, std=1.0, mean=0.0):
        return mean + torch.randn(shp, generator=g, device=gdev) * std

    for name, shp in tensor_shapes(cfg).items():
        leaf = name.rsplit(".", 1)[-1]
        if leaf.startswith("canon"):
            t = rn(shp, 0.2)
        elif leaf == "conv":
            t = rn(shp, 0.3, 1.0 / shp[1])
        elif leaf == "A_log":
            t = rn(shp, 0.5, 0.0 if len(shp) == 1 else 0.5)
        elif leaf == "dt_bias" or name.endswith("dt.b"):
            t = rn(shp, 0.5, -2.0)
        elif leaf in ("r1", "r2"):
            t = torch.rand(shp, generator=g, device=gdev) * 0.5 + 0.1
        elif name == "pos":
            t = rn(shp, 0.1)
        elif name.endswith("conv.b"):
            t = rn(shp, 0.1)
        elif len(shp) == 2:
            std = shp[1] ** -0.5 if name != "embed" else 1.0
            t = rn(shp, 2.0 * std if leaf == "router" else std)
        else:
            t = rn(shp, 0.1, 1.0)
        out[name] = t.to(torch.bfloat16).to(device)
    return out


class Sublayer:
    """What surrounds one mixer or feed-forward: the input convolution's
    taps [taps, W], the output's factors, the norm after the sum (fp32), and
    where the convolution's tail sits in the layer's state pieces."""

    def __init__(self, cfg: NoridraConfig, t, p: str, q: str, piece: int,
                 device):
        f32 = dict(device=device, dtype=torch.float32)
        self.norm = t[p + "norm" + q].to(**f32).contiguous()
        self.ls = t[p + "ls" + q].to(**f32).contiguous()
        if cfg.canon_taps:
            self.taps_w = t[p + "canon" + q].to(**f32).t().contiguous()
        else:                # no convolution: one tap of weight 0
            self.taps_w = torch.zeros(1, cfg.width, **f32)
        self.piece = piece


class NoridraLayer(nn.Module):
    """State pieces: input tail of the mixer, input tail of the feed-forward
    (if there is one), then the mixer's own."""

    def __init__(self, cfg: NoridraConfig, idx: int,
                 t: Dict[str, torch.Tensor], device, dtype):
        super().__init__()
        L = cfg.layers[idx]
        p = f"l{idx}."
        W = cfg.width
        self.sub1 = Sublayer(cfg, t, p, "1", 0, device)
        self.mixer = MIXERS[L.type](L.mixer, W, cfg.norm_eps, t, p + "mix.",
                                    device, dtype)
        self.ff = None
        self.own = 1
        if L.mlp is not None:
            self.sub2 = Sublayer(cfg, t, p, "2", 1, device)
            self.ff = RoutedMoE(L.mlp, W, t, p + "mlp.", device, dtype)
            self.own = 2
        self.tail_shape = (self.sub1.taps_w.shape[0] - 1, W)

    def state_shape(self):
        return [self.tail_shape] * self.own + list(self.mixer.state_shape()
                                                   or [])


class NoridraModel(nn.Module):
    family = "noridra"
    op_groups = ("delta",)      # kernel groups the forward pass needs

    def __init__(self, cfg: NoridraConfig, device="cuda", dtype="bf16",
                 tensors: Optional[Dict[str, torch.Tensor]] = None,
                 max_position: int = 4096, seed: int = 0):
        super().__init__()
        if parallel.tp_size() != 1:
            raise NotImplementedError("Noridra runs with tp_size == 1 only")
        if cfg.width % cfg.norm_groups:
            raise ValueError("norm groups must divide the width")
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
        self.embed = nn.Parameter(tensors["embed"].to(dev).to(dt),
                                  requires_grad=False)
        self.pos = (nn.Parameter(tensors["pos"].to(dev).to(dt),
                                 requires_grad=False)
                    if cfg.max_positions else None)
        self.head = nn.Parameter(tensors["head"].to(dev).to(dt).contiguous(),
                                 requires_grad=False)
        self.layers = nn.ModuleList(
            [NoridraLayer(cfg, i, tensors, dev, dt)
             for i in range(cfg.num_layers)])
        self.final_norm = tensors["final.norm"].to(dev).float().contiguous()
        self.zero_b = torch.zeros(cfg.width, dtype=torch.float32, device=dev)
        self.max_position = cfg.max_positions or max_position

    @classmethod
    def from_checkpoint(cls, model_dir: str, device="cuda", dtype="bf16",
                        max_position: int = 4096):
        from kukeon_amd.models.weights import read_checkpoint
        config, tensors = read_checkpoint(model_dir)
        cfg = NoridraConfig.from_json(config)
        return cfg, cls(cfg, device=device, dtype=dtype, tensors=tensors,
                        max_position=max_position)

    def set_max_position(self, n: int) -> None:
        """Positions are rows of a learned table: there is nothing to
        rebuild, and the table bounds the longest sequence."""
        self.max_position = min(n, self.cfg.max_positions or n)

    # ---- what the engine asks of a model with its own cache layout ----
    def kv_specs(self):
        return [L.mixer.kv_spec() for L in self.layers]

    def state_shapes(self):
        return [L.state_shape() for L in self.layers]

    def activation_dtype(self) -> torch.dtype:
        return self.dtype

    # ---- forward ----
    def _input_conv(self, x, sub: Sublayer, tail, meta, one: bool):
        """h = x + conv(x) over the packed rows; the slots move on."""
        h = torch.empty(x.shape, dtype=self.dtype, device=x.device)
        ops.conv_act(h, x, 0, sub.taps_w, self.zero_b, tail, meta.positions,
                     meta.row_seq, meta.cu_rows, meta.state_slots, 0, one,
                     True)
        if not one and sub.taps_w.shape[0] > 1:
            ops.conv_tail_update(tail, x, 0, self.zero_b, meta.positions,
                                 meta.cu_rows, meta.state_slots)
        return h

    def forward(self, input_ids: torch.Tensor, kv_k, kv_v, meta,
                taps: Optional[list] = None) -> torch.Tensor:
        """-> final-normed hidden [T, W]. `taps`, if a list, receives the
        fp32 residual stream after every layer."""
        cfg = self.cfg
        T = input_ids.shape[0]
        one = meta.max_rows == 1 and T == meta.cu_rows.numel() - 1
        x = torch.empty(T, cfg.width, dtype=torch.float32,
                        device=input_ids.device)
        ops.embed_streams(x.view(T, 1, cfg.width), input_ids, meta.positions,
                          self.embed, self.pos, 1.0)
        # every sublayer in running order with its state
        subs = []
        for i, layer in enumerate(self.layers):
            st = meta.state[i]
            subs.append((layer, layer.sub1, i, st))
            if layer.ff is not None:
                subs.append((layer, layer.sub2, i, st))
        _, sub, _, st = subs[0]
        h = self._input_conv(x, sub, st[sub.piece], meta, one)
        for n, (layer, sub, i, st) in enumerate(subs):
            if sub.piece == 0:
                y = layer.mixer(h, kv_k[i], st[layer.own:], meta, kv_v[i])
            else:
                y = layer.ff(h, input_ids, meta)
            args = (x, y, cfg.alpha, sub.ls, sub.norm, cfg.norm_groups,
                    cfg.norm_eps, meta.positions)
            if n + 1 == len(subs):
                h = torch.empty_like(h)
                ops.postnorm_residual_norm(*args, h, self.final_norm)
            else:
                _, nxt, _, nst = subs[n + 1]
                if one:
                    h = torch.empty_like(h)
                    ops.postnorm_residual_conv(*args, h, nxt.taps_w,
                                               nst[nxt.piece],
                                               meta.state_slots)
                else:
                    ops.postnorm_residual(*args)
                    h = self._input_conv(x, nxt, nst[nxt.piece], meta, False)
            if taps is not None and (n + 1 == len(subs)
                                     or subs[n + 1][2] != i):
                taps.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor) -> torch.Tensor:
        return ops.linear_f32(hidden, self.head)
