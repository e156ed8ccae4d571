"""Decoders whose layers choose their own mixer, with a 32-bit residual stream and layers that run again with the weights of
another one.  Two designs of a layer:

Fivitar (``HybridDecoder``), norms on the sublayers' outputs and gated sublayers:
    x <- x + norm1(mixer(x) * sigmoid(rg1 x + b1)),   x <- x + norm2(ff(x) * sigmoid(rg2 x + b2))
Fekulix (``PreNormDecoder``), a dynamic tanh on the sublayers' inputs:
    x <- x + mixer(norm1(x)),   x <- x + ff(norm2(x))

Every product that reads the same input is one matrix: [mixer inputs | rg1] and [up | rg2].  A step of several tokens runs
them as library products over all rows; a one-token step runs on the library's GEMV and step kernels, touches only the
position in device memory, and can be captured in a HIP graph."""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Optional

import torch
import torch.nn as nn

from . import mixer_ops as M
from .cache import SequenceState
from .mixers import MIXER_TYPES, Workspace


@dataclass
class LayerConfig:
    type: str
    mixer: dict
    ff: Optional[int] = None                 # None: no feed-forward
    weights_of: Optional[int] = None         # index of the layer whose weights this one runs with


@dataclass
class HybridConfig:
    vocab_size: int
    dim: int
    layers: list = field(default_factory=list)
    norm_eps: float = 1e-6
    logit_scale: float = 1.0
    block_size: int = 1 << 20                # no learned positions: bounded by the cache alone
    model_name: Optional[str] = None

    @classmethod
    def from_dict(cls, cfg: dict) -> "HybridConfig":
        layers = []
        for i, l in enumerate(cfg["layers"]):
            mlp = l.get("mlp")
            if l["type"] not in MIXER_TYPES:
                raise ValueError(f"layer {i}: unknown mixer {l['type']!r}, available: {sorted(MIXER_TYPES)}")
            if mlp is not None and mlp["kind"] != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward {mlp['kind']!r}")
            layers.append(LayerConfig(l["type"], l["mixer"], None if mlp is None else mlp["ff"], l.get("weights_of")))
        return cls(vocab_size=cfg["vocab"], dim=cfg["width"], layers=layers, norm_eps=cfg["norm"]["eps"],
                   logit_scale=cfg.get("logit_scale", 1.0), model_name=cfg.get("architecture"))

    @property
    def n_layer(self) -> int:
        return len(self.layers)

    def source(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        seen = set()
        while self.layers[i].weights_of is not None:
            if i in seen:
                raise ValueError(f"layer {i}: weights_of refers back to itself")
            seen.add(i)
            i = self.layers[i].weights_of
        return i


def _stack(parts, dtype, device):
    """Rows of several matrices in one, each part padded with zero rows to a multiple of 8; the first row of each part."""
    offsets, at = [], 0
    for w in parts:
        offsets.append(at)
        at += (w.shape[0] + 7) // 8 * 8
    out = torch.zeros(at, parts[0].shape[1], dtype=dtype, device=device)
    for o, w in zip(offsets, parts):
        out[o:o + w.shape[0]] = w
    return out, offsets


class HybridLayer(nn.Module):
    """The weights of one layer (shared by all runs of it): the mixer with its stacked input and its output projections."""

    def __init__(self, cfg: LayerConfig, dim: int, eps: float, workspace: Workspace):
        super().__init__()
        self.dim, self.eps, self.ff = dim, eps, cfg.ff
        self.mixer = MIXER_TYPES[cfg.type](cfg.mixer, workspace)

    def fit(self, shapes: dict) -> None:
        self.mixer.fit({n[4:]: s for n, s in shapes.items() if n.startswith("mix.")})

    def weight_shapes(self) -> dict:
        return {"mix." + n: shape for n, shape in self.mixer.weight_shapes(self.dim).items()}

    def load_mixer(self, w: dict, also, dtype, device):
        """Stacks the mixer's inputs and the layer's tensors `also`; returns the first rows of the latter."""
        names = [n for n, _ in self.mixer.inputs]
        stacked, offs = _stack([w["mix." + n] for n in names] + [w[n] for n in also], dtype, device)
        self.register_buffer("w_in", stacked)
        rest = {n[4:]: t.to(device=device, dtype=dtype).contiguous() for n, t in w.items()
                if n.startswith("mix.") and n[4:] not in names}
        self.register_buffer("w_o", self.mixer.output(rest))
        self.mixer.bind(rest, dict(zip(names, offs)), self.eps)
        return offs[len(names):]

    def keep(self, w: dict, names, dtype, device) -> None:
        for n in names:
            self.register_buffer(n.replace(".", "_"), w[n].to(device=device, dtype=dtype).contiguous())

    @staticmethod
    def product(w, a):
        if a.shape[0] > 1:
            return torch.mm(a, w.t())
        out = torch.empty(1, w.shape[0], dtype=a.dtype, device=a.device)
        M.gemv(w, a, out)
        return out

    def mix(self, h, state, pos, start):
        """(the mixer's result behind its output projection, the stacked products of its input)."""
        proj = self.product(self.w_in, h)
        read = torch.empty(h.shape[0], self.mixer.width, dtype=h.dtype, device=h.device)
        self.mixer(proj, state, pos, start, read)
        return self.product(self.w_o, read), proj


class GatedPostLayer(HybridLayer):
    """Gated sublayers with the norm on their outputs, xIELU."""

    def weight_shapes(self) -> dict:
        d, s = self.dim, super().weight_shapes()
        s.update({"norm1": (d,), "rg1": (d, d), "rg1.b": (d,)})
        if self.ff is not None:
            s.update({"mlp.up": (self.ff, d), "mlp.down": (d, self.ff), "mlp.act": (2,), "norm2": (d,), "rg2": (d, d), "rg2.b": (d,)})
        return s

    def load(self, w: dict, dtype, device) -> None:
        self.gate1, = self.load_mixer(w, ["rg1"], dtype, device)
        self.keep(w, ["norm1", "rg1.b"], dtype, device)
        if self.ff is not None:
            stacked, offs = _stack([w["mlp.up"], w["rg2"]], dtype, device)
            self.register_buffer("w_up", stacked)
            self.gate2 = offs[-1]
            self.keep(w, ["mlp.down", "mlp.act", "norm2", "rg2.b"], dtype, device)

    def forward(self, x, x_e, state, pos, start, after=(None, None)):
        """x [rows, dim] fp32, updated in place; x_e the same as the products read it (x itself in float32).  after: weight
        and result of a norm behind the layer."""
        copy = None if x_e.dtype == torch.float32 else x_e
        y, proj = self.mix(x_e, state, pos, start)
        last = after if self.ff is None else (None, None)
        M.gated_residual(x, y, proj[:, self.gate1:], proj.shape[1], self.rg1_b, self.norm1, copy, self.eps, *last)
        if self.ff is None:
            return
        if x.shape[0] == 1:
            up = torch.empty(1, self.w_up.shape[0], dtype=x_e.dtype, device=x.device)
            M.gemv(self.w_up, x_e, up, self.mlp_act, self.ff)
            act = up[:, :self.ff]
        else:
            up = torch.mm(x_e, self.w_up.t())
            act = torch.empty(x.shape[0], self.ff, dtype=x_e.dtype, device=x.device)
            M.activation(up, self.ff, self.mlp_act, act)
        M.gated_residual(x, self.product(self.mlp_down, act), up[:, self.gate2:], up.shape[1], self.rg2_b, self.norm2, copy, self.eps, *after)


class PreTanhLayer(HybridLayer):
    """Sublayers behind a dynamic tanh, GELU."""

    def weight_shapes(self) -> dict:
        d, s = self.dim, super().weight_shapes()
        s.update(tanh_norm_shapes("norm1", d))
        if self.ff is not None:
            s.update({"mlp.up": (self.ff, d), "mlp.down": (d, self.ff), **tanh_norm_shapes("norm2", d)})
        return s

    def load(self, w: dict, dtype, device) -> None:
        self.load_mixer(w, [], dtype, device)
        names = list(tanh_norm_shapes("norm1", self.dim))
        if self.ff is not None:
            names += ["mlp.up", "mlp.down", *tanh_norm_shapes("norm2", self.dim)]
        self.keep(w, names, dtype, device)

    @property
    def first_norm(self):
        return self.norm1_alpha, self.norm1, self.norm1_b

    def forward(self, x, h, state, pos, start, after):
        """x [rows, dim] fp32, updated in place; h: norm1 of it on entry, the norm `after` of the result on return."""
        y, _ = self.mix(h, state, pos, start)
        if self.ff is None:
            M.residual_tanh(x, y, after, h)
            return
        M.residual_tanh(x, y, (self.norm2_alpha, self.norm2, self.norm2_b), h)
        if x.shape[0] == 1:
            up = torch.empty(1, self.ff, dtype=h.dtype, device=x.device)
            M.gemv(self.mlp_up, h, up, None, self.ff, M.ACT_GELU_TANH)
        else:
            up = torch.mm(h, self.mlp_up.t())
            M.activation(up, self.ff, None, up, M.ACT_GELU_TANH)
        M.residual_tanh(x, self.product(self.mlp_down, up), after, h)


def tanh_norm_shapes(name: str, dim: int) -> dict:
    return {name: (dim,), name + ".b": (dim,), name + ".alpha": ()}


class HybridDecoder(nn.Module):
    layer_class = GatedPostLayer

    def __init__(self, dtype, config: HybridConfig, device="cuda"):
        super().__init__()
        if dtype not in (torch.float32, torch.bfloat16):
            raise ValueError("this model runs in float32 or bfloat16")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.workspace = Workspace(self.device)
        self.weights = nn.ModuleDict({str(i): self.layer_class(l, config.dim, config.norm_eps, self.workspace)
                                      for i, l in enumerate(config.layers) if l.weights_of is None})
        self.max_batch_size = self.max_seq_length = -1
        self.decode_kernels = self.device.type == "cuda"
        self.state = None

    @classmethod
    def from_config(cls, cfg: dict, dtype, device="cuda") -> "HybridDecoder":
        return cls(dtype, HybridConfig.from_dict(cfg), device)

    def layer(self, i: int) -> HybridLayer:
        return self.weights[str(self.config.source(i))]

    def weight_shapes(self) -> dict:
        d, v = self.config.dim, self.config.vocab_size
        s = {"embed": (v, d), "head": (v, d), **self.final_norm_shapes()}
        for i, layer in self.weights.items():
            s.update({f"l{i}.{n}": shape for n, shape in layer.weight_shapes().items()})
        return s

    def final_norm_shapes(self) -> dict:
        return {"final.norm": (self.config.dim,)}

    def load_weights(self, w: dict) -> None:
        """Tensors by checkpoint name."""
        for i, layer in self.weights.items():
            p = f"l{i}."
            layer.fit({n[len(p):]: tuple(t.shape) for n, t in w.items() if n.startswith(p)})
        for name, shape in self.weight_shapes().items():
            if name not in w:
                raise KeyError(f"tensor {name} is missing")
            if tuple(w[name].shape) != tuple(shape):
                raise ValueError(f"tensor {name} has shape {tuple(w[name].shape)}, expected {tuple(shape)}")
        put = lambda t: t.to(device=self.device, dtype=self.dtype).contiguous()
        for name in ("embed", "head", *self.final_norm_shapes()):
            self.register_buffer(name.replace(".", "_"), put(w[name]))
        for i, layer in self.weights.items():
            p = f"l{i}."
            layer.load({n[len(p):]: t for n, t in w.items() if n.startswith(p)}, self.dtype, self.device)

    def init_random_weights(self, seed: int = 0) -> None:
        """Random tensors of the magnitudes a trained model has (matrices keep the scale of their input)."""
        gen = torch.Generator(device=self.device).manual_seed(seed)
        w = {}
        for name, shape in self.weight_shapes().items():
            t = torch.randn(shape, generator=gen, device=self.device)
            if name == "embed" or name.endswith((".b", "A_log", "dt_bias", ".act", ".sink")) and len(shape) == 1:
                pass
            elif len(shape) == 0:
                t = 0.5 + 0.1 * t
            elif len(shape) == 1:
                t = 1 + 0.1 * t
            else:
                t = t / shape[1] ** 0.5
            w[name] = t.to(self.dtype)
        self.load_weights(w)

    def setup_caches(self, max_batch_size: int, max_seq_length: int) -> None:
        if max_batch_size != 1:
            raise ValueError("one sequence at a time")
        if self.max_seq_length >= max_seq_length:
            return
        self.max_batch_size, self.max_seq_length = 1, max_seq_length
        self.state = SequenceState([self.layer(i).mixer.new_state(max_seq_length, self.dtype, self.device)
                                    for i in range(self.config.n_layer)], max_seq_length)

    def forward(self, idx: torch.Tensor, input_pos: torch.Tensor, start: Optional[int] = None, want=None) -> torch.Tensor:
        """idx [1, S] token ids, input_pos [S] neighbouring positions (int64); returns logits [1, S, vocab], or
        [1, len(want), vocab] for the places `want` among the S tokens.  `start` is the first position where the caller
        knows it (read back from the device otherwise, with S > 1)."""
        assert self.max_seq_length > 0, "Caches must be initialized first"
        S = idx.shape[1]
        assert idx.shape[0] == 1 and input_pos.numel() == S, "one sequence, one position per token"
        if S > 1:
            start = int(input_pos[0]) if start is None else start
            assert 0 <= start and start + S <= self.max_seq_length, f"{start} + {S} positions do not fit a cache of {self.max_seq_length}"
        x, h = self.open(idx.contiguous().view(-1))
        n_layer = self.config.n_layer
        for i in range(n_layer):
            self.layer(i)(x, h, self.state.entries[i], input_pos, start, self.after(i, h))
        if S > 1 and want is not None:
            if len(want) == 0:
                return torch.empty(1, 0, self.config.vocab_size, dtype=self.dtype, device=idx.device)
            rows = torch.as_tensor(want, dtype=torch.int64, device=idx.device)
            x, h = x[rows], h[rows]
        return self.logits(self.close(x, h))

    def logits(self, normed: torch.Tensor) -> torch.Tensor:
        n, v = normed.shape[0], self.config.vocab_size
        out = torch.empty(n, v, dtype=self.dtype, device=normed.device)
        if n == 1:
            M.gemv(self.head, normed, out, scale=self.config.logit_scale)
        elif self.config.logit_scale == 1.0:
            torch.mm(normed, self.head.t(), out=out)
        else:
            torch.addmm(out, normed, self.head.t(), beta=0.0, alpha=self.config.logit_scale, out=out)
        return out.view(1, n, v)

    # what a design has around its layers
    def open(self, tokens: torch.Tensor):
        """(residual stream [rows, dim] in float32, what the first layer reads)."""
        x = torch.empty(tokens.numel(), self.config.dim, dtype=torch.float32, device=tokens.device)
        x_e = x if self.dtype == torch.float32 else torch.empty(x.shape, dtype=self.dtype, device=x.device)
        M.embed(self.embed, tokens, x, None if x_e is x else x_e)
        return x, x_e

    def after(self, i: int, h: torch.Tensor):
        """The norm behind layer i: a one-token step takes the model's with its last layer."""
        self.normed = None
        if h.shape[0] == 1 and i == self.config.n_layer - 1:
            self.normed = torch.empty(h.shape, dtype=self.dtype, device=h.device)
        return (None, None) if self.normed is None else (self.final_norm, self.normed)

    def close(self, x: torch.Tensor, h: torch.Tensor) -> torch.Tensor:
        """The rows that the head reads."""
        normed, self.normed = getattr(self, "normed", None), None
        if normed is None:
            normed = torch.empty(x.shape, dtype=self.dtype, device=x.device)
            M.rmsnorm(x, self.final_norm, normed, self.config.norm_eps)
        return normed


class PreNormDecoder(HybridDecoder):
    """Layers that leave the next layer's (or the model's) norm of the residual stream behind them."""
    layer_class = PreTanhLayer

    def final_norm_shapes(self) -> dict:
        return tanh_norm_shapes("final.norm", self.config.dim)

    def norm_ahead_of(self, i: int):
        if i < self.config.n_layer:
            return self.layer(i).first_norm
        return self.final_norm_alpha, self.final_norm, self.final_norm_b

    def open(self, tokens):
        x = torch.empty(tokens.numel(), self.config.dim, dtype=torch.float32, device=tokens.device)
        h = torch.empty(x.shape, dtype=self.dtype, device=x.device)
        M.embed(self.embed, tokens, x, h, self.norm_ahead_of(0))
        return x, h

    def after(self, i, h):
        return self.norm_ahead_of(i + 1)

    def close(self, x, h):
        return h
