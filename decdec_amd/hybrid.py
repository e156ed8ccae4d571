"""Decoder whose layers choose their own mixer, with a 32-bit residual stream, norms on the sublayers' outputs, gated
sublayers and layers that run again with the weights of another one (the Fivitar design).

    x <- x + norm1(mixer(x) * sigmoid(rg1 x + b1)),   x <- x + norm2(ff(x) * sigmoid(rg2 x + b2))

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
        return cls(vocab_size=cfg["vocab"], dim=cfg["width"], layers=layers, norm_eps=cfg["norm"]["eps"], model_name=cfg.get("architecture"))

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
    """Rows of several matrices in one, padded with zero rows to a multiple of 8; the first row of each part."""
    offsets, at = [], 0
    for w in parts:
        offsets.append(at)
        at += w.shape[0]
    out = torch.zeros((at + 7) // 8 * 8, parts[0].shape[1], dtype=dtype, device=device)
    for o, w in zip(offsets, parts):
        out[o:o + w.shape[0]] = w
    return out, offsets


class HybridLayer(nn.Module):
    """The weights of one layer (shared by all runs of it)."""

    def __init__(self, cfg: LayerConfig, dim: int, eps: float, workspace: Workspace):
        super().__init__()
        self.dim, self.eps, self.ff = dim, eps, cfg.ff
        self.mixer = MIXER_TYPES[cfg.type](cfg.mixer, workspace)

    def weight_shapes(self) -> dict:
        d = self.dim
        s = {"mix." + n: shape for n, shape in self.mixer.weight_shapes(d).items()}
        s.update({"norm1": (d,), "rg1": (d, d), "rg1.b": (d,)})
        if self.ff is not None:
            s.update({"mlp.up": (self.ff, d), "mlp.down": (d, self.ff), "mlp.act": (2,), "norm2": (d,), "rg2": (d, d), "rg2.b": (d,)})
        return s

    def load(self, w: dict, dtype, device) -> None:
        names = [n for n, _ in self.mixer.inputs]
        stacked, offs = _stack([w["mix." + n] for n in names] + [w["rg1"]], dtype, device)
        self.register_buffer("w_in", stacked)
        self.gate1 = offs[-1]
        rest = {n[4:]: t.to(device=device, dtype=dtype).contiguous() for n, t in w.items()
                if n.startswith("mix.") and n[4:] not in names}
        self.register_buffer("w_o", rest.pop("o"))
        self.mixer.bind(rest, dict(zip(names, offs)), self.eps)
        keep = ["norm1", "rg1.b"]
        if self.ff is not None:
            stacked, offs = _stack([w["mlp.up"], w["rg2"]], dtype, device)
            self.register_buffer("w_up", stacked)
            self.gate2 = offs[-1]
            keep += ["mlp.down", "mlp.act", "norm2", "rg2.b"]
        for n in keep:
            self.register_buffer(n.replace(".", "_"), w[n].to(device=device, dtype=dtype).contiguous())

    def forward(self, x, x_e, state, pos, start, final=(None, None)):
        """x [rows, dim] fp32, updated in place; x_e the same as the products read it (x itself in float32)."""
        rows, dt = x.shape[0], x_e.dtype
        one = rows == 1
        new = lambda n: torch.empty(rows, n, dtype=dt, device=x.device)

        def product(w, a):
            if not one:
                return torch.mm(a, w.t())
            out = new(w.shape[0])
            M.gemv(w, a, out)
            return out
        copy = None if x_e.dtype == torch.float32 else x_e
        proj = product(self.w_in, x_e)
        read = new(self.mixer.width)
        self.mixer(proj, state, pos, start, read)
        last = final if self.ff is None else (None, None)
        M.gated_residual(x, product(self.w_o, read), proj[:, self.gate1:], proj.shape[1], self.rg1_b, self.norm1, copy, self.eps, *last)
        if self.ff is None:
            return
        if one:
            up = new(self.w_up.shape[0])
            M.gemv(self.w_up, x_e, up, self.mlp_act, self.ff)
            act = up[:, :self.ff]
        else:
            up, act = torch.mm(x_e, self.w_up.t()), new(self.ff)
            M.xielu(up, self.ff, self.mlp_act, act)
        M.gated_residual(x, product(self.mlp_down, act), up[:, self.gate2:], up.shape[1], self.rg2_b, self.norm2, copy, self.eps, *final)


class HybridDecoder(nn.Module):
    def __init__(self, dtype, config: HybridConfig, device="cuda"):
        super().__init__()
        if dtype not in (torch.float32, torch.bfloat16):
            raise ValueError("this model runs in float32 or bfloat16")
        self.config, self.dtype, self.device = config, dtype, torch.device(device)
        self.workspace = Workspace(self.device)
        self.weights = nn.ModuleDict({str(i): HybridLayer(l, config.dim, config.norm_eps, self.workspace)
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
        s = {"embed": (v, d), "final.norm": (d,), "head": (v, d)}
        for i, layer in self.weights.items():
            s.update({f"l{i}.{n}": shape for n, shape in layer.weight_shapes().items()})
        return s

    def load_weights(self, w: dict) -> None:
        """Tensors by checkpoint name."""
        for name, shape in self.weight_shapes().items():
            if name not in w:
                raise KeyError(f"tensor {name} is missing")
            if tuple(w[name].shape) != tuple(shape):
                raise ValueError(f"tensor {name} has shape {tuple(w[name].shape)}, expected {tuple(shape)}")
        put = lambda t: t.to(device=self.device, dtype=self.dtype).contiguous()
        self.register_buffer("embed", put(w["embed"]))
        self.register_buffer("final_norm", put(w["final.norm"]))
        self.register_buffer("head", put(w["head"]))
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
        S, d = idx.shape[1], self.config.dim
        assert idx.shape[0] == 1 and input_pos.numel() == S, "one sequence, one position per token"
        if S > 1:
            start = int(input_pos[0]) if start is None else start
            assert 0 <= start and start + S <= self.max_seq_length, f"{start} + {S} positions do not fit a cache of {self.max_seq_length}"
        x = torch.empty(S, d, dtype=torch.float32, device=idx.device)
        x_e = x if self.dtype == torch.float32 else torch.empty(S, d, dtype=self.dtype, device=idx.device)
        M.embed(self.embed, idx.contiguous().view(-1), x, None if x_e is x else x_e)
        n_layer = self.config.n_layer
        normed = torch.empty(S, d, dtype=self.dtype, device=idx.device) if S == 1 else None
        for i in range(n_layer):
            final = (self.final_norm, normed) if S == 1 and i == n_layer - 1 else (None, None)
            self.layer(i)(x, x_e, self.state.entries[i], input_pos, start, final)
        if S == 1:
            if n_layer == 0:
                M.rmsnorm(x, self.final_norm, normed, self.config.norm_eps)
            logits = torch.empty(1, 1, self.config.vocab_size, dtype=self.dtype, device=idx.device)
            M.gemv(self.head, normed, logits)
            return logits
        if want is not None and len(want) == 0:
            return torch.empty(1, 0, self.config.vocab_size, dtype=self.dtype, device=idx.device)
        if want is not None:
            x = x[torch.as_tensor(want, dtype=torch.int64, device=idx.device)]
        normed = torch.empty(x.shape, dtype=self.dtype, device=idx.device)
        M.rmsnorm(x, self.final_norm, normed, self.config.norm_eps)
        return torch.mm(normed, self.head.t()).view(1, x.shape[0], -1)
