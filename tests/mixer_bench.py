"""A mixer on the GPU with random weights beside the oracle's read-out of it (before the output projection)."""
from __future__ import annotations

import torch

from decdec_amd import mixers as X
from oracle import hybrid_oracle as O
import hybrid_cases as cases

TOL = {torch.float32: 2e-5, torch.bfloat16: 2.5e-2}


def close(got, want, dtype, what="", factor=1.0):
    got, want = got.detach().double().cpu(), want.double().cpu()
    assert torch.isfinite(got).all(), what
    err = float((got - want).abs().max() / (want.abs().max() + 1e-9))
    assert err <= TOL[dtype] * factor, (what, err)


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def portions(T, *sizes):
    out, i = [], 0
    while sum(out) < T:
        out.append(min(sizes[i % len(sizes)], T - sum(out)))
        i += 1
    return out


def grouped(m, workspace):
    return X.GroupedAttention(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], m["rot"]["base"], rope_dims=m["rot"]["dims"],
                              sink=m.get("sink", 0.0), qk_norm=m.get("qk_norm", True), gated=m.get("gated", True), out_scale=m.get("out_scale", 1.0))


def gated_linear(m, workspace):
    return X.LinearRecurrence(m["heads"], m["dim"], m["vdim"], workspace, channel=True, tau=m["tau"], out_scale=m.get("out_scale", 1.0))


def grouped_readout(h, w, m, eps):
    return m.get("out_scale", 1.0) * O.gated_attention(h, w, m, eps)


def gated_linear_readout(h, w, m, eps):
    return m.get("out_scale", 1.0) * O.gated_linear(h, w, m, eps)


# mixers that a design only has beside another one
ALONE = {"grouped": (grouped, grouped_readout), "gated_linear": (gated_linear, gated_linear_readout)}


class Bench:
    """A mixer on the GPU with random weights, and the oracle's read-out (before the output projection)."""

    def __init__(self, kind, m, dtype, T, seed=0, width=40, eps=1e-5, edit=None, max_seq=None):
        g = torch.Generator().manual_seed(seed)
        self.w = {n: cases.random_tensor("mix." + n, s, g) for n, s in cases.mixer_shapes(kind, m, width).items()}
        if "o" in self.w:
            self.w["o"] = torch.eye(self.w["o"].shape[1]).to(torch.bfloat16)      # the oracle's output is the read-out itself
        else:                                                                     # side by side: the read-outs one after another
            n = [self.w[side + ".o"].shape[1] for side in ("left", "right")]
            eye = torch.eye(sum(n)).to(torch.bfloat16)
            self.w["left.o"], self.w["right.o"] = eye[:, :n[0]], eye[:, n[0]:]
        self.h = torch.randn(T, width, generator=g).to(torch.bfloat16)
        self.m, self.kind, self.eps, self.dtype, self.T = m, kind, eps, dtype, T
        if edit:
            edit(self)
        make = ALONE[kind][0] if kind in ALONE else X.MIXER_TYPES[kind]
        self.mixer = make(m, X.Workspace(torch.device("cuda")))
        self.mixer.fit({n: tuple(t.shape) for n, t in self.w.items()})
        names, off = [n for n, _ in self.mixer.inputs], {}
        for n, r in self.mixer.inputs:
            off[n] = sum(off_r for _, off_r in self.mixer.inputs[:names.index(n)])
        rows = sum(r for _, r in self.mixer.inputs)
        # projections in float64, rounded once to the storage type; the oracle sees the unrounded ones
        proj = torch.cat([self.h.double() @ self.w[n].double().T for n in names], 1)
        self.proj = torch.zeros(T, (rows + 7) // 8 * 8, dtype=dtype)
        self.proj[:, :rows] = proj.to(dtype)
        self.proj = self.proj.cuda()
        self.mixer.bind({n: t.to(dtype).cuda() for n, t in self.w.items() if n not in names and n.split(".")[-1] != "o"}, off, eps)
        self.max_seq = max_seq or T
        self.new_state()

    def new_state(self):
        self.state = self.mixer.new_state(self.max_seq, self.dtype, "cuda")

    def want(self):
        f = ALONE[self.kind][1] if self.kind in ALONE else O.MIXERS[self.kind]
        return f(self.h.double(), {n: t.double() for n, t in self.w.items()}, self.m, self.eps)

    def run(self, portions, t=0):
        out = []
        for n in portions:
            y = torch.empty(n, self.mixer.width, dtype=self.dtype, device="cuda")
            self.mixer(self.proj[t:t + n].contiguous(), self.state, torch.tensor([t], device="cuda"), t, y)
            out.append(y)
            t += n
        return torch.cat(out)
