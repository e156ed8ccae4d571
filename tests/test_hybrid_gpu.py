"""The Fivitar and Fekulix decoders on the GPU against the plain oracle: logits over cuts of the prompt, states used again, captured
steps, greedy generation through the command line's own path, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from decdec_amd import generate as G, registry
from decdec_amd.generate import DecodeStep, Session
from oracle import hybrid_oracle as O
import hybrid_cases as cases

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
TOL = {torch.float32: 1e-4, torch.bfloat16: 6e-2}
_cache = {}


def _model(name, dtype):
    cfg = cases.CONFIGS[name]()
    w = cases.weights(cfg, seed=len(name))
    m = registry.model_class(cfg).from_config(cfg, dtype)
    m.load_weights(w)
    return m, cfg, w


def _want(name, cfg, w, toks):
    key = (name, tuple(toks))
    if key not in _cache:
        _cache[key] = O.forward(cfg, w, toks)
    return _cache[key]


def _close(got, want, dtype, what=""):
    d = got.double().cpu() - want
    rows = (d - d.mean(-1, keepdim=True)).pow(2).mean(-1) / want.var()
    err, worst = float(rows.mean().sqrt()), float(rows.max().sqrt())
    assert err <= TOL[dtype] and worst <= 4 * TOL[dtype], (what, err, worst)


def _feed(m, toks, sizes, max_tokens=200):
    s, out, at, i = Session(m, max_tokens), [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        out.append(s.feed(toks[at:at + n], range(n)))
        at, i = at + n, i + 1
    s.close()
    return torch.cat(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_logits_do_not_depend_on_the_cut(name, dtype):
    m, cfg, w = _model(name, dtype)
    toks = cases.tokens(cfg, 131)
    want = _want(name, cfg, w, toks)
    for sizes in ((131,), (2,), (1, 64, 2, 3), (63, 5), (65,), (100, 1), (1,)):
        _close(_feed(m, toks, sizes), want, dtype, (name, sizes))


@pytest.mark.parametrize("name", ["odd", "fek_odd"])
def test_residual_after_every_layer(name):
    m, cfg, w = _model(name, torch.float32)
    toks, want, got = cases.tokens(cfg, 70, seed=5), [], []
    O.forward(cfg, w, toks, layers_out=want)
    hooks = [l.register_forward_hook(lambda mod, inp, out: got.append(inp[0].double().cpu())) for l in m.weights.values()]
    Session(m, 100).feed(toks)
    for h in hooks:
        h.remove()
    assert len(got) == len(want)
    for i, (a, b) in enumerate(zip(got, want)):
        assert float((a - b).abs().max() / b.abs().max()) < 1e-5, i


@pytest.mark.parametrize("name", ["odd", "fek_odd"])
def test_a_finished_request_leaves_nothing_behind(name):
    m, cfg, w = _model(name, torch.float32)
    a, b = cases.tokens(cfg, 131), cases.tokens(cfg, 9, seed=2)
    _feed(m, a, (131,))
    first = _feed(m, b, (9,))
    _close(first, _want(name, cfg, w, b), torch.float32)
    _feed(m, a, (50, 1))
    again = _feed(m, b, (9,))
    assert torch.equal(first, again)
    _feed(m, a, (131,))
    _close(_feed(m, b, (1,)), _want(name, cfg, w, b), torch.float32)


@pytest.mark.parametrize("name", ["tiny", "fek_tiny"])
def test_wanted_places_and_limits(name):
    m, cfg, w = _model(name, torch.float32)
    toks = cases.tokens(cfg, 60)
    want = _want(name, cfg, w, toks)
    s = Session(m, 60, portion=16)
    _close(s.feed(toks[:50], [49, 0, 17, 17, 16]), want[[49, 0, 17, 17, 16]], torch.float32)
    assert s.feed(toks[50:51]).shape == (0, cfg["vocab"]) and s.feed(toks[51:57]).shape[0] == 0
    _close(s.feed(toks[57:], [2]), want[[59]], torch.float32)
    with pytest.raises(ValueError, match="do not fit"):
        s.feed([0] * 1000)


@pytest.mark.parametrize("name", ["odd", "tiny", "fek_odd", "fek_tiny"])
def test_graph_replays_equal_eager_steps(name):
    m, cfg, w = _model(name, torch.bfloat16)
    toks = cases.tokens(cfg, 40)
    Session(m, 80).feed(toks)
    start = m.state.snapshot()
    step = DecodeStep(m, max_tokens=16, keep_logits=True)
    step.start(toks[0], 40)
    eager = []
    with torch.no_grad():
        for _ in range(6):
            step._step()
            eager.append(step.logits.clone())
    m.state.restore(start)
    step.start(toks[0], 40)
    step.capture()
    for a, b in zip(m.state.snapshot(), start):
        assert torch.equal(a, b)                          # capturing leaves the sequence where it was
    for want in eager:
        torch.randn(256, 256, device="cuda") @ torch.randn(256, 256, device="cuda")
        step.graph.replay()
        torch.cuda.synchronize()
        assert torch.equal(step.logits, want)


@pytest.mark.parametrize("graph", [True, False])
@pytest.mark.parametrize("name,n", [("odd", 12), ("wide", 8), ("tiny", 150), ("fek_odd", 12), ("fek_wide", 8), ("fek_tiny", 150)])
def test_greedy_generation(name, n, graph):
    m, cfg, w = _model(name, torch.float32)
    prompt = torch.tensor(cases.tokens(cfg, 20, seed=7))
    seq, _ = G.generate(m, prompt.cuda(), n, use_graph=graph)
    seq = seq.tolist()
    assert seq[:20] == prompt.tolist() and len(seq) == 20 + n
    logits = _want(name, cfg, w, seq[:-1])
    for i in range(n):
        row = logits[19 + i]
        assert float(row.max() - row[seq[20 + i]]) < 1e-3 * float(row.std()), i


def _checkpoint(tmp_path, name):
    from safetensors.torch import save_file
    cfg = cases.CONFIGS[name]()
    w = cases.weights(cfg, seed=len(name))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    return cfg, w


@pytest.mark.parametrize("name", ["tiny", "fek_tiny"])
def test_command_line_generates_from_a_checkpoint_folder(name, tmp_path, capsys):
    cfg, w = _checkpoint(tmp_path, name)
    G.main(["--model", str(tmp_path), "--dtype", "float32", "--prompt-tokens", "5,9,2", "--max-new-tokens", "6"])
    line = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert line["model"] == cfg["architecture"] and len(line["tokens"]) == 6
    logits = O.forward(cfg, w, [5, 9, 2] + line["tokens"][:-1])
    for i, t in enumerate(line["tokens"]):
        assert float(logits[2 + i].max() - logits[2 + i][t]) < 1e-3 * float(logits[2 + i].std())


@pytest.mark.parametrize("name", ["odd", "fek_odd"])
def test_trace_runner(name, tmp_path):
    cfg, w = _checkpoint(tmp_path, name)
    a, b = cases.tokens(cfg, 30), cases.tokens(cfg, 9, seed=2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:25], "want": [0, 24]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[25:29], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[29:], "want": [0]}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": b, "want": [8, 3]}], "end": ["y"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", "float32",
                        "--out", str(tmp_path), "--max-tokens", "40"], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    read = lambda n: torch.from_numpy(np.fromfile(tmp_path / f"{n}.f32", "<f4").reshape(-1, cfg["vocab"]))
    wa, wb = O.forward(cfg, w, a), O.forward(cfg, w, b)
    _close(read(0), wa[[0, 24]], torch.float32)
    assert not (tmp_path / "1.f32").exists()
    _close(read(2), wa[[29]], torch.float32)
    _close(read(3), wb[[8, 3]], torch.float32)
