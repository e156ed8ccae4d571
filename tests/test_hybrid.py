"""Hybrid decoder without a GPU: configuration, registry, sequence state, rotary frequencies, the library's symbols, and
properties of the oracle itself."""
import json
import math
import os
import re

import pytest
import torch

from decdec_amd import _lib, registry
from decdec_amd.cache import GroupedCache, JoinedState, KVCache, LatentCache, RecurrentState, SequenceState
from decdec_amd.generate import Session
from decdec_amd.hybrid import HybridConfig, HybridDecoder, PreNormDecoder
from decdec_amd.mixers import LinearRecurrence, Workspace
from decdec_amd.model import ModelArgs, Transformer, rope_frequencies, rope_tables
from oracle import hybrid_oracle as O
import hybrid_cases as cases

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_every_tensor_of_a_configuration_is_expected_by_name_and_shape(name):
    cfg = cases.CONFIGS[name]()
    model = registry.model_class(cfg).from_config(cfg, torch.float32, device="cpu")
    for i, layer in model.weights.items():
        layer.fit({n[len(f"l{i}."):]: s for n, s in cases.shapes(cfg).items() if n.startswith(f"l{i}.")})
    assert {n: tuple(s) for n, s in model.weight_shapes().items()} == cases.shapes(cfg)


@pytest.mark.parametrize("make,gone", [(cases.config_odd, "l2.norm1"), (cases.config_fek_odd, "l0.norm1.alpha"), (cases.config_fek_odd, "l0.mix.a1")])
def test_checkpoint_folder_round_trip(make, gone, tmp_path):
    from safetensors.torch import save_file
    cfg = make()
    w = cases.weights(cfg)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    assert registry.is_checkpoint(str(tmp_path)) and registry.read_config(str(tmp_path)) == cfg
    del w[gone]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(KeyError, match=gone):
        registry.load_model(str(tmp_path), torch.float32, device="cpu")
    with pytest.raises(KeyError, match="Unknown architecture"):
        registry.model_class({"architecture": "no-such-design"})


def test_configuration_errors_are_named():
    cfg = cases.config_odd()
    cfg["layers"][0]["type"] = "no-such-mixer"
    with pytest.raises(ValueError, match="unknown mixer"):
        HybridConfig.from_dict(cfg)
    cfg = cases.config_odd()
    cfg["layers"][0]["weights_of"] = 5
    with pytest.raises(ValueError, match="refers back to itself"):
        HybridConfig.from_dict(cfg).source(0)
    with pytest.raises(ValueError, match="float32 or bfloat16"):
        HybridDecoder.from_config(cases.config_tiny(), torch.float16, device="cpu")
    cfg = cases.config_tiny()
    cfg["layers"][0]["mixer"]["decay"] = [0.5, 0.5]
    with pytest.raises(ValueError, match="decays for 1 heads"):
        HybridDecoder.from_config(cfg, torch.float32, device="cpu")
    cfg = cases.config_fek_odd()
    cfg["layers"][1]["mixer"]["left"]["kv_heads"] = 4
    with pytest.raises(ValueError, match="do not divide"):
        PreNormDecoder.from_config(cfg, torch.float32, device="cpu")


def test_a_recurrence_has_one_kind_of_decay():
    ws = Workspace("cpu")
    for bad in (dict(), dict(decay=[0.5, 0.5], conv=4), dict(channel=True), dict(channel=True, conv=4, tau=2.0), dict(conv=4, low_rank_gate=True)):
        with pytest.raises(ValueError):
            LinearRecurrence(2, 8, 8, ws, **bad)


def test_layers_that_share_weights_keep_states_of_their_own():
    cfg = HybridConfig.from_dict(cases.config_odd())
    assert [cfg.source(i) for i in range(cfg.n_layer)] == [0, 1, 2, 0, 1, 0, 2]


def test_sequence_state_counts_and_restores():
    rec = RecurrentState(2, 4, 3, "cpu", taps=2, channels=5, dtype=torch.float32)
    lat = LatentCache(70, 6, 2, torch.float32, "cpu")
    assert lat.rows.shape == (128, 8)
    grp = GroupedCache(70, 2, 6, 5, torch.float32, "cpu")
    assert grp.keys.shape == (2, 128, 6) and grp.values.shape == (10, 128)
    st = SequenceState([JoinedState([grp, rec]), lat, KVCache(1, 8, 1, 4, torch.float32, "cpu")], max_tokens=10)
    st.advance(0, 4)
    with pytest.raises(ValueError, match="start at position 3"):
        st.advance(3, 1)
    with pytest.raises(ValueError, match="do not fit"):
        st.advance(4, 7)
    saved = st.snapshot()
    assert len(saved) == 2
    rec.state += 1; rec.ring += 2
    st.restore(saved)
    assert float(rec.state.abs().sum() + rec.ring.abs().sum()) == 0
    st.release()
    st.advance(0, 10)


def test_session_feeds_portions_to_the_plain_decoder():
    """The same session drives the models that were there before."""
    torch.manual_seed(0)
    m = Transformer(torch.float32, ModelArgs.from_name("tiny-llama-test"), linear_class=torch.nn.Linear,
                    linear_kwargs={"dtype": torch.float32, "device": "cpu"}, device="cpu")
    toks = torch.randint(0, m.config.vocab_size, (21,))
    s = Session(m, 40)
    whole = s.feed(toks, range(21))
    s.close()
    s = Session(m, 40, portion=4)
    parts, at = [], 0
    for n in (1, 9, 2, 9):
        parts.append(s.feed(toks[at:at + n], range(n)))
        at += n
    assert torch.allclose(torch.cat(parts), whole, atol=1e-5)
    assert s.feed(toks[:2]).shape == (0, m.config.vocab_size) and s.length == 23
    with pytest.raises(ValueError, match="wanted places"):
        s.feed(toks[:2], [2])
    with pytest.raises(ValueError, match="do not fit"):
        s.feed(torch.zeros(30))


@pytest.mark.parametrize("dims,base,scaling", [(8, 1000.0, None), (10, 500.0, cases.YARN), (64, 1e4, dict(factor=4.0, original=512, fast=32.0, slow=1.0)),
                                               (32, 1e6, dict(factor=1.0, original=128, fast=8.0, slow=8.0)),
                                               (16, 50.0, dict(factor=16.0, original=8, fast=4.0, slow=0.1))])
def test_rotary_frequencies_and_pair_tables(dims, base, scaling):
    want, mag = O.rotary_frequencies(dims, base, scaling)
    got, m = rope_frequencies(dims, base, scaling)
    assert m == pytest.approx(mag) and got.tolist() == pytest.approx(want)
    cos, sin = rope_tables(dims + 6, 50, base, layout="pairs", dims=dims, scaling=scaling)
    assert cos.shape == (50, dims // 2 + 3) and torch.all(cos[:, dims // 2:] == 1) and torch.all(sin[:, dims // 2:] == 0)
    i, p = dims // 2 - 1, 37
    assert float(cos[p, i]) == pytest.approx(math.cos(p * want[i]) * mag, abs=1e-6)
    assert float(sin[p, 0]) == pytest.approx(math.sin(p * want[0]) * mag, abs=1e-6)


def test_mixers_library_exports_what_the_header_declares():
    text = open(os.path.join(ROOT, "include", "decdec_mixers.h")).read()
    names = set(re.findall(r"\b(decdec_mix\w+)\s*\(", re.sub(r"/\*.*?\*/", "", text, flags=re.S)))
    lib = _lib.load_mixers()
    assert names == set(_lib.MIXERS_SIGNATURES) | set(_lib.MIXERS_OTHER)
    assert all(hasattr(lib, n) for n in names)
    # the ctypes mirrors list the fields of the C structs in order
    for cls, tag in ((_lib.Recurrence, "decdec_recurrence"), (_lib.Latent, "decdec_latent"), (_lib.Grouped, "decdec_grouped"),
                     (_lib.TanhNorm, "decdec_tanh_norm")):
        body = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
        body = body[:body.index("} " + tag + ";")]
        body = body[body.rindex("typedef struct {") + len("typedef struct {"):]
        fields = [re.sub(r".*[\s*]", "", f.strip()) for decl in body.split(";") for f in decl.split(",") if f.strip()]
        assert fields == [f[0] for f in cls._fields_]


def test_arguments_are_checked_before_any_launch():
    lib = _lib.load_mixers()
    err = lambda: lib.decdec_mixers_last_error().decode()
    assert lib.decdec_mix_gemv(None, None, None, None, 0, 0, 1.0, 0, 8, 8, None) != 0 and "null pointer" in err()
    assert lib.decdec_mix_gemv(8, 8, 8, None, 0, 0, 1.0, 1, 8, 8, None) != 0 and "fp32 or bf16" in err()
    r = _lib.Recurrence(proj=16, state=16, pos=16, heads=3, kv_heads=2, dim=8, vdim=8, ld=1000)
    assert lib.decdec_mix_recurrence_step(r, 16, None, None, 0.0, 0, 0, None) != 0 and "multiple of kv_heads" in err()
    r = _lib.Recurrence(proj=16, state=16, pos=16, heads=2, kv_heads=2, dim=300, vdim=8, ld=1000)
    assert lib.decdec_mix_recurrence_step(r, 16, None, None, 0.0, 0, 0, None) != 0 and "dim must be" in err()
    p = _lib.Latent(proj=16, norm=16, cache=16, pos=16, cos_table=16, sin_table=16, heads=2, dim=8, rot=4, vdim=8, rank=8, max_seq=64,
                    off_q=0, off_c=24, ld=36)
    assert lib.decdec_mix_latent_attention(p, 16, 16, 16, 64, 16, 0, 60, 5, None) != 0 and "do not fit a cache" in err()
    assert lib.decdec_mix_latent_attention(p, 16, 16, 16, 63, 16, 0, 10, 5, None) != 0 and "multiple of 64" in err()


def test_oracle_is_causal_and_a_missing_mechanism_shows():
    cfg = cases.config_tiny()
    w, toks = cases.weights(cfg, 3), cases.tokens(cfg, 20)
    full = O.forward(cfg, w, toks)
    assert torch.allclose(O.forward(cfg, w, toks[:13]), full[:13])
    for change in ("l2.mix.sink", "l1.mix.A_log", "l0.rg1.b", "l0.mlp.act", "l1.mix.dt_bias", "l2.mix.dkv.norm"):
        other = dict(w)
        other[change] = w[change] + 1.0
        assert not torch.allclose(O.forward(cfg, other, toks), full, atol=1e-3), change


def test_fekulix_oracle_is_causal_and_every_tensor_shows():
    cfg = cases.config_fek_odd()
    w, toks = cases.weights(cfg, 3), cases.tokens(cfg, 20)
    full = O.forward(cfg, w, toks)
    assert torch.allclose(O.forward(cfg, w, toks[:13]), full[:13])
    for change in w:
        other = {**w, change: w[change] * 1.3 + 0.2}
        assert not torch.allclose(O.forward(cfg, other, toks), full, atol=1e-3), change


def test_fekulix_oracle_tells_mistakes_apart(monkeypatch):
    """Mistakes planted in the oracle move the logits by far more than the tolerance of the GPU tests."""
    cfg = cases.config_fek_odd()
    w, toks = cases.weights(cfg, 3), cases.tokens(cfg, 40)
    full = O.forward(cfg, w, toks)
    attention, rotate, O_sum = O.sink_attention, O.rotate, O.channel_decayed_sum

    def half_layout(x, positions, rot):
        n = rot["dims"]
        order = torch.arange(n).view(2, n // 2).T.reshape(-1)
        y = x.clone()
        y[..., order] = rotate(x[..., :n][..., order], positions, rot)
        return y

    def late_decay(q, k, v, g, beta):                      # the decay after the write
        T, H, D = q.shape
        S, out = torch.zeros(H, D, v.shape[-1], dtype=q.dtype), []
        for t in range(T):
            u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
            S = S + k[t][:, :, None] * u[:, None, :]
            out.append((S * q[t][:, :, None]).sum(1))
            S = g[t][:, :, None] * S
        return torch.stack(out), S
    mistakes = {"no sink": ("sink_attention", lambda q, k, v, s, sink=0.0: attention(q, k, v, s, -math.inf)),
                "other key heads": ("sink_attention", lambda q, k, v, s, sink=0.0: attention(q, k.flip(0), v.flip(0), s, sink)),
                "half layout": ("rotate", half_layout),
                "decay after the write": ("channel_delta_rule", late_decay),
                "decay left out": ("channel_decayed_sum", lambda q, k, v, g: O_sum(q, k, v, torch.ones_like(g)))}
    for what, (name, f) in mistakes.items():
        with monkeypatch.context() as p:
            p.setattr(O, name, f)
            wrong = O.forward(cfg, w, toks)
        assert float((wrong - full).std() / full.std()) > 0.05, what
