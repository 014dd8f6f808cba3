"""The hybrid decoder's host side (no GPU): configuration, checkpoint loading, page and slot management, sampling,
command lines, the C ABI's argument checks, and the plain restatement against itself."""
import json
import os
import re
import subprocess
import sys

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

from khaosz_amd import AutoRegressiveLM, Engine, LMConfig, _abi, load_model, model_names
from khaosz_amd.cache import FreeList, SequenceCache
from khaosz_amd.hybrid import HybridConfig, HybridLM
from khaosz_amd.mixers import rotary_pairs
from khaosz_amd.sampling import Sampler
from oracle import hybrid as plain

import hybrid_cases as hc

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def test_seq_library_exports_every_declared_symbol():
    header = open(os.path.join(ROOT, "include", "astrai_seq.h")).read()
    declared = set(re.findall(r"\b(aqs_[a-z0-9_]+)\s*\(", header))
    assert declared == set(_abi.SEQ_SYMBOLS), declared ^ set(_abi.SEQ_SYMBOLS)
    lib = _abi.load_seq()
    for name in declared:
        assert hasattr(lib, name), name


def test_seq_arguments_are_checked_before_any_launch():
    lib, P = _abi.load_seq(), 1 << 20
    add = lambda dtype, K, top=0, post=None: lib.aqs_add_rmsnorm(P, None, 8, dtype, None, None, top, post, 1.0, P, 1.0, 1e-6, P, 1, K, None)
    assert add(1, 0) == -2 and add(7, 8) == -3
    assert add(1, 8, top=2) == -1 and add(1, 8, post=P) == -1                                                # routed rows missing; nothing to norm
    assert lib.aqs_gemv_ok(1, 1, 64, 20) == 0 and lib.aqs_gemv_ok(1, 9, 64, 64) == 0 and lib.aqs_gemv_ok(1, 8, 64, 64) == 1
    def gemv(i, o, x=P, xf=None, yf=None, post=None, x_out=None, gain=None, w=P, routers=0, res=None, ldo=64):
        return lib.aqs_gemv(i, o, 1, x, 64, xf, yf, post, x_out, gain, 0.0, 1e-6, 1, w, None, 1.0, 0.0, routers, res, P, ldo, None, 1, 64, 64, None)
    assert gemv(0, 0, w=P + 2) == -4
    assert gemv(2, 3, xf=P, gain=P, res=P) == -2                                                             # pair not served
    assert gemv(3, 0, xf=P, gain=P) == -1                                                                    # no branch output
    assert gemv(3, 0, xf=P, yf=P, post=P, x_out=P, gain=P) == -2                                             # the old stream is still read
    assert gemv(0, 0, routers=8) == -2 and gemv(3, 4, xf=P, yf=P, post=P, x_out=2 * P, gain=P, res=P) == -2  # routers only with kind 4
    assert lib.aqs_delta_scan(P, P, P, P, P, P, P, P, P, 1, 4, 3, 2, 8, 8, None) == -2                       # heads over kv heads
    assert lib.aqs_delta_scan(P, P, P, P, P, P, P, P, P, 1, 4, 2, 2, 257, 8, None) == -6
    assert lib.aqs_ssd_scan(P, P, 2, 1, P, P, P, None, P, P, P, P, 0, 4, 2, 2, 8, 8, None) == 0              # nothing to do
    assert lib.aqs_ssd_scan(P, P, 0, 1, None, None, None, P, P, P, P, P, 0, 4, 2, 2, 8, 8, None) == 0        # constant decays need no steps
    assert lib.aqs_ssd_scan(P, P, 0, 1, None, None, None, None, P, P, P, P, 1, 4, 2, 2, 8, 8, None) == -2
    assert lib.aqs_attn_window_ok(1, 24, 40, 64) == 1 and lib.aqs_attn_window_ok(0, 24, 40, 64) == 0
    assert lib.aqs_attn_window_ok(1, 20, 40, 64) == 0 and lib.aqs_attn_window_ok(1, 24, 40, 16) == 0
    for window in (1, 2, 63, 64, 65, 127, 128, 129, 300):
        most = max(p // 64 - max(0, p - window + 1) // 64 + 1 for p in range(2000))
        assert lib.aqs_attn_decode_slices(window, 1 << 20) == most, window


def test_registry_knows_both_models_and_refuses_others(tmp_path):
    assert {"Rudilix", "autoregressive_lm"} <= set(model_names())
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "NoSuchModel"}))
    with pytest.raises(ValueError, match="NoSuchModel"):
        load_model(str(tmp_path), device="cpu")


@pytest.mark.parametrize("case", list(hc.CASES))
def test_checkpoint_round_trip(case, tmp_path):
    cfg, _ = hc.CASES[case]
    w = hc.weights(case)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({n: t.bfloat16().contiguous() for n, t in w.items()}, str(tmp_path / "model.safetensors"))
    m = load_model(str(tmp_path), torch.float32, "cpu")
    got = m.tensors()
    assert set(got) == set(w)
    for n in w:
        assert torch.equal(got[n].float(), w[n]), n
    # the parts of a fused matrix are not overlapping views
    total = sum(t.numel() for t in got.values())
    assert total <= sum(p.numel() for p in m.parameters())
    del w["head"]
    save_file({n: t.contiguous() for n, t in w.items()}, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="head"):
        load_model(str(tmp_path), torch.float32, "cpu")


def test_configuration_is_checked():
    cfg, shapes = hc.config([hc.layer("mamba2", hc.mamba())])
    with pytest.raises(ValueError, match="mixer"):
        HybridConfig.from_dict({**cfg, "layers": [{**cfg["layers"][0], "type": "other"}]})
    with pytest.raises(ValueError, match="feed-forward"):
        HybridConfig.from_dict({**cfg, "layers": [{**cfg["layers"][0], "mlp": {"kind": "other", "ff": 8, "limit": 1.0}}]})
    with pytest.raises(ValueError):
        HybridLM(HybridConfig.from_dict(hc.config([hc.layer("mamba2", hc.mamba(5, 2))])[0]), device="cpu")
    with pytest.raises(ValueError, match="rank"):
        HybridLM(HybridConfig.from_dict(hc.config([hc.layer("channel_delta", hc.delta())])[0]), device="cpu")


def test_loaded_autoregressive_model(tmp_path):
    cfg = LMConfig(vocab_size=31, dim=32, n_layers=2, n_heads=4, n_kv_heads=2, dim_ffn=48, max_len=64)
    m = AutoRegressiveLM(cfg)
    (tmp_path / "config.json").write_text(json.dumps({"model_type": "autoregressive_lm", **cfg.__dict__, "unread": 1}))
    save_file({n: t.detach().clone() for n, t in m.tensors().items()}, str(tmp_path / "model.safetensors"))
    got = load_model(str(tmp_path), torch.float32, "cpu")
    ids = torch.arange(7).unsqueeze(0)
    with torch.inference_mode():
        assert torch.equal(m(ids)["logits"], got(ids)["logits"])


class _Stub:
    window = 10

    def __init__(self):
        self.asked = None

    def new_sequence_state(self, *a):
        self.asked = a
        return None


def test_pages_and_slots_are_taken_and_given_back():
    stub = _Stub()
    c = SequenceCache(stub, 32, 2, page=4)
    assert stub.asked == (2, 9, 4, 32)
    a, b = c.open(), c.open()
    with pytest.raises(RuntimeError, match="slot"):
        c.open()
    c.reserve([a], 5)
    c.commit([a], 5)
    assert len(c.pages) == 7 and (c.table[a][:2] >= 0).all() and (c.table[a][2:] < 0).all()
    c.reserve([b], 8)
    c.commit([b], 8)
    assert len(set(c.table[a][:2]) | set(c.table[b][:2])) == 4
    # window 10, page 4: after 13 tokens the next one (position 13) sees 4 .. 13, so page 0 is free again
    c.reserve([a], 8)
    c.commit([a], 8)
    assert c.table[a][0] == -1 and c.table[a][1] >= 0
    words = np.zeros(c.words(2, 3), np.int64)
    c.pack([b, a], [[1, 2, 3], [4, 5, 6]], words)
    ids, batch = c.unpack(torch.from_numpy(words), 2, 3)
    assert ids.tolist() == [[1, 2, 3], [4, 5, 6]] and batch.pos.tolist() == [8, 13] and batch.slots.tolist() == [b, a]
    assert batch.table.tolist() == [c.table[b].tolist(), c.table[a].tolist()]
    c.close(a)
    c.close(b)
    assert len(c.pages) == 9 and len(c.slots) == 2 and (c.table < 0).all()
    h = c.open()
    with pytest.raises(ValueError, match="does not fit"):
        c.reserve([h], 33)


def test_free_list_refuses_a_second_return():
    f = FreeList(2, "page")
    i = f.take()
    f.give(i)
    with pytest.raises(ValueError):
        f.give(i)


def test_rotary_pairs():
    t = rotary_pairs(6, 50, 300.0).double().numpy()
    for p in (0, 1, 49):
        for i in range(3):
            a = p * 300.0 ** (-2 * i / 6)
            assert abs(t[p, i, 0] - np.cos(a)) < 1e-7 and abs(t[p, i, 1] - np.sin(a)) < 1e-7
    assert rotary_pairs(0, 5, 10.0).shape == (5, 0, 2)


def test_sampler():
    z = torch.tensor([[0.0, 3.0, 1.0, 2.9], [5.0, 0.0, 0.0, 0.0]])
    assert Sampler()(z).tolist() == [1, 0]
    assert Sampler(1.0, top_k=1, seed=0)(z).tolist() == [1, 0]
    assert Sampler(1.0, top_p=1e-6, seed=0)(z).tolist() == [1, 0]
    s = Sampler(1.0, top_k=2, seed=3)
    draws = torch.stack([s(z) for _ in range(200)])
    assert set(draws[:, 0].tolist()) == {1, 3}
    one, two = Sampler(0.8, seed=5), Sampler(0.8, seed=5)
    assert [one(z).tolist() for _ in range(5)] == [two(z).tolist() for _ in range(5)]
    with pytest.raises(ValueError):
        Sampler(top_p=0.0)


def test_engine_generates_with_the_autoregressive_model_on_the_cpu():
    """Scheduling over the paged cache: prompts of unequal length, fewer places than prompts, a stop token."""
    torch.manual_seed(3)
    m = AutoRegressiveLM(LMConfig(vocab_size=41, dim=32, n_layers=2, n_heads=4, n_kv_heads=2, dim_ffn=48, max_len=64)).eval()
    prompts = [[1, 2, 3], [7], [9, 8, 7, 6, 5, 4, 3], [1, 2, 4]]

    def alone(p, n):
        ids, out = list(p), []
        for _ in range(n):
            with torch.inference_mode():
                out.append(int(m(torch.tensor([ids]))["logits"][0, -1].argmax()))
            ids.append(out[-1])
        return out
    want = [alone(p, 6) for p in prompts]
    e = Engine(m, 40, 2, page=4)
    assert e.generate(prompts, 6) == want
    assert len(e.cache.slots) == 2 and (e.cache.table < 0).all()
    stop = want[0][2]
    cut = [w[:w.index(stop) + 1] if stop in w else w for w in want]
    assert e.generate(prompts, 6, stop=[stop]) == cut
    with pytest.raises(ValueError, match="fit"):
        e.generate([[1] * 40], 6)
    with pytest.raises(ValueError, match="vocabulary"):
        e.step([e.open()], [[41]])


@pytest.mark.parametrize("tool", ["trace_run", "generate"])
def test_command_lines_explain_themselves(tool):
    r = subprocess.run([os.path.join(ROOT, "bin", tool), "--help"], capture_output=True, text=True, timeout=60)
    assert r.returncode == 0 and "--model" in r.stdout
    assert os.access(os.path.join(ROOT, "bin", tool), os.X_OK) and sys.version_info >= (3, 8)


@pytest.mark.parametrize("case", list(hc.CASES))
def test_plain_restatement_carries_its_state(case):
    """The oracle fed whole, in portions and token by token."""
    cfg, _ = hc.CASES[case]
    w = {n: t.numpy() for n, t in hc.weights(case).items()}
    ids = hc.prompt(case, 23)
    whole = plain.Sequence(cfg, w).run(ids)
    for cuts in ([5, 7, 9, 2], [1] * 23):
        s, at, out = plain.Sequence(cfg, w), 0, []
        for n in cuts:
            out.append(s.run(ids[at:at + n]))
            at += n
        assert np.allclose(np.concatenate(out), whole, rtol=1e-9, atol=1e-9)
    assert whole.std() > 0.1
