"""The Lomozen design's host side (no GPU): configuration, checkpoint loading, rotary tables, page need, argument checks of
its kernels, and the plain restatement against itself."""
import json
import math

import numpy as np
import pytest
import torch
from safetensors.torch import save_file

from khaosz_amd import _abi, load_model, model_names
from khaosz_amd.cache import SequenceCache
from khaosz_amd.hybrid import HybridConfig, HybridLM
from khaosz_amd.mixers import rotary_pairs
from khaosz_amd.seq_ops import Batch, LatentSpec, latent_rows
from oracle import lomozen as plain

import lomozen_cases as lc


def test_registered_beside_the_other_designs():
    assert {"Lomozen", "Rudilix", "autoregressive_lm"} <= set(model_names())


@pytest.mark.parametrize("case", list(lc.CASES))
def test_checkpoint_round_trip(case, tmp_path):
    cfg, w = lc.CASES[case], lc.weights(case)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({n: t.bfloat16().contiguous() for n, t in w.items()}, str(tmp_path / "model.safetensors"))
    m = load_model(str(tmp_path), torch.float32, "cpu")
    got = m.tensors()
    assert set(got) == set(w)
    for n in w:
        assert torch.equal(got[n].float(), w[n]), n
    assert sum(t.numel() for t in got.values()) <= sum(p.numel() for p in m.parameters())  # parts of a matrix do not overlap
    missing = "l0.mix.o"
    del w[missing]
    save_file({n: t.contiguous() for n, t in w.items()}, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match=missing):
        load_model(str(tmp_path), torch.float32, "cpu")


def test_names_of_a_layer():
    names = set(lc.weights("mixed"))
    for n in ("l0.mix.q", "l0.mix.k", "l0.mix.v", "l0.mix.g", "l0.mix.norm", "l1.mix.dq", "l1.mix.dq.norm", "l1.mix.uq", "l1.mix.dkv", "l1.mix.dkv.norm",
              "l1.mix.uk", "l1.mix.uv", "l1.mix.g", "l1.mix.o", "l1.mlp.e5.down", "l1.mlp.router", "l1.mlp.shared.gate", "l2.norm1b", "l2.norm2b"):
        assert n in names, n
    assert not any(n.startswith("l3.mlp") or n in ("l3.norm2", "l3.norm2b") for n in names)


def test_configuration_is_checked():
    cfg = lc.CASES["mixed"]
    with pytest.raises(ValueError, match="mixer"):
        HybridConfig.from_dict({**cfg, "layers": [{**cfg["layers"][0], "type": "mamba2"}]})  # another design's
    with pytest.raises(ValueError, match="feed-forward"):
        HybridConfig.from_dict({**cfg, "layers": [{**cfg["layers"][0], "mlp": {"kind": "dense", "ff": 8, "limit": 1.0}}]})
    with pytest.raises(ValueError, match="design"):
        HybridConfig.from_dict({**cfg, "architecture": "other"})
    build = lambda l: HybridLM(HybridConfig.from_dict(lc.config([l])), device="cpu")
    with pytest.raises(ValueError, match="decay"):
        build(lc.layer(lc.lightning(2, 8, 8, [0.5])))
    with pytest.raises(ValueError, match="decay"):
        build(lc.layer(lc.lightning(1, 8, 8, [1.5])))
    with pytest.raises(ValueError, match="experts"):
        build(lc.layer(lc.lightning(), lc.moe(3, 4)))
    with pytest.raises(ValueError, match="rotated"):
        build(lc.layer(lc.latent(dims=7)))


def test_windows_of_the_layers_decide_what_the_cache_keeps():
    build = lambda *ls: HybridLM(HybridConfig.from_dict(lc.config(list(ls))), device="cpu")
    assert build(lc.layer(lc.latent(window=9)), lc.layer(lc.lightning()), lc.layer(lc.latent(window=33))).window == 33
    m = build(lc.layer(lc.lightning()))
    assert m.window == 1
    m = build(lc.layer(lc.latent(window=65, kv_rank=48, rot_dim=8)))
    c = SequenceCache(m, 640, 1)
    assert tuple(c.state[0][0]["kv"].k.shape) == (10, 64, 1, 56) and c.state[0][0]["kv"].v.numel() == 0
    h = c.open()
    for _ in range(600):
        c.reserve([h], 1)
        c.commit([h], 1)
        first = max(0, c.length(h) - 64) // 64  # the next token sees itself and the 64 before it
        assert (c.table[h][first:(c.length(h) - 1) // 64 + 1] >= 0).all() and (c.table[h][:first] < 0).all()


@pytest.mark.parametrize("scaling", [None, {"factor": 4.0, "original": 64, "fast": 6.0, "slow": 1.5}, {"factor": 1.0, "original": 32, "fast": 4.0, "slow": 1.0},
                                     {"factor": 16.0, "original": 4096, "fast": 32.0, "slow": 1.0}, {"factor": 2.0, "original": 8, "fast": 64.0, "slow": 40.0}])
@pytest.mark.parametrize("dims,base", [(8, 500.0), (2, 90.0), (64, 1e4), (16, 5e5)])
def test_rotary_tables(dims, base, scaling):
    t = rotary_pairs(dims, 3000, base, scaling).double().numpy()
    freq, grow = plain.yarn(dims, base, scaling)
    for p in (0, 1, 77, 2999):
        for i in range(dims // 2):
            assert abs(t[p, i, 0] - grow * math.cos(p * freq[i])) < 3e-7 and abs(t[p, i, 1] - grow * math.sin(p * freq[i])) < 3e-7
    if scaling and scaling["factor"] > 1:
        assert grow > 1


def test_rotation_in_halves():
    x = np.arange(1.0, 8.0)
    y = plain.rotate_half(x, 3, 4, 10.0)
    assert (y[4:] == x[4:]).all()
    for i in range(2):
        a = 3 * 10.0 ** (-2 * i / 4)
        assert np.allclose([y[i], y[i + 2]], [x[i] * math.cos(a) - x[i + 2] * math.sin(a), x[i + 2] * math.cos(a) + x[i] * math.sin(a)])


def test_rows_laid_out_for_a_portion():
    for window in (1, 2, 63, 64, 65, 130):
        s = LatentSpec(1, 8, 8, 8, 8, 8, 8, window, 1.0, 1e-5)
        for S in (1, 2, 64, 100):
            most = 0
            for p in range(400):
                b = Batch(None, None, None, 1, S, (p,))
                base, rows = max(p - window + 1, 0) // 64 * 64, latent_rows(s, b, 10 ** 6)
                assert rows % 64 == 0 and base + rows > p + S - 1 >= base + rows - 64
                most = max(most, rows)
            unknown = Batch(None, None, None, 1, S)
            assert latent_rows(s, unknown, 10 ** 6) >= most and latent_rows(s, unknown, 64) == 64
        lib = _abi.load_seq()
        n = max(p // 64 - max(0, p - window + 1) // 64 + 1 for p in range(2000))
        assert lib.aqs_latent_decode_slices(window, 1 << 20) == n
    assert lib.aqs_latent_decode_slices(1 << 20, 1 << 20) <= 64


def test_arguments_are_checked_before_any_launch():
    lib, P = _abi.load_seq(), 1 << 20
    prep = lambda ld=64, rd=8, rows=64, packed=P: lib.aqs_latent_prep(P, ld, 0, 24, 1, P, P, 1e-5, P, 64, P, P, 1, 64, 1, 9, P, P, packed, rows, 1, 4, 24, 32, 8, rd, None)
    assert prep(ld=40) == -2 and prep(rd=7) == -2 and prep(rd=16) == -2 and prep(rows=0) == -2
    assert lib.aqs_latent_rotate(None, 1, P, 64, P, 1, 4, 2, 8, 8, 8, None) == -1
    win = lambda rows, ld_gate: lib.aqs_latent_window(P, P, 96, P, 40, 32, 1, 1.0, 9, P, ld_gate, P, rows, P, 48, 1, 4, 2, 24, 8, 24, 0, None)
    assert win(60, 48) == -2 and win(64, 40) == -2
    assert lib.aqs_latent_decode_ok(1, 24, 8, 48, 40, 64) == 1 and lib.aqs_latent_decode_ok(9, 24, 8, 48, 40, 64) == 0
    assert lib.aqs_latent_decode_ok(1, 20, 8, 48, 40, 64) == 0 and lib.aqs_latent_decode_ok(1, 24, 8, 48, 40, 16) == 0
    assert lib.aqs_moe_route(P, 8, 1, P, P, P, 4, 8, 4, 5, None) == -2 and lib.aqs_moe_route(P, 8, 1, P, P, P, 4, 8, 513, 1, None) == -6
    assert lib.aqs_moe_sort(P, 8, 4, 64, P, P, P, 3, None) == -2
    assert lib.aqs_moe_product(1, P, 8, 1, P, P, 5, 64, P, None, 8, 1, P, 16, 8, None) == -1  # no scores
    assert lib.aqs_moe_product(0, P, 12, 1, P, P, 5, 128, P, None, 8, 1, P, 16, 12, None) == -4
    assert lib.aqs_moe_step_ok(8, 64, 8, 8, 4, 4) == 1 and lib.aqs_moe_step_ok(9, 64, 8, 8, 4, 4) == 0 and lib.aqs_moe_step_ok(1, 64, 12, 8, 4, 4) == 0
    assert lib.aqs_moe_tile(1, 10, 4, 64, 64) != 64 and lib.aqs_moe_tile(0, 10, 4, 64, 64) == 64 and lib.aqs_moe_tile(1, 10, 4, 64, 12) == 64


@pytest.mark.parametrize("case", list(lc.CASES))
def test_plain_restatement_carries_its_state(case):
    """The oracle fed whole, in portions and token by token."""
    cfg = lc.CASES[case]
    w = {n: t.numpy() for n, t in lc.weights(case).items()}
    ids = lc.prompt(case, 23)
    whole = plain.Sequence(cfg, w).run(ids)
    for cuts in ([5, 7, 9, 2], [1] * 23):
        s, at, out = plain.Sequence(cfg, w), 0, []
        for n in cuts:
            out.append(s.run(ids[at:at + n]))
            at += n
        assert np.allclose(np.concatenate(out), whole, rtol=1e-9, atol=1e-9)
    assert whole.std() > 0.1


def test_choice_of_experts():
    best, s = plain.choose(np.array([0.5, 2.0, -1.0, 1.0]), 2)
    assert best == [1, 3] and np.allclose(s, 1 / (1 + np.exp([-2.0, -1.0])))
