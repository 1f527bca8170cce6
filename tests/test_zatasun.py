"""Zatasun on the CPU: the oracle's equations, configuration, checkpoint
names, state specifications and registry."""
import json
import math

import pytest
import torch

import zatasun_oracle as oracle
import zatasun_util as util
import lfmq
from lfmq.bench.compare import SIZES, layer_params
from lfmq.cli import MODEL_PRESETS
from lfmq.models.registry import ARCHS, read_plain_config, spec_of
from lfmq.models.seqcache import SequenceCache
from lfmq.models.zatasun import ZatasunConfig, convert_state
from lfmq.ops.functional import rope_inv_freq

D = torch.float64


# ---- the oracle itself ------------------------------------------------------

def test_oracle_recurrence_matches_its_closed_form():
    g = torch.Generator().manual_seed(0)
    a = torch.rand(9, 3, generator=g, dtype=D)
    z = torch.randn(9, 3, generator=g, dtype=D)
    out, last = oracle.lru(a, z)
    for t in range(9):
        want = sum(z[s] * a[s + 1:t + 1].prod(0) for s in range(t + 1))
        assert torch.allclose(out[t], want, atol=1e-12)
    assert torch.equal(last, out[-1])
    again, _ = oracle.lru(a[4:], z[4:], out[3])
    assert torch.allclose(again, out[4:], atol=1e-12)


def test_oracle_convolution_is_causal_and_resumes():
    g = torch.Generator().manual_seed(1)
    x, w, b = (torch.randn(*s, generator=g, dtype=D)
               for s in ((8, 5), (5, 4), (5,)))
    full = oracle.causal_conv(x, w, b)
    want = torch.nn.functional.conv1d(
        torch.nn.functional.pad(x.t(), (3, 0))[None], w[:, None], b,
        groups=5)[0].t()
    assert torch.allclose(full, want, atol=1e-12)
    assert torch.allclose(oracle.causal_conv(x[5:], w, b, x[2:5]), full[5:])


def test_oracle_sink_is_in_the_denominator_only():
    v = torch.ones(2, 3, dtype=D)
    o = oracle.sink_attend(torch.zeros(2, dtype=D), v,
                           torch.tensor(0.0, dtype=D))
    assert torch.allclose(o, torch.full((3,), 2 / 3, dtype=D))


def test_oracle_gelu_and_weight_on_the_input():
    z = torch.linspace(-4, 4, 33, dtype=D)
    assert torch.allclose(oracle.gelu_tanh(z), torch.nn.functional.gelu(
        z, approximate="tanh"))
    g = torch.Generator().manual_seed(2)
    gate, up, down, h = (torch.randn(*s, generator=g, dtype=D)
                         for s in ((6, 4), (6, 4), (4, 6), (4,)))
    a = oracle.expert(0.3 * h, gate, up, down, 0.5)
    b = 0.3 * oracle.expert(h, gate, up, down, 0.5)
    assert float((a - b).abs().max()) > 0.05


# ---- rotation frequencies --------------------------------------------------------

@pytest.mark.parametrize("scaling", [
    None, util.SCALING, {"factor": 8.0, "low": 1.0, "high": 4.0,
                         "original": 900}])
def test_frequencies(scaling):
    got = rope_inv_freq(32, 5000.0, "cpu", scaling)
    want = torch.tensor(oracle.frequencies(32, 5000.0, scaling))
    assert torch.allclose(got, want.float(), rtol=1e-6)
    if scaling is not None:               # all three ranges are there
        plain = torch.tensor(oracle.frequencies(32, 5000.0))
        ratio = plain / want
        n = scaling["factor"]
        assert float(ratio.min()) == 1.0 and math.isclose(ratio.max(), n)
        assert bool(((ratio > 1.01) & (ratio < n - 0.01)).any())


# ---- configuration and registry ------------------------------------------------

def test_config_round_trip():
    for cfg in util.CONFIGS.values():
        c = ZatasunConfig.from_dict(cfg)
        assert c.n_layers == len(cfg["layers"])
        assert ZatasunConfig.from_dict(c.to_dict()) == c
        assert spec_of(c.to_dict()) is spec_of(cfg) is ARCHS["zatasun"]


def test_config_rejects_what_it_cannot_run():
    def bad(**kw):
        return util.config([{**util.layer(), **kw}])
    with pytest.raises(ValueError, match="unknown mixer"):
        ZatasunConfig.from_dict(bad(type="x"))
    with pytest.raises(ValueError, match="feed-forward"):
        ZatasunConfig.from_dict(bad(mlp={"kind": "sparse"}))
    with pytest.raises(ValueError, match="needs layers"):
        ZatasunConfig.from_dict(util.config([]))
    for wrong, msg in ((util.layer(rot=26), "rotate"),
                       (util.layer(heads=5, kv=2), "share"),
                       (util.layer(blocks=3), "blocks"),
                       (util.layer(mlp=util.moe(top=8)), "choose")):
        with pytest.raises(ValueError, match=msg):
            lfmq.build_model(util.config([wrong]))


def test_depth_override_and_presets():
    c = ZatasunConfig.from_dict(util.CONFIGS["mixed"])
    c.n_layers = 6
    assert c.layers[4] == c.layers[0] and c.layers[5] == c.layers[1]
    c.n_layers = 2
    assert len(c.layers) == 2
    assert MODEL_PRESETS["zatasun-8b"] == ("zatasun", "sized_8b")
    small = lfmq.build_model(SIZES["tiny-debug"]["zatasun"](2), seed=0)
    total, active = layer_params(small)
    idle = 6 * 3 * 256 * 128          # six of eight experts, one such layer
    assert total - active == idle


# ---- checkpoint --------------------------------------------------------------

def test_plain_checkpoint_loads(tmp_path):
    cfg = util.CONFIGS["mixed"]
    w = util.weights(cfg)
    path = util.write_checkpoint(tmp_path / "m", cfg, w)
    assert read_plain_config(path) == cfg
    for dt in (torch.bfloat16, torch.float32):
        m = lfmq.load(path, dtype=dt)
        mix = m.blocks[0].mixer
        assert mix.in_proj.weight.dtype == dt
        lr = mix.branches["right"]
        assert lr.gate_w.dtype == dt
        for p in (lr.lam, lr.conv_w, lr.gate_b, mix.branches["left"].sink,
                  m.norm.weight, m.embed_norm.weight):
            assert p.dtype == torch.float32
        assert torch.equal(lr.gate_w[:, 1], w["l0.mix.right.ri"].to(dt))
        n = w["l0.mix.left.q"].shape[0]
        k = w["l0.mix.left.k"]
        assert torch.equal(mix.in_proj.weight[n:n + len(k)], k.to(dt))
        assert torch.equal(mix.o_proj.weight[:, -64:],
                           w["l0.mix.right.o"].to(dt))
        e = m.blocks[1].mlp
        assert torch.equal(e.down[5], w["l1.mlp.e5.down"].to(dt))
        assert torch.equal(e.router[-1:], w["l1.mlp.shared.sg"].to(dt))
        assert m.blocks[2].mlp is None and m.blocks[3].mlp.shared is None
        assert not any(p.is_meta for p in m.parameters())


def test_checkpoint_names_are_checked(tmp_path):
    cfg = util.CONFIGS["mixed"]
    c = ZatasunConfig.from_dict(cfg)
    w = util.weights(cfg)
    with pytest.raises(KeyError, match="l1.mlp.e3.up"):
        convert_state(c, {k: v for k, v in w.items() if k != "l1.mlp.e3.up"})
    with pytest.raises(KeyError, match="unknown"):
        convert_state(c, {**w, "l2.norm2": w["l0.norm2"]})
    bad = {**w, "final.norm": w["final.norm"][:-1].contiguous()}
    with pytest.raises(ValueError, match="norm.weight"):
        lfmq.load(util.write_checkpoint(tmp_path / "b", cfg, bad))


def test_gpu_only_and_rtn_only():
    m = lfmq.build_model(util.CONFIGS["mixed"])
    with pytest.raises(RuntimeError, match="GPU"):
        m(torch.zeros(1, 3, dtype=torch.int64), m.make_cache(1, max_seq=8))
    with pytest.raises(NotImplementedError, match="rtn"):
        lfmq.quantize(m, lfmq.QuantConfig(scheme="gptq"))


def test_packed_checkpoint_takes_the_dtype_asked_for(tmp_path):
    """32-bit parameters stay 32-bit in a 16-bit model and all are in a
    32-bit one."""
    m = lfmq.build_model(util.CONFIGS["mixed"], seed=1)
    qc = lfmq.QuantConfig(scheme="rtn", bits=8, group_size=16)
    lfmq.save(m, str(tmp_path), qc)
    for dt in (torch.bfloat16, torch.float32):
        got = lfmq.load(str(tmp_path), dtype=dt)
        assert got.embed_tokens.weight.dtype == dt
        assert got.norm.weight.dtype == torch.float32
        assert torch.equal(got.embed_tokens.weight.bfloat16(),
                           m.embed_tokens.weight)


# ---- cache -------------------------------------------------------------------

def test_state_of_a_layer():
    m = lfmq.build_model(util.CONFIGS["mixed"])
    c = m.make_cache(3, max_seq=50)
    assert len(c.layers) == 4
    st = {k: tuple(t.shape) for k, t in c.layers[0].items()}
    assert st == {"left.k": (3, 50, 2, 24), "left.v": (3, 50, 2, 40),
                  "right.S": (3, 64), "right.conv": (3, 4, 64)}
    assert c.layers[0]["right.S"].dtype == torch.float32
    assert c.layers[0]["left.k"].dtype == torch.bfloat16


def test_snapshot_leaves_rows_alone_that_positions_own():
    spec = {"k": ((6, 2), torch.float32, "by_position"),
            "S": ((2,), torch.float32)}
    c = SequenceCache([spec], 2, 6, "cpu")
    c.layers[0]["S"].fill_(3.0)
    snap = c.snapshot()
    assert list(snap[1][0]) == ["S"]
    c.layers[0]["S"].zero_()
    c.layers[0]["k"].fill_(1.0)
    c.restore(snap)
    assert float(c.layers[0]["S"].min()) == 3.0
    assert float(c.layers[0]["k"].min()) == 1.0
    c.reserve(4)
    assert c.layers[0]["k"].shape == (4, 6, 2)


def test_cli_info_reads_a_plain_checkpoint(tmp_path):
    from typer.testing import CliRunner
    from lfmq.cli import app
    cfg = util.CONFIGS["odd"]
    path = util.write_checkpoint(tmp_path / "m", cfg, util.weights(cfg))
    r = CliRunner().invoke(app, ["info", "--ckpt", path])
    assert r.exit_code == 0, r.output
    d = json.loads(r.output)
    assert d["arch"] == "zatasun" and d["n_layers"] == 2
