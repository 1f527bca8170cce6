"""Rapivik on the CPU: configuration, checkpoint names, cache bookkeeping,
request batching and the trace runner's protocol."""
import io
import json
import math

import numpy as np
import pytest
import torch

import rapivik_oracle as oracle
import rapivik_util as util
import lfmq
from lfmq.models.generation import PackedStepper, generate_batch
from lfmq.models.rapivik import RapivikConfig, convert_state
from lfmq.models.registry import ARCHS, read_plain_config, spec_of
from lfmq.models.seqcache import SequenceCache


# ---- the oracle itself ------------------------------------------------------

def test_oracle_recurrence_matches_its_closed_form():
    """Unrolled, the state is a decayed sum of outer products."""
    g = torch.Generator().manual_seed(0)
    T, dk, dv = 9, 3, 4
    q, k, v = (torch.randn(T, n, generator=g, dtype=torch.float64)
               for n in (dk, dk, dv))
    i = torch.randn(T, generator=g, dtype=torch.float64) * 3
    f = -torch.rand(T, generator=g, dtype=torch.float64)
    st = (torch.zeros(dk, dv, dtype=torch.float64),
          torch.zeros(dk, dtype=torch.float64), 0.0)
    for t in range(T):
        o, st = oracle.mlstm_cell(q[t], k[t], v[t], float(i[t]), float(f[t]),
                                  st)
        decay = torch.stack([f[s + 1:t + 1].sum() + i[s] for s in range(t + 1)])
        m = max(float(f[:t + 1].sum()), float(decay.max()))
        p = torch.exp(decay - m) * (k[:t + 1] @ q[t])
        den = max(abs(float(p.sum())), math.exp(-m)) + 1e-6
        assert torch.allclose(o, (p @ v[:t + 1]) / den, atol=1e-12)


def test_oracle_bigram_rows():
    assert oracle.bigram_rows([4, 2, 9], 10, 3, 7) == [10, 26 % 10, 69 % 10]
    assert oracle.bigram_rows([2], 10, 3, 7, prev=4) == [6]


def test_oracle_sink_is_in_the_denominator_only():
    v = torch.ones(2, 3, dtype=torch.float64)
    o = oracle.sink_attend(torch.zeros(2, dtype=torch.float64), v,
                           torch.tensor(0.0))
    assert torch.allclose(o, torch.full((3,), 2 / 3, dtype=torch.float64))


# ---- configuration and registry ------------------------------------------------

def test_config_round_trip():
    for cfg in util.CONFIGS.values():
        c = RapivikConfig.from_dict(cfg)
        assert c.n_layers == len(cfg["layers"])
        assert RapivikConfig.from_dict(c.to_dict()) == c
        assert spec_of(c.to_dict()) is spec_of(cfg) is ARCHS["rapivik"]


def test_config_rejects_what_it_cannot_run():
    with pytest.raises(ValueError, match="unknown mixer"):
        RapivikConfig.from_dict(util.config([{**util.mlstm(), "type": "x"}]))
    with pytest.raises(ValueError, match="feed-forward"):
        RapivikConfig.from_dict(util.config(
            [{**util.mlstm(), "mlp": {"kind": "moe", "ff": 8}}]))
    with pytest.raises(ValueError, match="differs"):
        RapivikConfig.from_dict(util.config(
            [util.mlstm(), util.mlstm(dim=16, weights_of=0)]))
    with pytest.raises(ValueError, match="circular"):
        RapivikConfig.from_dict(util.config(
            [util.mlstm(weights_of=1), util.mlstm(weights_of=0)]))
    with pytest.raises(ValueError, match="unknown arch"):
        lfmq.build_model({"arch": "nope"})


def test_shared_weights_are_one_module_with_states_of_their_own():
    cfg = RapivikConfig.from_dict(util.CONFIGS["mixed"])
    m = lfmq.build_model(cfg)
    assert m.order == ["l0", "l1", "l2", "l3", "l0", "l1"]
    assert list(m.blocks) == ["l0", "l1", "l2", "l3"]
    cache = m.make_cache(2, max_seq=100)
    assert len(cache.layers) == 6
    assert cache.layers[0]["S"].data_ptr() != cache.layers[4]["S"].data_ptr()


def test_depth_override():
    c = RapivikConfig.from_dict(util.CONFIGS["mixed"])
    c.n_layers = 9
    assert [e["type"] for e in c.layers[:2]] == [e["type"]
                                                 for e in c.layers[6:8]]
    assert all("weights_of" not in e for e in c.layers)
    c.n_layers = 2
    assert len(c.layers) == 2


# ---- checkpoint --------------------------------------------------------------

def test_plain_checkpoint_loads(tmp_path):
    cfg = util.CONFIGS["mixed"]
    w = util.weights(cfg)
    path = util.write_checkpoint(tmp_path / "m", cfg, w)
    assert read_plain_config(path) == cfg
    for dt in (torch.bfloat16, torch.float32):
        m = lfmq.load(path, dtype=dt)
        b = m.blocks["l0"].mixer
        assert b.in_proj.weight.dtype == dt
        assert b.norm_w.dtype == b.gate_b.dtype == torch.float32
        assert torch.equal(b.gate_w, torch.cat([w["l0.mix.i"],
                                                w["l0.mix.f"]]).to(dt))
        n = w["l0.mix.q"].shape[0]
        assert torch.equal(b.in_proj.weight[n:2 * n], w["l0.mix.k"].to(dt))
        a = m.blocks["l1"].mixer
        uk, uv = a.absorbed()
        assert torch.equal(uk.reshape(-1, a.rank), w["l1.mix.uk"].to(dt))
        assert torch.equal(uv.transpose(1, 2).reshape(-1, a.rank),
                           w["l1.mix.uv"].to(dt))
        assert torch.equal(a.sink, w["l1.mix.sink"].float())
        assert not any(p.is_meta for p in m.parameters())


def test_checkpoint_names_are_checked(tmp_path):
    cfg = util.CONFIGS["mixed"]
    c = RapivikConfig.from_dict(cfg)
    w = util.weights(cfg)
    with pytest.raises(KeyError, match="l3.mix.sink"):
        convert_state(c, {k: v for k, v in w.items() if k != "l3.mix.sink"})
    with pytest.raises(KeyError, match="unknown"):
        convert_state(c, {**w, "l9.norm1": w["l0.norm1"]})
    bad = {**w, "head": w["head"][:-1].contiguous()}
    with pytest.raises(ValueError, match="lm_head"):
        lfmq.load(util.write_checkpoint(tmp_path / "b", cfg, bad))


def test_absorbed_weights_follow_the_parameter():
    m = lfmq.build_model(RapivikConfig.from_dict(util.CONFIGS["mixed"]),
                         seed=1)
    a = m.blocks["l1"].mixer
    first = a.absorbed()[1]
    assert a.absorbed()[1] is first
    with torch.no_grad():
        a.kv_up.mul_(2.0)
    assert torch.equal(a.absorbed()[1], first * 2)


def test_gpu_only_and_rtn_only():
    m = lfmq.build_model(RapivikConfig.from_dict(util.CONFIGS["mixed"]))
    with pytest.raises(RuntimeError, match="GPU"):
        m(torch.zeros(1, 3, dtype=torch.int64), m.make_cache(1, max_seq=8))
    with pytest.raises(NotImplementedError, match="rtn"):
        lfmq.quantize(m, lfmq.QuantConfig(scheme="gptq"))


# ---- cache -------------------------------------------------------------------

def _cache(n=3, max_seq=50):
    return SequenceCache([{"ring": ((4, 2), torch.float32)}], n, max_seq,
                         "cpu")


def test_slots_are_given_out_and_back():
    c = _cache()
    a, b, d = c.alloc(), c.alloc(), c.alloc()
    assert sorted((a, b, d)) == [0, 1, 2]
    with pytest.raises(RuntimeError, match="slots"):
        c.alloc()
    c.lens_host[b], c.lens[b] = 7, 7
    c.free([b])
    assert c.lens_host[b] == 0 and int(c.lens[b]) == 0
    assert c.alloc() == b
    c.free([a])
    with pytest.raises(ValueError, match="free already"):
        c.free([a])


def test_reserve_keeps_live_slots():
    c = _cache()
    s = c.alloc()
    c.layers[0]["ring"][s] = 5.0
    c.lens_host[s], c.lens[s] = 3, 3
    c.reserve(6)
    assert c.n_slots == 6 and c.free_slots == 5
    assert float(c.layers[0]["ring"][s].min()) == 5.0
    assert c.layers[0]["ring"].shape[0] == 6 and int(c.lens[s]) == 3
    assert len({c.alloc() for _ in range(5)} | {s}) == 6


def test_step_batches_are_checked():
    c = _cache()
    with pytest.raises(ValueError):
        c.batch([0], [0])
    with pytest.raises(ValueError):
        c.batch([0, 0], [1, 1])
    with pytest.raises(RuntimeError, match="overflow"):
        c.batch([0], [51])


def test_step_batch_layout():
    c = _cache()
    c.lens_host = [0, 30, 2]
    b = c.batch([2, 0, 1], [3, 1, 2])
    assert b.seq.tolist() == [0, 0, 0, 1, 2, 2]
    assert b.cu.tolist() == [0, 3, 4, 6]
    assert b.slots.tolist() == [2, 0, 1]
    assert b.last_rows_host == [2, 3, 5] and not b.single
    r = b.key_rows(5)            # windows of 5 reach back 4 tokens
    assert r.prior.tolist() == [2, 0, 4]
    assert r.own.tolist() == [2, 5, 10] and r.total == 12 and r.any_prior
    assert b.key_rows(1).total == 6 and not b.key_rows(1).any_prior
    base, total = b.chunks(2)
    assert base.tolist() == [0, 2, 3] and total == 4


def test_snapshot_restores():
    c = _cache()
    c.layers[0]["ring"].fill_(2.0)
    c.lens_host[0], c.lens[0] = 4, 4
    snap = c.snapshot()
    c.layers[0]["ring"].zero_()
    c.replayed(3)
    c.lens += 3
    c.restore(snap)
    assert float(c.layers[0]["ring"].min()) == 2.0
    assert c.lens_host == [4, 0, 0] and c.lens.tolist() == [4, 0, 0]


# ---- batching, over a stand-in model --------------------------------------------

class Echo:
    """Next token = (sum of the sequence's tokens) mod vocab."""
    packed = True

    class cfg:
        vocab_size = 11
        arch = "echo"

    class norm:
        weight = torch.zeros(1)

    def __init__(self):
        self.batches = []

    def make_cache(self, n, max_seq=None, device=None):
        c = SequenceCache([{"sum": ((1,), torch.float32)}], n, max_seq, "cpu")
        return c

    def forward_tokens(self, tok, batch, cache, select):
        self.batches.append(list(batch.slot_ids))
        out = torch.zeros(batch.n, 11)
        at = 0
        for s, n in zip(batch.slot_ids, batch.counts):
            if cache.lens_host[s] == 0:
                cache.layers[0]["sum"][s] = 0
            for t in tok[at:at + n].tolist():
                cache.layers[0]["sum"][s] += t
                out[at, int(cache.layers[0]["sum"][s]) % 11] = 1.0
                at += 1
            cache.lens_host[s] += n
        return out[select]


def test_generate_batch_unequal_prompts_and_eos():
    m = Echo()
    alone = [generate_batch(Echo(), [p], 6)[0] for p in ([1, 2], [5], [3] * 4)]
    assert generate_batch(m, [[1, 2], [5], [3] * 4], 6) == alone
    eos = alone[1][2]
    cut = generate_batch(m, [[1, 2], [5], [3] * 4], gen_cfg=
                         lfmq.GenerationConfig(max_new_tokens=6,
                                               eos_token_id=eos))
    for got, full, n in zip(cut, alone, (2, 1, 4)):
        new = full[n:]
        end = new.index(eos) + 1 if eos in new else len(new)
        assert got == full[:n + end]
    assert len(m.batches[-1]) < 3          # the finished ones left


def test_stepper_reuses_slots_and_validates():
    st = PackedStepper(Echo(), 40, 1)
    a = st.step([("a", [1, 2], [1]), ("b", [4], [0])])
    assert a.argmax(-1).tolist() == [3, 4] and st.cache.n_slots == 2
    st.end(["a"])
    assert st.step([("c", [6], [0]), ("b", [3], [0])]).argmax(-1).tolist() \
        == [6, 7]
    assert st.cache.n_slots == 2
    assert st.step([("b", [1], [])]).shape[0] == 0
    for bad in ([("b", [], [])], [("b", [11], [])], [("b", [-1], [])],
                [("b", [1], [1])], [("b", [1], []), ("b", [1], [])]):
        with pytest.raises(ValueError):
            st.step(bad)


def test_trace_runner_protocol(tmp_path, monkeypatch, capsys):
    from lfmq import api, replay
    from lfmq.ops import build
    seen = {}

    def load(path, device, dtype):
        seen.update(path=path, dtype=dtype)
        return Echo()

    monkeypatch.setattr(api, "load", load)
    monkeypatch.setattr(build, "ensure_built", lambda name: None)
    lines = [
        {"step": 0, "entries": [{"id": "a", "tokens": [1, 2], "want": [0, 1]},
                                {"id": "b", "tokens": [5], "want": []}],
         "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": [5], "want": []}],
         "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": [4], "want": [0]}],
         "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "".join(json.dumps(x) + "\n" for x in lines)))
    assert replay.main(["--model", "m", "--dtype", "float32", "--out",
                        str(tmp_path), "--max-tokens", "16"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1",
                                                      "done 2"]
    assert seen == {"path": "m", "dtype": torch.float32}
    assert sorted(p.name for p in tmp_path.iterdir()) == ["0.f32", "2.f32"]
    a = np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, 11)
    assert a.argmax(-1).tolist() == [1, 3]


def test_server_rejects_unequal_prompts_without_packed_batches():
    from fastapi.testclient import TestClient
    from lfmq.models.llama import LlamaConfig
    from lfmq.obs.serve import make_app
    app = TestClient(make_app(lfmq.build_model(LlamaConfig.tiny(), seed=0)))
    r = app.post("/generate", json={"input_ids": [[1, 2], [3]],
                                    "max_new_tokens": 2})
    assert r.status_code == 400
    assert app.post("/generate", json={"input_ids": [[]]}).status_code == 400


def test_cli_info_reads_a_plain_checkpoint(tmp_path):
    from typer.testing import CliRunner
    from lfmq.cli import app
    cfg = util.CONFIGS["odd"]
    path = util.write_checkpoint(tmp_path / "m", cfg, util.weights(cfg))
    r = CliRunner().invoke(app, ["info", "--ckpt", path])
    assert r.exit_code == 0, r.output
    d = json.loads(r.output)
    assert d["arch"] == "rapivik" and d["n_layers"] == 3
