"""Napadra without a GPU: configuration and registry, the reach of chunks in the scheduler, the step batch's tiles, tensor-parallel
slices, and the plain evaluation's mechanisms against values worked out by hand."""
import copy
import math
import random
import types

import pytest
import torch

from napadra_util import CONFIGS, attn, config, make_model, mlstm
from oracle import napadra_oracle as O
from test_dafolorn_cpu import _drive, _scheduler

D = torch.float64


def t64(x):
    return torch.tensor(x, dtype=D)


# ---- mechanisms of the plain evaluation ------------------------------------------------------------------------------------
def test_sinusoid_by_hand():
    s = O.sinusoid(3, 6)
    for p in range(3):
        for i in range(3):
            a = p / 10000 ** (2 * i / 6)
            assert abs(s[p, 2 * i] - math.sin(a)) < 1e-12 and abs(s[p, 2 * i + 1] - math.cos(a)) < 1e-12


def test_streams_by_hand():
    x = t64([[[1.0, 2.0], [10.0, 20.0]]])                 # one token, two streams
    assert O.collapse(x, t64([3.0, 0.5])).tolist() == [[8.0, 16.0]]
    out = O.spread(x, t64([[1.0, 2.0], [3.0, 4.0]]), t64([0.0, 1.0]), t64([[100.0, 200.0]]))
    # to stream 0: 1 x_0 + 3 x_1; to stream 1: 2 x_0 + 4 x_1 + y
    assert out.tolist() == [[[31.0, 62.0], [142.0, 284.0]]]


def test_shift_and_norm_by_hand():
    h = t64([[2.0, 4.0], [6.0, 8.0]])
    assert O.token_shift(h, t64([0.5, 1.0])).tolist() == [[1.0, 0.0], [4.0, 4.0]]
    assert torch.allclose(O.unit_rms(t64([[3.0, 4.0]]), 0.5), t64([[3.0, 4.0]]) / math.sqrt(13.0))


def test_clamped_glu_by_hand():
    sg = lambda z: 1 / (1 + math.exp(-1.702 * z))  # noqa: E731
    got = O.clamped_glu(t64([1.0, 5.0, -5.0, 1.0]), t64([0.5, 9.0, -9.0, 0.0]), 2.0).tolist()
    want = [1 * sg(1) * 1.5, 2 * sg(2) * 3, -5 * sg(-5) * -1, sg(1)]
    assert all(abs(a - b) < 1e-12 for a, b in zip(got, want))


def test_chunks_bias_and_sink_by_hand():
    assert O.chunk_mask(5, 2).int().tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
    assert [O.slope(h, 4) for h in range(4)] == [0.25, 0.0625, 0.015625, 0.00390625]
    # two heads on one key/value head, two tokens of one chunk: weights of token 1 are 1 / e^slope : 1 : e^sink
    W = O.Weights({"q": torch.zeros(2, 1), "k": torch.zeros(1, 1), "v": torch.tensor([[1.0]]), "o": torch.eye(2), "sink": torch.tensor([0.0, math.log(2.0)])})
    spec = {"heads": 2, "kv_heads": 1, "dim": 1, "vdim": 1, "scale": 1.0, "mask": {"size": 8}}
    h = t64([[3.0], [5.0]])
    out = O.attention(h, W, "", spec, O.keys_values(h, W, "", spec))
    for i, (sl, sink) in enumerate(((2.0 ** -4, 1.0), (2.0 ** -8, 2.0))):
        e = math.exp(-sl)
        assert abs(out[1, i] - (3 * e + 5) / (e + 1 + sink)) < 1e-6 and abs(out[0, i] - 3 / (1 + sink)) < 1e-6


def test_matrix_memory_by_hand():
    """One dimension: the recurrence written out for three tokens; the maximum starts at zero, not at minus infinity."""
    q, k, v, i, f = [0.5, 2.0, -1.0], [1.0, -1.0, 3.0], [2.0, 4.0, 8.0], [-3.0, 1.0, -2.0], [-0.1, -0.7, -2.0]
    S = n = m = 0.0
    want = []
    for a in range(3):
        mn = max(f[a] + m, i[a])
        S, n = math.exp(f[a] + m - mn) * S + math.exp(i[a] - mn) * k[a] * v[a], math.exp(f[a] + m - mn) * n + math.exp(i[a] - mn) * k[a]
        m = mn
        want.append(S * q[a] / (max(abs(n * q[a]), math.exp(-m)) + 1e-6))
    got = O.mlstm_cell(t64(q)[:, None], t64(k)[:, None], t64(v)[:, None], t64(i), t64(f))
    assert torch.allclose(got[:, 0], t64(want), atol=1e-12) and m != max(i)
    assert abs(float(O.log_sigmoid(t64(-3.0))) + math.log(1 + math.exp(3.0))) < 1e-12 and abs(float(O.soft_cap(t64(5.0), 2.0)) - 2 * math.tanh(2.5)) < 1e-12


# ---- configuration and registry -----------------------------------------------------------------------------------------------
def test_registry_and_config(tmp_path):
    from nanovllm.config import Config
    from nanovllm.models.registry import find_model
    assert find_model({"architecture": "Napadra"}).name == "napadra" and find_model({"architecture": "Dafolorn"}).name == "dafolorn"
    make_model(tmp_path, "odd")
    c = Config(str(tmp_path), dtype="float32", max_model_len=100000, max_num_batched_tokens=64)
    hf = c.hf_config
    assert c.kvcache_block_size == 64 and hf.torch_dtype == torch.float32 and hf.key_reach.chunks == (33, 150) and hf.key_reach.span == 150
    assert [s.type for s in hf.layers] == ["attention", "mlstm", "attention", "mlstm"] and hf.layers[2].kv_from == 0 and hf.layers[1].mlp is None
    assert hf.streams == 3 and hf.residual_mult == 0.4 and hf.layers[3].limit == 0.7 and hf.layers[3].gate_cap == 4.0
    with pytest.raises(ValueError):
        Config(str(tmp_path), dtype="float16")


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][1].update(type="mystery"), "mystery"), (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "sparse"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(sinks=4), "sinks"), (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "layer 3"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "layer 1"), (lambda c: c["layers"][2]["mixer"].update(dim=24), "layer 0"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=2), "5 heads over 2"), (lambda c: c.update(streams=0), "0 streams")])
def test_what_the_design_does_not_have_is_refused(edit, match):
    from nanovllm.models.napadra.config import read_config
    c = copy.deepcopy(CONFIGS["odd"])
    edit(c)
    with pytest.raises((NotImplementedError, ValueError), match=match):
        read_config(c)


def test_loader_reports_missing_tensors(tmp_path):
    from nanovllm.models.napadra.config import read_config
    from nanovllm.models.napadra.model import NapadraForCausalLM
    cfg, t = make_model(tmp_path, "odd")
    for name in ("l1.mix.i.b", "l0.hc2.out", "l2.shift"):
        u = {k: v for k, v in t.items() if k != name}
        O.write_model(str(tmp_path / name), cfg, u)
        with pytest.raises(KeyError, match=name.split(".")[-1]):
            NapadraForCausalLM(read_config(cfg)).load_weights(str(tmp_path / name))


# ---- scheduler and step tables --------------------------------------------------------------------------------------------------
def test_key_reach():
    from nanovllm.engine.key_reach import KeyReach
    r = KeyReach(windows=(5,), chunks=(8, 12))
    for p in range(60):
        seen = [j for q in range(p, 60) for j in range(q + 1) if q - j < 5 or q // 8 == j // 8 or q // 12 == j // 12]
        assert r.first_visible(p) == min(seen), p
    assert KeyReach().first_visible(17) == 17 and KeyReach().span == 0


@pytest.mark.parametrize("chunks,preempts", [((40, 56), False), ((1000,), True), ((), False)])
def test_scheduler_with_chunks(chunks, preempts):
    """Blocks behind the chunks are given back, never one that a later token still sees."""
    from nanovllm.engine.key_reach import KeyReach
    from nanovllm.engine.sequence import Sequence
    from nanovllm.sampling_params import SamplingParams
    reach = KeyReach(chunks=chunks)
    sch = _scheduler(num_kvcache_blocks=13 if preempts else 8, max_num_batched_tokens=48, hf_config=types.SimpleNamespace(key_reach=reach))
    seqs = [Sequence(list(range(i * 1000, i * 1000 + n)), SamplingParams(temperature=0.0, max_tokens=60, ignore_eos=True)) for i, n in enumerate((120, 120, 120) if preempts else (340, 60, 90))]
    for s in seqs:
        sch.add(s)
    preempted, real = [], sch.preempt
    sch.preempt = lambda s: (preempted.append(s.seq_id), real(s))

    def check(batch):
        for _, c in batch:
            first = reach.first_visible(c.start)
            assert all(b >= 0 for b in c.block_table[first // 32:])

    done = _drive(sch, seqs, check, window=0)
    assert len(done) == 3 and all(s.num_completion_tokens == 60 for s in seqs) and bool(preempted) is preempts
    assert len(sch.block_manager.free_block_ids) == (13 if preempts else 8)


def test_step_tables_with_chunk_tiles():
    from nanovllm.engine.step_batch import Chunk, build_step
    rng = random.Random(3)
    for case in range(20):
        wanted = sorted({(rng.choice([1, 7, 64, 300]), rng.choice([64, 128])) for _ in range(3)})
        spec = types.SimpleNamespace(windows=(), tile_sizes=[1, 4], max_short_portion=16, chunk_tiles=wanted)
        chunks = []
        for i in range(rng.randint(1, 4)):
            start, n = rng.choice([0, 1, 63, 500]), rng.choice([1, 2, 16, 17, 130, 400])
            chunks.append(Chunk([1] * n, start, list(range(100 * i, 100 * i + -(-(start + n) // 64))), 2 * i, 2 * i + 1, []))
        host, on_device, _ = build_step(chunks, spec, 64)
        b = on_device(torch.from_numpy(host))
        longs = [c for c in chunks if len(c.tokens) > 16]
        assert b.n_short == len(chunks) - len(longs)
        if not longs:
            continue
        assert sorted(b.chunk_tiles) == wanted
        for (c, rows), (seq, off) in b.chunk_tiles.items():
            tiles = list(zip(seq.tolist(), off.tolist()))
            assert sorted(tiles) == sorted((s, o) for s, x in enumerate(longs) for o in range(0, len(x.tokens), rows))
            seen = [(longs[s].start + min(o + rows, len(longs[s].tokens)) - 1) % c for s, o in tiles]
            assert seen == sorted(seen, reverse=True)


# ---- tensor parallelism -----------------------------------------------------------------------------------------------------------
def test_tensor_parallel_slices_add_up(monkeypatch):
    """Two ranks' heads, state heads and feed-forward columns, evaluated in plain arithmetic over the loaded (padded, sliced) weights: the sum
    over the ranks is the whole model's sublayer."""
    from nanovllm.layers import dense_mlp, group_attention, matrix_memory
    cfg = config(40, 64, 2, [attn(8, 4, 12, 20, 9, 44, 1.5), mlstm(4, 12, 20)])
    t = {k: v.float() for k, v in O.random_tensors(cfg, 3).items()}
    h = torch.randn(21, 40, generator=torch.Generator().manual_seed(1))
    W, hd = O.Weights(t), h.double()
    sa, sm = cfg["layers"][0]["mixer"], cfg["layers"][1]["mixer"]
    want = [O.attention(hd, W, "l0.mix.", sa, O.keys_values(hd, W, "l0.mix.", sa)), O.dense_mlp(hd, W, "l0.mlp.", 1.5), O.mlstm(hd, W, "l1.mix.", sm, 1e-5)]
    got = [0.0, 0.0, 0.0]
    part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
    dist = (torch.arange(21)[:, None] - torch.arange(21)[None, :]).double()
    for rank in range(2):
        g = types.SimpleNamespace(world_size=2, rank=rank)
        for mod in (dense_mlp, group_attention, matrix_memory):
            monkeypatch.setattr(mod, "get_tp_group", lambda: g)
        a = group_attention.GroupAttention(40, 8, 4, 12, 20, 12 ** -0.5, torch.float32, chunk=9, biased=True)
        a.load(part("l0.mix."), "cpu")
        x = (h @ a.qkv_proj.weight.T).double()
        q, k, v = x[:, : 4 * 16].view(21, 4, 16), x[:, 64: 64 + 32].view(21, 2, 16), x[:, 96:].view(21, 2, 24)
        out = torch.stack([O.sink_softmax(q[:, i] @ k[:, i // 2].T * a.scale - a.slope[i].double() * dist, O.chunk_mask(21, 9), a.sink[i].double()) @ v[:, i // 2] for i in range(4)], 1)
        got[0] = got[0] + out.reshape(21, -1).float() @ a.o_proj.weight.T
        m = dense_mlp.GatedMLP(40, 44, 1.5, torch.float32)
        m.load(part("l0.mlp."), "cpu")
        z = h @ m.gate_up.weight.T
        got[1] = got[1] + O.clamped_glu(z[:, :24], z[:, 24:], 1.5) @ m.down.weight.T
        e = matrix_memory.MatrixMemory(40, 4, 12, 20, 9.0, 1e-5, torch.float32)
        e.load(part("l1.mix."), "cpu")
        x, z = (h @ e.in_proj.weight.T).double(), (h @ e.gates.weight[:4].T + e.gate_bias).double()
        q, k, v, gt = x[:, :32].view(21, 2, 16) * 12 ** -0.5, x[:, 32:64].view(21, 2, 16), x[:, 64:112].view(21, 2, 24), x[:, 112:]
        o = torch.stack([O.mlstm_cell(q[:, i], k[:, i], v[:, i], O.soft_cap(z[:, i], 9.0), O.log_sigmoid(O.soft_cap(z[:, 2 + i], 9.0))) for i in range(2)], 1)
        o = o / torch.sqrt((o * o).sum(-1, keepdim=True) / 20 + 1e-5)
        got[2] = got[2] + (o.reshape(21, -1) * e.norm * torch.sigmoid(gt)).float() @ e.o_proj.weight.T
    for a, b in zip(got, want):
        assert torch.allclose(a[:, :40].double(), b, atol=2e-5, rtol=1e-4)
    with pytest.raises(ValueError, match="do not split"):
        monkeypatch.setattr(group_attention, "get_tp_group", lambda: types.SimpleNamespace(world_size=8, rank=0))
        group_attention.GroupAttention(40, 8, 4, 12, 20, 0.3, torch.float32)
