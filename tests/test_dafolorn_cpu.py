"""Dafolorn without a GPU: configuration and registry, the step batch's tables, the scheduler for step batches, tensor-parallel
slices, and the plain evaluation's mechanisms against values worked out by hand."""
import json
import math
import random
import types

import numpy as np
import pytest
import torch

from dafolorn_util import CONFIGS, config, layer, make_model
from oracle import dafolorn_oracle as O


# ---- mechanisms of the plain evaluation ------------------------------------------------------------------------------------
def test_norms_by_hand():
    x = torch.tensor([[3.0, 4.0]]).double()
    r = 1 / math.sqrt(12.5 + 0.5)
    assert torch.allclose(O.norm_zero_centred(x, torch.tensor([0.0, 1.0]).double(), 0.5), torch.tensor([[3 * r, 8 * r]]).double())
    assert torch.allclose(O.norm_plain(x, torch.tensor([0.0, 1.0]).double(), 0.5), torch.tensor([[0.0, 4 * r]]).double())


def test_xielu_by_hand():
    p, q = torch.tensor(0.0).double(), torch.tensor(1.0).double()
    z = torch.tensor([2.0, 0.0, -1.0]).double()
    sp0, sp1 = math.log(2), math.log(1 + math.e)
    want = [sp0 * 4 + 1, 0.0, (0.5 + sp1) * (math.exp(-1) - 1 + 1) - 0.5]
    assert torch.allclose(O.xielu(z, p, q), torch.tensor(want).double())
    from nanovllm.layers.dense_mlp import xielu_constants
    _, a, b = xielu_constants(torch.tensor([0.0, 1.0]).to(torch.bfloat16))
    assert abs(a - sp0) < 1e-6 and abs(b - (0.5 + sp1)) < 1e-6


def test_canon_by_hand():
    h = torch.tensor([[1.0], [10.0], [100.0]]).double()
    w = torch.tensor([[2.0, 3.0]]).double()      # previous token x 2, current x 3
    assert O.canon(h, w).flatten().tolist() == [1 + 3, 10 + 2 + 30, 100 + 20 + 300]


def test_window_and_sink_by_hand():
    vis = O.window_mask(4, 2)
    assert vis.int().tolist() == [[1, 0, 0, 0], [1, 1, 0, 0], [0, 1, 1, 0], [0, 0, 1, 1]]
    a = O.sink_softmax(torch.zeros(4, 4).double(), vis, torch.tensor(math.log(3.0)).double())
    assert torch.allclose(a[0, 0], torch.tensor(1 / 4).double()) and torch.allclose(a[3], torch.tensor([0, 0, 1 / 5, 1 / 5]).double())


# ---- configuration and registry -----------------------------------------------------------------------------------------------
def test_registry_and_config(tmp_path):
    from nanovllm.config import Config
    from nanovllm.models.registry import find_model
    assert find_model({"model_type": "glm4_moe"}).name == "glm4_moe" and find_model({"architecture": "Dafolorn"}).name == "dafolorn"
    assert find_model({"architectures": ["Glm4MoeForCausalLM"]}).name == "glm4_moe"
    with pytest.raises(NotImplementedError):
        find_model({"architecture": "Unheard"})
    make_model(tmp_path, "odd")
    c = Config(str(tmp_path), dtype="float32", max_model_len=100000, max_num_batched_tokens=64)
    assert c.kvcache_block_size == 64 and c.hf_config.torch_dtype == torch.float32 and c.max_model_len == 100000
    assert c.hf_config.logit_softcap is None and c.hf_config.max_window == 150 and c.hf_config.layers[1].mlp is None
    with pytest.raises(ValueError):
        Config(str(tmp_path), dtype="float16")
    bad = json.loads(json.dumps(CONFIGS["odd"]))
    bad["layers"][1]["type"] = "mystery"
    with open(tmp_path / "config.json", "w") as f:
        json.dump(bad, f)
    with pytest.raises(NotImplementedError, match="mystery"):
        Config(str(tmp_path))


def test_layer_runs():
    from nanovllm.models.dafolorn.config import layer_runs, read_config
    runs = {n: layer_runs(read_config(c)) for n, c in CONFIGS.items()}
    assert runs["odd"] == [(0, 0), (1, None), (0, 1), (1, None), (0, 2), (1, None), (2, None)]
    assert runs["wide"] == [(0, None), (1, 0), (2, None)] and runs["tall"] == [(0, None), (1, None)]
    assert runs["huge"] == [(0, 0), (0, 1), (1, None)]
    assert runs["tail"] == [(0, None), (1, 0), (2, None), (1, 1), (2, None)]


def test_trace_runner_refuses_a_dtype_no_model_runs_in(tmp_path):
    from nanovllm import trace
    with open(tmp_path / "config.json", "w") as f:
        json.dump({"model_type": "glm4_moe"}, f)
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"]) == 3


# ---- step batches ---------------------------------------------------------------------------------------------------------------
def _spec(windows, tiles, limit):
    return types.SimpleNamespace(windows=windows, tile_sizes=tiles, max_short_portion=limit)


def test_step_tables():
    """Every row's token, position, cache row and history, and the tiles, against a direct walk over the chunks."""
    from nanovllm.engine.step_batch import Chunk, build_step
    rng = random.Random(4)
    bs = 32
    for case in range(20):
        free = list(range(200))
        rng.shuffle(free)
        windows, tiles, limit = sorted({rng.choice([1, 5, 33, 64, 200]) for _ in range(2)}), sorted({1, rng.choice([3, 10])}), rng.choice([1, 8, 20])
        chunks = []
        for _ in range(rng.randint(1, 5)):
            start, n = rng.choice([0, 1, 31, 32, 150]), rng.choice([1, 1, 2, 9, 40, 300])
            table = [free.pop() for _ in range(-(-(start + n) // bs))]
            dead = max(0, start - max(windows) + 1) // bs         # blocks behind every window have been given back
            table[:dead] = [-1] * dead
            want = sorted(rng.sample(range(n), rng.randint(0, min(n, 3))))
            chunks.append(Chunk([rng.randint(0, 99) for _ in range(n)], start, table, rng.randint(0, 9), rng.randint(0, 9), want))
        host, on_device, _ = build_step(chunks, _spec(windows, tiles, limit), bs)
        b = on_device(torch.from_numpy(host))
        order = sorted(range(len(chunks)), key=lambda i: len(chunks[i].tokens) > limit)
        row, first = 0, {}
        slot = lambda c, p: c.block_table[p // bs] * bs + p % bs  # noqa: E731
        for s, i in enumerate(order):
            c = chunks[i]
            first[i] = row
            assert b.q_start[s] == row and b.state_in[s] == c.state_in and b.state_out[s] == c.state_out
            for k, t in enumerate(c.tokens):
                assert (b.ids[row + k], b.pos[row + k], b.seq_of[row + k], b.slots[row + k]) == (t, c.start + k, s, slot(c, c.start + k))
            row += len(c.tokens)
        assert b.q_start[-1] == row == b.ids.numel()
        assert b.want.tolist() == [first[i] + w for i, c in enumerate(chunks) for w in c.want]
        short = [i for i in order if len(chunks[i].tokens) <= limit]
        assert b.Ta == sum(len(chunks[i].tokens) for i in short)
        for size, (tok, cnt) in b.tiles.items():
            rows = [r for t, n in zip(tok.tolist(), cnt.tolist()) for r in range(t, t + n)]
            assert rows == list(range(b.Ta)) and (not cnt.numel() or cnt.max() <= size)
            assert all(b.seq_of[t] == b.seq_of[t + n - 1] for t, n in zip(tok.tolist(), cnt.tolist()))
        if b.Ta == row:
            continue
        longs = order[len(short):]
        cover = {(s, o) for s, o in zip(b.long_tile_seq.tolist(), b.long_tile_off.tolist())}
        assert cover == {(s, o) for s, i in enumerate(longs) for o in range(0, len(chunks[i].tokens), 128)}
        assert b.long_q_start.tolist() == [first[i] - b.Ta for i in longs] + [row - b.Ta]
        for w, t in b.windows.items():
            k, seen = 0, set()
            for s, i in enumerate(longs):
                c, hist = chunks[i], min(chunks[i].start, w - 1)
                assert t.k_start[s] == k
                for j in range(hist):
                    m = (t.hist_rows == k + j).nonzero().flatten()
                    assert m.numel() == 1 and t.hist_slots[m] == slot(c, c.start - hist + j)
                for j in range(len(c.tokens)):
                    assert t.crow[first[i] + j] == k + hist + j
                    seen.add(first[i] + j)
                k += hist + len(c.tokens)
            assert t.rows == k == t.k_start[-1] and all(t.crow[r] == -1 for r in range(row) if r not in seen)


def test_padded_decode_step_has_the_same_layout_whatever_it_holds():
    from nanovllm.engine.step_batch import Chunk, build_step
    spec = _spec([64], [1], 16)
    empty, on_empty, _ = build_step([], spec, 64, pad_rows=4, table_width=3)
    some, on_some, _ = build_step([Chunk([7], 70, [5, 9], 2, 3, [0]), Chunk([8], 0, [1], 0, 1, [0])], spec, 64, pad_rows=4, table_width=3)
    assert empty.shape == some.shape
    a = on_empty(torch.from_numpy(some))      # a captured step reads the new contents through the old views
    assert a.ids.tolist() == [7, 8, 0, 0] and a.pos.tolist() == [70, 0, -1, -1] and a.slots.tolist() == [9 * 64 + 6, 64, -1, -1]
    assert a.state_out.tolist() == [3, 1, -1, -1] and a.q_start.tolist() == [0, 1, 2, 3, 4] and a.block_tables[0].tolist() == [5, 9, -1]


# ---- scheduler ------------------------------------------------------------------------------------------------------------------
def _scheduler(**kw):
    from nanovllm.engine.scheduler import StepScheduler
    base = dict(max_num_seqs=3, max_num_batched_tokens=40, eos=-1, num_kvcache_blocks=12, kvcache_block_size=32,
                hf_config=types.SimpleNamespace(max_window=50))
    base.update(kw)
    return StepScheduler(types.SimpleNamespace(**base))


def _drive(sch, seqs, check=lambda batch: None, window=50):
    """Runs to the end; a token is its predecessor + 1.  Every token of every sequence must be computed in order."""
    done = {}
    for _ in range(2000):
        if sch.is_finished():
            return done
        batch = sch.schedule()
        check(batch)
        toks = []
        held = [b for s in list(sch.running) for b in s.block_table if b >= 0]
        assert len(held) == len(set(held)) == len(sch.block_manager.used_block_ids)
        states = [s.state_slot for s in sch.running]
        assert min(states) >= 0 and len(set(states)) == len(states)
        for seq, c in batch:
            assert c.start == seq.num_computed_tokens and c.tokens == seq.token_ids[c.start: c.start + len(c.tokens)]
            assert len(c.block_table) * 32 >= c.start + len(c.tokens)
            first = max(0, c.start - window + 1)   # (window 0: the caller checks the blocks)
            assert all(b >= 0 for b in c.block_table[first // 32: -(-(c.start + len(c.tokens)) // 32)])
            assert {c.state_in, c.state_out} == {2 * seq.state_slot, 2 * seq.state_slot + 1}
            if c.want:
                assert c.want == [len(c.tokens) - 1]
                toks.append(c.tokens[-1] + 1)
        sch.postprocess(batch, toks)
        done.update({s.seq_id: s for s, _ in batch if s.is_finished})
    raise AssertionError("the scheduler does not come to an end")


def test_step_scheduler_mixes_portions_and_decoded_tokens():
    from nanovllm.engine.sequence import Sequence
    from nanovllm.sampling_params import SamplingParams
    sch = _scheduler()
    seqs = [Sequence(list(range(1000 * i, 1000 * i + n)), SamplingParams(temperature=0.0, max_tokens=9, ignore_eos=True)) for i, n in enumerate((3, 130, 40, 1, 77))]
    for s in seqs:
        sch.add(s)
    mixed, budget = [], []

    def check(batch):
        n = [len(c.tokens) for _, c in batch]
        budget.append(sum(n))
        mixed.append(1 in n and max(n) > 1)

    done = _drive(sch, seqs, check)
    assert len(done) == 5 and all(s.completion_token_ids == list(range(s.prompt_token_ids[-1] + 1, s.prompt_token_ids[-1] + 10)) for s in seqs)
    assert any(mixed) and max(budget) <= 40
    assert len(sch.block_manager.free_block_ids) == 12 and len(sch.state_manager.free_slots) == 3


@pytest.mark.parametrize("window,preempts", [(50, False), (1000, True)])
def test_step_scheduler_under_want_of_pages(window, preempts):
    """With a window of 50 a sequence of 400 tokens holds a few blocks of 32 at a time and three run side by side in six; with a
    long window three sequences that grow from 4 to 6 blocks do not fit 13, the newest gives way and starts over."""
    from nanovllm.engine.sequence import Sequence
    from nanovllm.sampling_params import SamplingParams
    sch = _scheduler(num_kvcache_blocks=13 if preempts else 6, max_num_batched_tokens=64, hf_config=types.SimpleNamespace(max_window=window))
    seqs = [Sequence(list(range(i * 1000, i * 1000 + n)), SamplingParams(temperature=0.0, max_tokens=60, ignore_eos=True)) for i, n in enumerate((120, 120, 120) if preempts else (340, 60, 90))]
    for s in seqs:
        sch.add(s)
    preempted, real = [], sch.preempt
    sch.preempt = lambda s: (preempted.append(s.seq_id), real(s))
    done = _drive(sch, seqs, window=window)
    assert len(done) == 3 and all(s.num_completion_tokens == 60 for s in seqs) and bool(preempted) is preempts
    with pytest.raises(RuntimeError, match="too small"):
        tiny = _scheduler(num_kvcache_blocks=1, max_num_batched_tokens=64)
        tiny.add(Sequence(list(range(64))))
        tiny.schedule()


# ---- tensor parallelism -----------------------------------------------------------------------------------------------------------
def test_tensor_parallel_slices_add_up(monkeypatch):
    """Two ranks' heads and feed-forward columns, evaluated in plain fp32 over the loaded (padded, sliced) weights: the sum over
    the ranks is the whole model's sublayer."""
    from nanovllm.distributed import parallel_state
    from nanovllm.layers import dense_mlp, latent_attention
    cfg = config(40, 64, 2, [layer(4, 12, 20, 24, 9, 44)])
    t = {k: v.float() for k, v in O.random_tensors(cfg, 3).items()}
    h = torch.randn(21, 40, generator=torch.Generator().manual_seed(1))
    W = O.Weights(t)
    want_mix = O.latent_attention(h.double(), W, "l0.mix.", cfg["layers"][0]["mixer"], 1e-5)
    want_mlp = O.dense_mlp(h.double(), W, "l0.mlp.")
    got_mix = got_mlp = 0.0
    vis = O.window_mask(21, 9)
    for rank in range(2):
        g = types.SimpleNamespace(world_size=2, rank=rank)
        monkeypatch.setattr(latent_attention, "get_tp_group", lambda: g)
        monkeypatch.setattr(dense_mlp, "get_tp_group", lambda: g)
        a = latent_attention.LatentAttention(40, 4, 12, 20, 24, 9, 12 ** -0.5, 1e-5, torch.float32)
        a.load({k[7:]: v for k, v in t.items() if k.startswith("l0.mix.")}, "cpu")
        qc = h @ a.qc_proj.weight.T
        c = O.norm_plain(qc[:, 2 * a.dimp:], a.c_gain, 1e-5)
        out = torch.zeros(21, 2, a.vdimp)
        for i in range(2):
            q = qc[:, i * a.dimp: (i + 1) * a.dimp] @ a.wukt[i].T
            out[:, i] = O.sink_softmax(q @ c.T * a.scale, vis, a.sink[i]) @ c @ a.wuv[i].T
        got_mix = got_mix + out.reshape(21, -1) @ a.o_proj.weight.T
        m = dense_mlp.DenseMLP(40, 44, torch.float32)
        m.load({k[7:]: v for k, v in t.items() if k.startswith("l0.mlp.")}, "cpu")
        _, ca, cb = m.act
        z = h @ m.up.weight.T
        act = torch.where(z > 0, ca * z * z + z / 2, cb * (torch.expm1(z) - z) + z / 2)
        got_mlp = got_mlp + act @ m.down.weight.T
    assert torch.allclose(got_mix.double(), want_mix, atol=1e-5) and torch.allclose(got_mlp.double(), want_mlp, atol=1e-4)
    with pytest.raises(ValueError, match="do not split"):
        monkeypatch.setattr(latent_attention, "get_tp_group", lambda: types.SimpleNamespace(world_size=3, rank=0))
        latent_attention.LatentAttention(40, 4, 12, 20, 24, 9, 0.3, 1e-5, torch.float32)


def test_loader_reports_missing_tensors(tmp_path):
    from nanovllm.models.dafolorn.config import read_config
    from nanovllm.models.dafolorn.model import DafolornForCausalLM
    cfg, t = make_model(tmp_path, "odd")
    del t["l1.mix.uk"]
    O.write_model(str(tmp_path), cfg, t)
    with pytest.raises(KeyError, match="uk"):
        DafolornForCausalLM(read_config(cfg)).load_weights(str(tmp_path))
