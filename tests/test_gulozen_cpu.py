"""Gulozen without a GPU: configuration and registry, rotation frequencies, the scheduler with attention that sees everything, the step
batch's history, tensor-parallel slices, and the plain evaluation's mechanisms against values worked out by hand."""
import copy
import math
import types

import pytest
import torch

from gulozen_util import CONFIGS, YARN, config, latent, lightning, make_model, moe
from oracle import gulozen_oracle as O
from test_dafolorn_cpu import _drive, _scheduler

D = torch.float64


def t64(x):
    return torch.tensor(x, dtype=D)


# ---- mechanisms of the plain evaluation ------------------------------------------------------------------------------------
def test_norm_in_groups_by_hand():
    got = O.norm_groups(t64([[3.0, 4.0, 0.0, 2.0]]), t64([1.0, 2.0, 3.0, 4.0]), 2, 0.5)
    a, b = math.sqrt(12.5 + 0.5), math.sqrt(2.0 + 0.5)
    assert torch.allclose(got, t64([[3 / a, 8 / a, 0.0, 8 / b]]))
    assert torch.allclose(O.norm_groups(t64([[3.0, 4.0]]), t64([1.0, 1.0]), 1, 0.0), t64([[3.0, 4.0]]) / math.sqrt(12.5))


def test_convolution_by_hand():
    h = t64([[1.0, 10.0], [2.0, 20.0], [3.0, 30.0]])
    w = t64([[0.5, 0.25, 2.0], [1.0, 0.0, -1.0]])      # last tap: the token itself
    assert O.canon(h, w).tolist() == [[3.0, 0.0], [2 + 4 + 0.25, 0.0], [3 + 6 + 0.5 + 0.5, 10.0]]


def test_rotation_by_hand():
    """Neighbouring columns are a pair; columns behind rot.dims stay."""
    x = t64([[1.0, 2.0, 3.0, 4.0, 5.0, 6.0]]).repeat(3, 1)
    got = O.rotate(x, {"base": 100.0, "dims": 4})
    for p in range(3):
        for i, f in enumerate((1.0, 0.1)):
            u, v, a = x[p, 2 * i], x[p, 2 * i + 1], p * f
            assert torch.allclose(got[p, 2 * i: 2 * i + 2], torch.stack([u * math.cos(a) - v * math.sin(a), v * math.cos(a) + u * math.sin(a)]))
        assert got[p, 4:].tolist() == [5.0, 6.0]


def test_yarn_by_hand():
    """Eight pairs over an original length of 128: fast pairs keep their frequency, slow ones are four times slower, a ramp between."""
    scaling = {"factor": 4.0, "original": 128, "fast": 8.0, "slow": 1.0}
    at = lambda t: 16 * math.log(128 / (2 * math.pi * t)) / (2 * math.log(100.0))  # noqa: E731
    lo, hi = math.floor(at(8.0)), math.ceil(at(1.0))
    assert (lo, hi) == (1, 6)
    from nanovllm.layers.rotary_embedding import PairRotary, yarn_frequencies
    f, m = O.yarn_frequencies(100.0, 16, scaling)
    for i in range(8):
        base, r = 100.0 ** (-i / 8), min(max((i - lo) / (hi - lo), 0), 1)
        assert abs(f[i] - (base / 4 * r + base * (1 - r))) < 1e-15
    assert abs(m - (0.1 * math.log(4.0) + 1)) < 1e-15 and f[1] == 100.0 ** (-1 / 8) and abs(f[7] - 100.0 ** (-7 / 8) / 4) < 1e-15
    # the product's own, over many settings (a range that is empty, clipped below and above)
    for base in (50.0, 1e4, 1e6):
        for dims in (2, 6, 64, 128):
            for s in (scaling, dict(scaling, fast=1.0, slow=1.0), dict(scaling, fast=1e4, slow=1e-4), YARN, dict(scaling, factor=1.0)):
                want, mw = O.yarn_frequencies(base, dims, s)
                got = yarn_frequencies(base, dims, s["factor"], s["original"], s["fast"], s["slow"])
                assert all(abs(a - b) < 1e-12 * b for a, b in zip(got, want)) and len(got) == dims // 2
                r = PairRotary(dims + 2, dims, base, s)
                assert r.mscale == mw and r.pairs == (dims + 2 + 7) // 8 * 4
    assert PairRotary(8, 4, 100.0).freq == (1.0, 100.0 ** -0.5) and PairRotary(8, 4, 100.0).mscale == 1.0
    for bad in ((8, 10), (8, 3), (7, 4), (8, 0)):
        with pytest.raises(ValueError, match="rotation"):
            PairRotary(*bad, 100.0)


def test_latent_attention_by_hand():
    """One head, latent and query of one dimension, two tokens: weights 1 : e^(score), the sink's mass, the gate."""
    one = torch.ones(1, 1)
    W = O.Weights({"dq": one, "dq.norm": torch.ones(1), "uq": torch.tensor([[2.0], [0.0], [0.0]]), "dkv": torch.tensor([[1.0], [0.0], [0.0]]), "dkv.norm": torch.ones(1) * 3, "uk": one,
                   "uv": one * 5, "sink": torch.tensor([math.log(7.0)]), "g": one * 0.5, "o": one})
    spec = {"heads": 1, "dim": 1, "rot_dim": 2, "vdim": 1, "kv_rank": 1, "rot": {"base": 10.0, "dims": 2}, "scale": 0.25}
    h = t64([[-4.0], [9.0]])
    out = O.latent_attention(h, W, "", spec, 0.0, O.Project())
    # normed latents are -3 and 3, queries -2 and 2
    e = [math.exp(2 * -3 * 0.25), math.exp(2 * 3 * 0.25)]
    assert abs(out[1, 0] - (e[0] * -15 + e[1] * 15) / (sum(e) + 7) / (1 + math.exp(-4.5))) < 1e-6
    first = math.exp(-2 * -3 * 0.25)
    assert abs(out[0, 0] - first * -15 / (first + 7) / (1 + math.exp(2.0))) < 1e-6


def test_lightning_by_hand():
    """One key dimension, three tokens: the decayed sum written out; the norm runs over both heads."""
    sl = lambda z: z / (1 + math.exp(-z))  # noqa: E731
    W = O.Weights({"q": torch.tensor([[1.0], [-1.0]]), "k": torch.tensor([[2.0], [0.5]]), "v": torch.tensor([[1.0], [3.0]]), "g": torch.zeros(2, 1), "norm": torch.tensor([1.0, 2.0]), "o": torch.eye(2)})
    spec = {"heads": 2, "dim": 1, "vdim": 1, "decay": [0.5, 0.0]}
    x = [1.0, -2.0, 3.0]
    got = O.lightning(t64(x)[:, None], W, "", spec, 0.25, O.Project())
    S = [0.0, 0.0]
    for t, h in enumerate(x):
        S = [0.5 * S[0] + sl(2 * h) * sl(h), sl(0.5 * h) * sl(3 * h)]
        o = [S[0] * sl(h), S[1] * sl(-h)]
        r = math.sqrt((o[0] ** 2 + o[1] ** 2) / 2 + 0.25)
        assert torch.allclose(got[t], t64([0.5 * o[0] / r, 0.5 * 2 * o[1] / r]))


def test_experts_by_hand():
    """Scores of the softmax over all experts, the two largest chosen, not renormalised."""
    sl = lambda z: z / (1 + math.exp(-z))  # noqa: E731
    t = {"router": torch.tensor([[1.0], [3.0], [2.0]])}
    for e in range(3):
        t.update({f"e{e}.gate": torch.ones(1, 1) * (e + 1), f"e{e}.up": torch.ones(1, 1) * 2, f"e{e}.down": torch.ones(1, 1) * 10 ** e})
    got = O.moe(t64([[0.5]]), O.Weights(t), "", moe(1, 3, 2), O.Project())
    z = [math.exp(0.5), math.exp(1.5), math.exp(1.0)]
    want = sum(z[e] / sum(z) * sl((e + 1) * 0.5) * 1.0 * 10 ** e for e in (1, 2))
    assert abs(float(got) - want) < 1e-12


def test_average_over_depth_by_hand():
    """With sublayers that give nothing (gains of zero) every layer hands on a multiple of the embedding: the products of the sums."""
    cfg = config(16, 9, 2, 2, [lightning(1, 4, 4, None, [0.5]), lightning(1, 4, 4, moe(4, 3, 1), [0.5])], 2.5)
    t = O.random_tensors(cfg, 1)
    for k in ("l0.norm1", "l1.norm1", "l1.norm2"):
        t[k] = torch.zeros_like(t[k])
    t["l0.dwa"], t["l1.dwa"] = torch.tensor([0.25, 0.5]), torch.tensor([1.0, -2.0, 4.0])
    layers = []
    O.forward(cfg, t, [3, 5], layers_out=layers)
    x0 = t["embed"][[3, 5]].double() * 2.5
    assert torch.allclose(layers[0], 0.75 * x0)
    assert torch.allclose(layers[1], x0 - 2.0 * x0 + 4.0 * 0.75 * x0)    # X_1 is layer 0's result before its average: x0 itself


# ---- configuration and registry -----------------------------------------------------------------------------------------------
def test_registry_and_config(tmp_path):
    from nanovllm.config import Config
    from nanovllm.engine.key_reach import EVERYTHING
    from nanovllm.models.registry import find_model
    assert find_model({"architecture": "Gulozen"}).name == "gulozen" and find_model({"architecture": "Napadra"}).name == "napadra"
    make_model(tmp_path, "odd")
    c = Config(str(tmp_path), dtype="float32", max_model_len=100000, max_num_batched_tokens=64)
    hf = c.hf_config
    assert c.kvcache_block_size == 64 and hf.torch_dtype == torch.float32 and hf.key_reach.windows == (EVERYTHING,)
    assert [s.type for s in hf.layers] == ["latent_attention", "lightning", "latent_attention"] and hf.layers[1].mlp is None
    a, b, e = hf.layers
    assert (a.q_rank, a.kv_rank, a.rot_dim, a.rot_pairs_dim, a.experts, a.top, a.ff) == (44, 36, 6, 4, 5, 2, 20) and a.rot_scaling["factor"] == 3.0 and e.rot_scaling is None
    assert hf.norm_groups == 4 and hf.conv_taps == 3 and hf.embedding_scale == 3.0 and len(b.decay) == 3
    from nanovllm.models.gulozen.config import read_config
    assert read_config(CONFIGS["memory"]).key_reach.windows == ()
    with pytest.raises(ValueError):
        Config(str(tmp_path), dtype="float16")


@pytest.mark.parametrize("edit,match", [
    (lambda c: c["layers"][1].update(type="mystery"), "mystery"), (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "sparse"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(sections=[1, 2]), "sections"), (lambda c: c["layers"][1]["mixer"].update(decay=[0.5]), "1 decays for 3 heads"),
    (lambda c: c["layers"][2]["mlp"]["router"].update(top=4), "4 of 3 experts"), (lambda c: c["norm"].update(groups=5), "in 5 groups"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=0), "positive")])
def test_what_the_design_does_not_have_is_refused(edit, match):
    from nanovllm.models.gulozen.config import read_config
    c = copy.deepcopy(CONFIGS["odd"])
    edit(c)
    with pytest.raises((NotImplementedError, ValueError), match=match):
        read_config(c)


def test_loader_reports_missing_tensors(tmp_path):
    from nanovllm.models.gulozen.config import read_config
    from nanovllm.models.gulozen.model import GulozenForCausalLM
    cfg, t = make_model(tmp_path, "odd")
    for name in ("l0.mix.dq.norm", "l1.mix.norm", "l2.dwa", "l0.mlp.e3.up"):
        O.write_model(str(tmp_path / name), cfg, {k: v for k, v in t.items() if k != name})
        with pytest.raises(KeyError, match=name.split(".")[-1]):
            GulozenForCausalLM(read_config(cfg)).load_weights(str(tmp_path / name))


# ---- scheduler and step tables --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("preempts", [False, True])
def test_scheduler_keeps_every_block(preempts):
    """Attention that sees everything: no block of a live sequence is given back, all of a finished one are."""
    from nanovllm.engine.key_reach import EVERYTHING, KeyReach
    from nanovllm.engine.sequence import Sequence
    from nanovllm.sampling_params import SamplingParams
    blocks = 13 if preempts else 20
    sch = _scheduler(num_kvcache_blocks=blocks, max_num_batched_tokens=48, hf_config=types.SimpleNamespace(key_reach=KeyReach(windows=(EVERYTHING,))))
    seqs = [Sequence(list(range(i * 1000, i * 1000 + n)), SamplingParams(temperature=0.0, max_tokens=60, ignore_eos=True)) for i, n in enumerate((120, 120, 120))]
    for s in seqs:
        sch.add(s)
    preempted, real = [], sch.preempt
    sch.preempt = lambda s: (preempted.append(s.seq_id), real(s))

    def check(batch):
        for _, c in batch:
            assert all(b >= 0 for b in c.block_table)

    done = _drive(sch, seqs, check, window=EVERYTHING)
    assert len(done) == 3 and all(s.num_completion_tokens == 60 for s in seqs) and bool(preempted) is preempts
    assert len(sch.block_manager.free_block_ids) == blocks


def test_history_of_long_portions():
    """A long portion's key rows: the whole history in front of its own tokens, gathered from its pages."""
    from nanovllm.engine.key_reach import EVERYTHING
    from nanovllm.engine.step_batch import Chunk, build_step
    spec = types.SimpleNamespace(windows=[EVERYTHING], tile_sizes=[2], max_short_portion=16)
    chunks = [Chunk([1] * 20, 150, [7, 3, 9], 0, 1, []), Chunk([2], 70, [5, 6], 2, 3, []), Chunk([3] * 100, 0, [1, 2], 4, 5, [])]
    host, on_device, first = build_step(chunks, spec, 64)
    b = on_device(torch.from_numpy(host))
    w = b.windows[EVERYTHING]
    assert first == [1, 21, 0] or first == [1, 0, 21]
    assert w.rows == 170 + 100 and w.k_start.tolist() == [0, 170, 270] and b.Ta == 1
    assert w.hist_rows.tolist() == list(range(150))
    assert w.hist_slots.tolist() == [[7, 3, 9][p // 64] * 64 + p % 64 for p in range(150)]
    assert w.crow.tolist() == [-1] + list(range(150, 170)) + list(range(170, 270))


# ---- tensor parallelism -----------------------------------------------------------------------------------------------------------
def test_tensor_parallel_slices_add_up(monkeypatch):
    """Two ranks' heads and expert columns, evaluated in plain arithmetic over the loaded (padded, sliced) weights: the sum over the ranks is
    the whole model's sublayer; the linear attention is whole on every rank."""
    from nanovllm.engine.key_reach import EVERYTHING
    from nanovllm.layers import expert_mlp, latent_attention
    from nanovllm.layers.linear_attention import LinearAttention
    from nanovllm.layers.rotary_embedding import PairRotary
    cfg = config(40, 64, 2, 2, [latent(4, 12, 6, 20, 28, 24, moe(44, 5, 2), dims=4, scaling=YARN), lightning(4, 12, 20)])
    t = {k: v.float() for k, v in O.random_tensors(cfg, 3).items()}
    h = torch.randn(21, 40, generator=torch.Generator().manual_seed(1))
    W, hd, spec = O.Weights(t), h.double(), cfg["layers"][0]["mixer"]
    part = lambda p: {k[len(p):]: v for k, v in t.items() if k.startswith(p)}  # noqa: E731
    want = [O.latent_attention(hd, W, "l0.mix.", spec, 1e-5, O.Project()), O.moe(hd, W, "l0.mlp.", cfg["layers"][0]["mlp"], O.Project())]
    got = [0.0, 0.0]
    visible = torch.tril(torch.ones(21, 21, dtype=torch.bool))
    for rank in range(2):
        g = types.SimpleNamespace(world_size=2, rank=rank)
        for mod in (latent_attention, expert_mlp):
            monkeypatch.setattr(mod, "get_tp_group", lambda: g)
        rot = PairRotary(6, 4, 10000.0, YARN)
        a = latent_attention.LatentAttention(40, 4, 12, 20, 24, EVERYTHING, spec["scale"], 1e-5, torch.float32, q_rank=28, rot_dim=6, rot=rot, gated=True)
        a.load(part("l0.mix."), "cpu")
        x = (h @ a.qc_proj.weight.T).double()
        assert a.heads == 2 and a.g_off == 32 + 24 + 8 and x.shape[1] == a.g_off + 2 * 24
        cq = x[:, :32] / torch.sqrt((x[:, :32] ** 2).sum(-1, keepdim=True) / 28 + 1e-5) * a.cq_gain
        q = (cq.float() @ a.uq_proj.weight.T).double().view(21, 2, 24)
        c = O.norm_plain(x[:, 32:56], a.c_gain[:24].double(), 1e-5)
        rr = dict(spec["rot"])
        kr, qr = O.rotate(x[:, 56:64], rr), O.rotate(q[..., 16:], rr)
        out = torch.zeros(21, 2, 24, dtype=D)
        for i in range(2):
            s = (q[:, i, :16] @ a.wukt[i].double().T @ c.T + qr[:, i] @ kr.T) * a.scale
            out[:, i] = O.sink_softmax(s, visible, a.sink[i].double()) @ c @ a.wuv[i].double().T
        got[0] = got[0] + (out.reshape(21, -1) * torch.sigmoid(x[:, a.g_off:])).float() @ a.o_proj.weight.T
        m = expert_mlp.ExpertMLP(40, 44, 5, 2, torch.float32)
        m.load(part("l0.mlp."), "cpu")
        s = torch.softmax(h @ m.router.weight[:5].T, -1)
        w, idx = s.topk(2, -1)
        y = torch.zeros(21, 40)
        for r in range(21):
            for j in range(2):
                z = m.w13[idx[r, j]] @ h[r]
                y[r] += w[r, j] * (m.w2[idx[r, j]] @ (O.silu(z[:24]) * z[24:]))
        got[1] = got[1] + y
        e = LinearAttention(40, 4, 12, 20, cfg["layers"][1]["mixer"]["decay"], 1e-5, torch.float32)
        e.load(part("l1.mix."), "cpu")
        assert e.heads == 4 and torch.equal(e.decay, torch.tensor(cfg["layers"][1]["mixer"]["decay"]))
    for a, b in zip(got, want):
        assert torch.allclose(a.double(), b, atol=2e-5, rtol=1e-4)
    for mod, args in ((latent_attention, lambda: latent_attention.LatentAttention(40, 4, 12, 20, 24, 9, 0.3, 1e-5, torch.float32)), (expert_mlp, lambda: expert_mlp.ExpertMLP(40, 44, 5, 2, torch.float32))):
        monkeypatch.setattr(mod, "get_tp_group", lambda: types.SimpleNamespace(world_size=8, rank=0))
        with pytest.raises(ValueError, match="do not split"):
            args()


def test_powers_of_the_decays():
    from nanovllm.layers.linear_attention import LinearAttention
    m = LinearAttention(16, 3, 8, 8, [0.0, 1.0, 0.9], 1e-5, torch.bfloat16)
    assert m.powers.shape == (3, 65) and m.powers[0].tolist() == [1.0] + [0.0] * 64 and m.powers[1].tolist() == [1.0] * 65
    assert all(abs(m.powers[2, j] - 0.9 ** j) < 1e-7 for j in range(65))
    with pytest.raises(ValueError, match="2 decays for 3 heads"):
        LinearAttention(16, 3, 8, 8, [0.5, 0.5], 1e-5, torch.float32)
