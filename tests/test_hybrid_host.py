"""Hybrid decoder host logic on the CPU: configuration and layer order, weight names, rotary tables,
portion plans, the portion scheduler over a fake runner, and the runner's portion inputs."""

import json

import numpy as np
import pytest
import torch

from hybrid_cases import (CONFIGS, NORMED, PARALLEL, SANDWICH, attend, config, delta, diff_attention, general, latent, low_rank,
                          make_normed_weights, make_parallel_weights, make_sandwich_weights, make_weights, normed_config,
                          parallel_config, rglru, routed, sandwich_config, side, ssd)
from oracle import hybrid_ref as ref
from skyrl_amd.inference_engines import mixers
from skyrl_amd.inference_engines.engine import BLOCK_SIZE, EngineCore, ModelRunner, RequestParams
from skyrl_amd.inference_engines.hybrid import HybridCache, HybridDecoder, HybridSpec
from skyrl_amd.inference_engines.registry import build_decoder, decoder_factory, load_decoder
from test_engine_host import V, FakeRunner, next_token, reference_output, run_all


def test_layer_order_with_and_without_loops():
    order = lambda cfg: [(r.layer, r.step) for r in HybridSpec.from_config(cfg).runs]  # noqa: E731
    for cfg in CONFIGS.values():
        assert order(cfg) == ref.layer_runs(cfg)
    assert order(CONFIGS["odd"]) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    with pytest.raises(ValueError):
        HybridSpec.from_config(config([delta()], loop=(0, 2, 1)))
    with pytest.raises(ValueError):
        HybridSpec.from_config(config([dict(delta(), type="unknown")]))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_weight_names_round_trip(dtype):
    for name, cfg in CONFIGS.items():
        m = HybridDecoder(cfg, "cpu", dtype=dtype, seed=None, max_model_len=64)
        w = make_weights(cfg)
        assert m.load_weights(w.items()) == len(w)
        ours = dict(m.hf_named_tensors())
        assert sorted(ours) == sorted(w)
        for k in w:
            assert torch.equal(ours[k].float(), w[k].float()), (name, k)
        assert m.num_params() == sum(t.numel() for t in w.values())
        for L in m.layers:  # derived tensors follow the weights
            if isinstance(L["mixer"], mixers.LatentAttention):
                x = L["mixer"]
                assert torch.equal(x.wuv_t, x.wuv.view(x.heads, x.vdim, x.rank).transpose(1, 2))
        with pytest.raises(KeyError):
            m.load_weights([("l9.norm1", w["final.norm"])])
        with pytest.raises(ValueError):
            m.load_weights([("final.norm", torch.zeros(3))])


def test_checkpoint_folder_and_registry(tmp_path):
    from safetensors.torch import save_file

    cfg, w = CONFIGS["odd"], make_weights(CONFIGS["odd"], 3)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    m = load_decoder(str(tmp_path), "cpu", max_model_len=64)
    assert isinstance(m, HybridDecoder) and torch.equal(dict(m.hf_named_tensors())["l1.mix.uv"], w["l1.mix.uv"])
    assert not m.prefix_cacheable and build_decoder(config([latent()]), "cpu", max_model_len=8).prefix_cacheable
    del w["l0.mix.norm"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l0.mix.norm"):
        load_decoder(str(tmp_path), "cpu", max_model_len=64)
    for bad in ({"architecture": "Nothing"}, {"model_type": "nothing"}, {}):
        with pytest.raises(ValueError):
            decoder_factory(bad)


@pytest.mark.parametrize("rot", [
    {"base": 10000.0, "dims": 8}, {"base": 500.0, "dims": 12, "scaling": {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 0.5}},
    {"base": 1e6, "dims": 64, "scaling": {"factor": 40.0, "original": 4096, "fast": 32.0, "slow": 1.0}},
    {"base": 20.0, "dims": 4, "scaling": {"factor": 2.0, "original": 7, "fast": 1.0, "slow": 1.0}},  # lo == hi
    {"base": 10.0, "dims": 2, "scaling": {"factor": 1.0, "original": 9, "fast": 3.0, "slow": 2.0}}])
def test_rotary_table(rot):
    n = 200
    t = mixers.rotary_table(rot, n).double()
    x = torch.randn(n, rot["dims"], generator=torch.Generator().manual_seed(0), dtype=torch.float64)
    y = ref.rotate_pairs(x, torch.arange(n), rot)
    c, s = t[:, :rot["dims"] // 2], t[:, rot["dims"] // 2:]
    u, v = x[:, 0::2], x[:, 1::2]
    torch.testing.assert_close(torch.stack([u * c - v * s, v * c + u * s], -1).reshape(n, -1), y, atol=1e-5, rtol=1e-5)


def test_sizes_outside_the_design_are_refused():
    for bad in (dict(rot_dim=7), dict(rot_dim=12)):
        e = latent(**bad)
        e["mixer"]["rot"]["dims"] = 7 if bad["rot_dim"] == 7 else 10
        with pytest.raises(ValueError):
            HybridDecoder(config([e]), "cpu", seed=None, max_model_len=8)
    with pytest.raises(ValueError):
        HybridDecoder(config([delta(heads=3, kv_heads=2)]), "cpu", seed=None, max_model_len=8)
    with pytest.raises(ValueError):
        HybridDecoder(config([delta()]), "cpu", dtype=torch.float16)


@pytest.mark.parametrize("window", [1, 16, 37, 100, None])
def test_prompt_plan_covers_every_visible_key(window):
    lens, starts = [1, 3, 40, 200, 129], [9, 0, 5, 0, 333]
    seg, tiles, rows, longest = mixers.prompt_plan(lens, starts, 2, 4, window)
    assert len(seg) == 3 and longest == seg[:, 2].max() and rows % 64 == 0
    tok, used = 4, 0
    for (row, lo, n, r0), i in zip(seg, range(2, 5)):
        first = max(0, starts[i] - window + 1) if window else 0
        assert row == i and lo % BLOCK_SIZE == 0 and first - BLOCK_SIZE < lo <= first
        assert lo + n == starts[i] + lens[i] and r0 == used and r0 % 64 == 0
        used += (n + 63) // 64 * 64
        mine = [t for t in tiles if t[3] == r0 and t[4] == lo]
        covered = []
        for t in mine:
            assert 0 < t[1] <= mixers.PREFILL_TILE and t[2] - starts[i] == t[0] - tok
            covered += range(t[0], t[0] + t[1])
        assert covered == list(range(tok, tok + lens[i]))
        tok += lens[i]
    assert used == rows
    chunk, ends = mixers.chunk_plan(lens, 2, 4)
    assert ends.tolist() == [0, 1, 5, 8] and chunk[:, 1].tolist() == [40, 64, 64, 64, 8, 64, 64, 1]
    assert chunk[:, 2].tolist() == [2, 3, 3, 3, 3, 4, 4, 4] and chunk[1, 0] == 44


class PortionRunner(FakeRunner):
    """Checks that every request's tokens are run once, in order, and answers from its whole history."""

    def __init__(self, num_blocks, budget):
        super().__init__(num_blocks)
        self.budget, self.seen = budget, {}

    def execute(self, batch):
        self.batches.append((batch.kind, len(batch.requests)))
        rows = [r.row for r in batch.requests]
        assert len(set(rows)) == len(rows) and min(rows) >= 0
        decodes = sum(c == 1 for c in batch.counts)
        assert sum(batch.counts) <= max(self.budget, decodes)
        owners = {}
        out = []
        for r, c, sup in zip(batch.requests, batch.counts, batch.suppress):
            assert c >= 1 and r.num_computed + c <= r.num_tokens <= len(r.blocks) * BLOCK_SIZE
            for b in r.blocks:
                assert owners.setdefault(b, r.rid) == r.rid
            hist = self.seen.setdefault(r.rid, [])
            del hist[r.num_computed:]  # a preempted request starts over
            assert len(hist) == r.num_computed
            hist += r.tokens(r.num_computed, r.num_computed + c)
            if r.num_computed + c == r.num_tokens:
                out.append(next_token(hist, sup))
        if batch.kind == "decode":
            assert len(out) == len(batch.requests)
        return np.array(out, dtype=np.int64), np.zeros(len(out), dtype=np.float32)


@pytest.mark.parametrize("num_blocks,budget", [(400, 64), (400, 5), (12, 16), (12, 1)])
def test_portion_scheduler_outputs_independent_of_budget_and_pressure(num_blocks, budget):
    rng = np.random.default_rng(1)
    runner = PortionRunner(num_blocks, budget)
    core = EngineCore(runner, num_blocks, max_num_seqs=6, max_model_len=200, max_prefill_tokens=budget, eos_token_id=3,
                      portions=True)
    reqs, expect = [], []
    for _ in range(12):
        prompt = rng.integers(0, V, size=int(rng.integers(1, 40))).tolist()
        params = RequestParams(max_tokens=int(rng.integers(1, 40)), min_tokens=int(rng.integers(0, 3)), stop_token_ids=(5,))
        reqs.append(core.add_request(prompt, params))
        expect.append(reference_output(prompt, params, eos=3))
    run_all(core)
    for r, (toks, reason) in zip(reqs, expect):
        assert r.out_tokens == toks and r.finish_reason == reason
    assert core.allocator.num_free == num_blocks and len(core._free_rows) == 6
    kinds = {k for k, _ in runner.batches}
    assert kinds == {"portions", "decode"}
    if (num_blocks, budget) == (12, 16):
        assert core.num_preemptions > 0


def test_decodes_are_not_held_up_by_a_long_prompt():
    runner = PortionRunner(100, 16)
    core = EngineCore(runner, 100, max_num_seqs=4, max_model_len=800, max_prefill_tokens=16, portions=True)
    a = core.add_request([1, 2], RequestParams(max_tokens=50))
    core.step()
    core.add_request(list(range(90)), RequestParams(max_tokens=5))
    before = len(a.out_tokens)
    for _ in range(4):
        core.step()
    assert len(a.out_tokens) == before + 4


def test_run_portions_admission_and_limits():
    class LogitRunner:
        def portion_logits(self, batch, want):
            self.last = (batch.kind, list(batch.counts), list(want))
            return "logits" if want else None

    r = LogitRunner()
    core = EngineCore(r, 4, max_num_seqs=2, max_model_len=64, portions=True)
    a, b = core.open_request(), core.open_request()
    with pytest.raises(RuntimeError, match="row"):
        core.open_request()
    assert core.run_portions([(a, [1] * 16, [3]), (b, [2], [])]) == "logits"
    assert r.last == ("portions", [16, 1], [(0, 3)]) and len(a.blocks) == 1 and len(b.blocks) == 1
    assert core.run_portions([(a, [5], [])]) is None and r.last[0] == "decode" and len(a.blocks) == 2
    core.run_portions([(b, [1, 2], [1])])
    assert r.last == ("portions", [2], [(0, 1)]) and b.num_computed == 3
    with pytest.raises(RuntimeError, match="blocks"):
        core.run_portions([(b, [1] * 40, [])])
    core.close_request(a)
    c = core.open_request()
    assert c.row == 0 and core.allocator.num_free == 3
    with pytest.raises(ValueError):
        core.run_portions([(a, [1], [])])
    with pytest.raises(ValueError):
        core.run_portions([(c, [1] * 65, [])])
    with pytest.raises(ValueError, match="places"):
        core.run_portions([(c, [1] * 5, [5])])


def test_portion_inputs_order_and_contents():
    """Short portions first, slots through the block tables, wanted places mapped to the new order."""
    m = HybridDecoder(CONFIGS["odd"], "cpu", seed=None, max_model_len=256)
    runner = ModelRunner(m, num_blocks=40, max_num_seqs=4)
    runner._h2d = torch.from_numpy
    core = EngineCore(runner, 40, max_num_seqs=4, max_model_len=256, portions=True)
    got = {}
    m.forward_portions = lambda inp, cache: got.setdefault("inp", inp)
    m.logits = lambda hidden: hidden
    m.forward_decode = lambda inp, cache: got.setdefault("dec", inp)
    runner.use_graphs = False
    a, b = core.open_request(), core.open_request()
    core.run_portions([(a, list(range(100, 140)), [0, 39]), (b, [7, 8], [1])])
    inp = got["inp"]
    assert inp.n_short == 1 and inp.short_tokens == 2 and inp.seq_lens == [2, 40] and inp.cu.tolist() == [0, 2, 42]
    assert inp.tokens.tolist() == [7, 8] + list(range(100, 140)) and inp.rows.tolist() == [b.row, a.row]
    assert inp.want.tolist() == [2, 41, 1] and inp.bt_row.tolist() == [0, 0] + [1] * 40
    assert inp.slots[2 + 17].item() == a.blocks[1] * BLOCK_SIZE + 1 and inp.positions[41].item() == 39
    assert inp.block_tables[1, :3].tolist() == a.blocks
    assert set(inp.plan) == {"chunks", 37, 16} and inp.plan[37][0].tolist() == [[1, 0, 40, 0]]
    for bad in ([CONFIGS["odd"]["vocab"]], [-1, 3]):
        b.prompt.extend(bad * 2)
        with pytest.raises(ValueError, match="token ids"):
            runner._portion_inputs(core._batch_of([(b, len(bad) * 2)]), [])
        del b.prompt[2:]
    # a decode step of one request leaves the other's row idle
    core.run_portions([(b, [9], [])])
    dec = got["dec"]
    assert dec.one_token and dec.rows.tolist() == [-1, b.row] and dec.tokens.tolist() == [0, 9]
    assert dec.slots.tolist() == [-1, b.blocks[0] * BLOCK_SIZE + 2]


def test_command_line_arguments():
    from skyrl_amd.inference_engines import __main__ as cli
    from skyrl_amd.inference_engines import trace

    a = cli.parse(["--model", "m", "--prompt-ids", "1,2", "--prompt-ids", "3", "--temperature", "0"])
    assert a.prompt_ids == ["1,2", "3"] and a.temperature == 0 and a.dtype == "bfloat16"
    with pytest.raises(SystemExit):
        trace.main(["--model", "m", "--dtype", "float16", "--out", "o", "--max-tokens", "64"])


# ---------------------------------------------------------------- parallel layers of differential attention
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("name", sorted(PARALLEL))
def test_parallel_weight_names_round_trip(name, dtype):
    cfg = PARALLEL[name]
    m = HybridDecoder(cfg, "cpu", dtype=dtype, seed=None, max_model_len=64)
    w = make_parallel_weights(cfg, 2)
    assert m.load_weights(w.items()) == len(w)
    ours = dict(m.hf_named_tensors())
    assert sorted(ours) == sorted(w) and m.num_params() == sum(t.numel() for t in w.values())
    for k in w:
        assert torch.equal(ours[k].float(), w[k].float()), k
    for i, L in enumerate(m.layers):  # derived tensors follow the weights
        x, p = L["mixer"], f"l{i}.mix."
        names = ["q"] if x.kv_from is not None else ["q", "k", "v"]
        assert torch.equal(x.conv_t, torch.cat([w[p + n + ".conv"] for n in names]).float().t())
        want = ref.differential_lambda({k: v.double() for k, v in w.items()}, p, x.diff)
        assert abs(float(x.lam) - float(want)) < 1e-5 * max(1, abs(float(want)))
        sub = L["subs"][0][1]
        assert len(L["subs"]) == 1 and all(a % 8 == 0 and c % 8 == 0 for a, c in sub.ranges)
        bias = torch.cat([w[p + n + ".b"] for n in names])
        assert torch.equal(sub.b_in[:len(bias)].float(), bias.float())
        assert not bool(sub.b_in[len(bias):len(bias) + x.heads].any())  # the output gate has none
    before, x0 = {k: v.clone() for k, v in ours.items()}, m.layers[0]["mixer"]
    m.load_weights([("l0.mix.lq1", torch.zeros_like(before["l0.mix.lq1"]))])
    assert abs(float(m.layers[0]["mixer"].lam) - float(ref.differential_lambda(
        dict({k: v.double() for k, v in w.items()}, **{"l0.mix.lq1": torch.zeros(1).double()}), "l0.mix.", x0.diff))) < 1e-5
    assert all(torch.equal(before[k], v) for k, v in m.hf_named_tensors() if k != "l0.mix.lq1")


def test_parallel_checkpoint_registry_and_prefixes(tmp_path):
    from safetensors.torch import save_file

    cfg, w = PARALLEL["odd"], make_parallel_weights(PARALLEL["odd"], 3)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    m = load_decoder(str(tmp_path), "cpu", max_model_len=64)
    assert isinstance(m, HybridDecoder) and m.plain_lm_head and m.spec.embed_scale == cfg["embedding"]["scale"]
    assert "l1.mix.k" in dict(m.hf_named_tensors()) and "l2.mix.k" not in dict(m.hf_named_tensors())
    assert not m.prefix_cacheable  # the convolutions' state is not in the pages
    one = parallel_config([diff_attention(conv=1)])
    assert build_decoder(one, "cpu", max_model_len=8).prefix_cacheable
    assert not HybridDecoder(CONFIGS["odd"], "cpu", seed=None, max_model_len=8).plain_lm_head
    del w["l3.mix.q.b"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l3.mix.q.b"):
        load_decoder(str(tmp_path), "cpu", max_model_len=64)


def test_shared_keys_and_values_hold_one_cache():
    m = HybridDecoder(PARALLEL["odd"], "cpu", seed=None, max_model_len=64)
    runs = HybridCache(m, 5, 3).runs
    assert runs[2][0] is runs[1][0] and runs[2][1] is runs[1][1] and runs[3][0] is runs[0][0] and runs[0][0] is not runs[1][0]
    for (k, v, ring), e in zip(runs, PARALLEL["odd"]["layers"]):
        x = e["mixer"]
        dp, vp = -(-x["dim"] // 16) * 16, -(-x["vdim"] // 16) * 16
        assert k.shape == (5, x["kv_heads"], BLOCK_SIZE, 2 * dp) and v.shape == (5, x["kv_heads"], vp, BLOCK_SIZE)
        own = 0 if "kv_from" in x else x["kv_heads"] * (2 * x["dim"] + x["vdim"])
        assert ring.shape == (3, x["conv"], 2 * x["heads"] * x["dim"] + own)
    assert m.block_bytes() == sum(t[0].numel() + t[1].numel() for t in runs[:2]) // 5 * 2
    assert m.row_bytes() == sum(t[2].numel() for t in runs) // 3 * 2


def test_parallel_sizes_outside_the_design_are_refused():
    build = lambda *layers: HybridDecoder(parallel_config(list(layers)), "cpu", seed=None, max_model_len=8)  # noqa: E731
    for bad in (diff_attention(heads=3, kv_heads=2), diff_attention(rot_dims=7), diff_attention(dim=8, rot_dims=10)):
        with pytest.raises(ValueError):
            build(bad)
    good = diff_attention()
    for bad in (diff_attention(kv_from=1), diff_attention(kv_from=-1), diff_attention(kv_from=0, dim=24),
                diff_attention(kv_from=0, vdim=20), diff_attention(kv_from=0, kv_heads=4)):
        with pytest.raises(ValueError, match="kv_from"):
            build(good, bad)
    with pytest.raises(ValueError, match="kv_from"):  # not an owner
        build(good, diff_attention(kv_from=0), diff_attention(kv_from=1))
    with pytest.raises(ValueError, match="parallel"):
        build(delta())


def test_tile_and_run_plans_cover_every_token():
    lens, starts = [1, 3, 40, 200, 129], [9, 0, 5, 0, 333]
    tiles, runs = mixers.tile_plan(lens, starts, 2, 4), mixers.run_plan(lens, starts, 2, 4)
    pos, seq, tok = {}, {}, 4
    for i in range(2, 5):
        for t in range(lens[i]):
            pos[tok], seq[tok] = starts[i] + t, i
            tok += 1
    covered = []
    for t, n, p, row in tiles.tolist():
        assert 0 < n <= mixers.PREFILL_TILE and pos[t] == p and {seq[t + k] for k in range(n)} == {row}
        covered += range(t, t + n)
    assert sorted(covered) == sorted(pos)
    ends = [p + n for _, n, p, _ in tiles.tolist()]
    assert ends == sorted(ends, reverse=True)
    covered = []
    for t, n in runs.tolist():
        assert 0 < n <= 8 and seq[t] == seq[t + n - 1] and pos[t + n - 1] // 8 == pos[t] // 8
        covered += range(t, t + n)
    assert covered == sorted(pos)


def test_parallel_plan_and_smallest_decode_step():
    m = HybridDecoder(PARALLEL["wide"], "cpu", seed=None, max_model_len=64)
    plan = m.plan([1, 40], [3, 0], 1)
    assert set(plan) == {"tiles"} and [len(p) for p in plan["tiles"]] == [1, 5] and m.plan([1, 2], [3, 0], 2) is None
    assert ModelRunner(m, 4, 6).buckets == [2, 4, 6] and ModelRunner(m, 4, 1).buckets == [1]
    assert ModelRunner(HybridDecoder(CONFIGS["once"], "cpu", seed=None, max_model_len=64), 4, 3).buckets == [1, 2, 3]


# ---------------------------------------------------------------- output norms, recurrences, mixers side by side
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("name", sorted(NORMED))
def test_normed_weight_names_round_trip(name, dtype):
    cfg = NORMED[name]
    m = HybridDecoder(cfg, "cpu", dtype=dtype, seed=None, max_model_len=64)
    w = make_normed_weights(cfg, 2)
    assert m.load_weights(w.items()) == len(w)
    ours = dict(m.hf_named_tensors())
    assert sorted(ours) == sorted(w) and m.num_params() == sum(t.numel() for t in w.values())
    for k in w:
        assert ours[k].shape == w[k].shape and torch.equal(ours[k].float(), w[k].float()), k
    for i, L in enumerate(m.layers):  # derived tensors follow the weights
        p, x = f"l{i}.mix.", L["mixer"]
        if isinstance(x, mixers.GatedLinearRecurrence):
            n = x.channels // x.blocks
            assert torch.equal(x.conv.conv_t, w[p + "conv"].float().t())
            for k, g in enumerate(("ra", "ri")):
                assert torch.equal(x.gate_w[:, k, :n, :n].float(), w[p + g].float())
                assert torch.equal(x.gate_b[k], w[p + g + ".b"].float().view(-1))
            assert not bool(x.gate_w[:, :, n:].any()) and not bool(x.gate_w[..., n:].any())
            torch.testing.assert_close(x.rate.double(), -8 * ref.softplus(w[p + "lam"].double()), rtol=1e-6, atol=0)
        else:
            left, right = x.parts
            sub = L["subs"][0][1]
            assert sub.apart and all(a % 8 == 0 for a, _ in sub.ranges) and sub.biased
            bias = torch.cat([w[p + f"left.{n}.b"] for n in "qkv"])
            assert torch.equal(left.b_in[:len(bias)].float(), bias.float()) and not bool(left.b_in[len(bias):].any())
            assert torch.equal(right.conv.conv_t, w[p + "right.conv"].float().t())
    with pytest.raises(KeyError):
        m.load_weights([("l0.mix.none", w["final.norm"])])
    with pytest.raises(ValueError):
        m.load_weights([("final.norm", torch.ones(cfg["width"]))])


def test_normed_checkpoint_registry(tmp_path):
    from safetensors.torch import save_file

    cfg, w = NORMED["odd"], make_normed_weights(NORMED["odd"], 3)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    m = load_decoder(str(tmp_path), "cpu", max_model_len=64)
    assert isinstance(m, HybridDecoder) and m.plain_lm_head and not m.prefix_cacheable and m.min_bucket == 2
    assert m.norm.shape == () and m.spec.embed_scale == cfg["embedding"]["scale"]
    del w["l1.mix.right.D"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l1.mix.right.D"):
        load_decoder(str(tmp_path), "cpu", max_model_len=64)


def test_kernel_libraries_of_a_checkpoint():
    from skyrl_amd.inference_engines.registry import kernel_libraries

    assert kernel_libraries(NORMED["odd"]) == ("layers", "attn", "rglru", "ssd")
    assert kernel_libraries(normed_config([rglru()])) == ("layers", "rglru")
    assert kernel_libraries(PARALLEL["odd"]) == ("layers", "diff") and kernel_libraries(CONFIGS["odd"]) == ("layers", "delta", "latent")
    assert kernel_libraries({"model_type": "qwen2"}) == ()
    with pytest.raises(ValueError, match="unknown layer"):
        kernel_libraries(normed_config([{"type": "none", "mixer": {}}]))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("name", sorted(SANDWICH))
def test_sandwich_weight_names_round_trip(name, dtype):
    cfg = SANDWICH[name]
    m = HybridDecoder(cfg, "cpu", dtype=dtype, seed=None, max_model_len=64)
    w = make_sandwich_weights(cfg, 2)
    assert m.load_weights(w.items()) == len(w)
    ours = dict(m.hf_named_tensors())
    assert sorted(ours) == sorted(w) and m.num_params() == sum(t.numel() for t in w.values())
    for k in w:
        assert ours[k].shape == w[k].shape and torch.equal(ours[k].float(), w[k].float()), k
    for i, L in enumerate(m.layers):
        p, x = f"l{i}.", L["mixer"]
        if isinstance(x, mixers.LatentAttention):  # derived tensors follow the weights
            uv = w[p + "mix.uv"].float().view(x.heads, x.vdim, x.rank)
            assert torch.equal(x.wuv_t.float(), uv.transpose(1, 2)) and x.halves and x.sinks.dtype == torch.float32
        sub = L["subs"][0][1].sub  # the result gate's rows follow the mixer's in one product
        a, b = sub.beside
        assert a % 8 == 0 and torch.equal(sub.w_in[a:b].float(), w[p + "rg1"].float())
    with pytest.raises(KeyError):
        m.load_weights([("l0.mix.none", w["final.norm"])])
    with pytest.raises(ValueError):
        m.load_weights([("final.norm", torch.ones(cfg["width"] + 1))])


def test_sandwich_checkpoint_gives_the_decay_rank(tmp_path):
    """The rank of the decay's projection is no part of a checkpoint's config: a tensor's shape gives it."""
    from safetensors.torch import save_file

    cfg, w = json.loads(json.dumps(SANDWICH["odd"])), make_sandwich_weights(SANDWICH["odd"], 3)
    for e in cfg["layers"]:
        e["mixer"].pop("decay_rank", None)
    with pytest.raises(ValueError, match="decay_rank"):
        HybridDecoder(cfg, "cpu", seed=None, max_model_len=64)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    m = load_decoder(str(tmp_path), "cpu", max_model_len=64)
    assert isinstance(m, HybridDecoder) and m.plain_lm_head and not m.prefix_cacheable and m.min_bucket == 1
    assert [L["mixer"].rank for L in m.layers if isinstance(L["mixer"], mixers.GeneralDelta)] == [5, 6]
    assert m.spec.norm_groups == cfg["norm"]["groups"] and m.spec.residual_mult == cfg["residual_mult"]
    del w["l1.rg1.b"]
    save_file(w, str(tmp_path / "model.safetensors"))
    with pytest.raises(ValueError, match="l1.rg1.b"):
        load_decoder(str(tmp_path), "cpu", max_model_len=64)


def test_shared_latents_hold_one_cache():
    cfg = SANDWICH["padded"]
    m = HybridDecoder(cfg, "cpu", seed=None, max_model_len=64)
    runs = HybridCache(m, 5, 3).runs
    assert runs[2] is runs[0] and runs[4] is runs[0] and runs[0].shape == (5, BLOCK_SIZE, 160)
    assert runs[1].shape == (3, 2, 72, 72) and runs[3].shape == (3, 1, 136, 136) and runs[1].dtype == torch.float32
    assert m.block_bytes() == runs[0].numel() * 2 // 5 and m.row_bytes() == 4 * (2 * 72 * 72 + 136 * 136)
    names = dict(m.hf_named_tensors())
    assert "l0.mix.dkv" in names and "l2.mix.dkv" not in names and "l4.mix.dkv.norm" not in names


def test_sandwich_sizes_outside_the_design_are_refused():
    build = lambda layers, mlps=None, **kw: HybridDecoder(  # noqa: E731
        dict(sandwich_config(layers, mlps or [None] * len(layers)), **kw), "cpu", seed=None, max_model_len=8)
    one = low_rank()
    for bad in (low_rank(kv_from=1), low_rank(kv_from=-1), low_rank(kv_from=0, kv_rank=44), low_rank(kv_from=0, rot_dim=8),
                low_rank(kv_from=0, base=77.0)):
        with pytest.raises(ValueError, match="kv_from"):
            build([one, bad])
    with pytest.raises(ValueError, match="kv_from"):
        build([one, low_rank(kv_from=0), low_rank(kv_from=1)])
    with pytest.raises(ValueError, match="kv_from"):  # a recurrent layer has nothing to share
        build([general(), dict(general(), mixer=dict(general()["mixer"], kv_from=0))])
    build([one, low_rank(heads=7, dim=9, vdim=5, q_rank=8, window=3, scale=0.5, kv_from=0)])  # all its own but the latents
    for bad in (routed(experts=10, groups=(3, 1)), routed(experts=10, groups=(5, 6)), routed(experts=10, top=3, groups=(5, 1)),
                routed(experts=10, top=0), routed(experts=2000)):
        with pytest.raises(ValueError):
            build([one], [bad])
    for layer in (general(dim=300), low_rank(rot_dim=7)):
        with pytest.raises(ValueError):
            build([layer])
    with pytest.raises(ValueError, match="norm.groups"):
        build([one], norm={"eps": 1e-5, "groups": 5})
    with pytest.raises(ValueError, match="looped"):
        build([one], loop={"start": 0, "stop": 1, "times": 2})
    with pytest.raises(ValueError, match="feed-forward"):
        build([one], [{"kind": "dense", "ff": 8}])


def test_sandwich_kernel_libraries_and_plans():
    from skyrl_amd.inference_engines.registry import kernel_libraries

    assert kernel_libraries(SANDWICH["odd"]) == ("layers", "gdelta", "latent", "moe")
    assert kernel_libraries(sandwich_config([general()], [None])) == ("layers", "gdelta")
    m = HybridDecoder(SANDWICH["odd"], "cpu", seed=None, max_model_len=64)
    assert set(m.plan([3, 40], [0, 5], 1)) == {21, None, "chunks"} and m.plan([1, 3], [7, 0], 2) is None


def test_experts_tiles_follow_the_mean_load():
    sh = mixers.lk.moe_shape(64, 32, 64, 8, 8, 4)
    assert [mixers.lk.moe_tile(sh, n) for n in (1, 64, 95, 96, 383, 384, 895, 896, 8192)] == [16, 16, 16, 64, 64, 128, 128, 256, 256]


def test_oracle_grouped_norm_and_routing():
    x, w = torch.randn(3, 12, dtype=torch.float64), torch.randn(12, dtype=torch.float64)
    got = ref.grouped_rms_norm(x, w, 3, 1e-3)
    for g in range(3):
        part = x[:, 4 * g:4 * g + 4]
        torch.testing.assert_close(got[:, 4 * g:4 * g + 4], part / (part.pow(2).mean(-1, keepdim=True) + 1e-3).sqrt() * w[4 * g:4 * g + 4])
    s = torch.tensor([[0.9, 0.1, 0.7, 0.6, 0.2, 0.3]])
    idx, weight = ref.route(s, torch.tensor([0.0, 0.0, 0.0, 0.0, -9.0, -9.0]), 2, 3, 1)
    assert idx.tolist() == [[2, 3]] and weight.tolist() == [[s[0, 2].item(), s[0, 3].item()]]  # 0.7 + 0.6 beats 0.9 + 0.1
    idx, _ = ref.route(s, torch.full((6,), -5.0), 3, 3, 2)
    assert idx.tolist() == [[0, 2, 3]]  # corrected scores below zero: other groups' count as less than any


def test_position_turns():
    m = HybridDecoder(NORMED["odd"], "cpu", seed=None, max_model_len=64)
    W, pos = NORMED["odd"]["width"], torch.tensor([0, 1, 5, 4000])
    a = pos[:, None].double() * m.turns[None] * 2 * torch.pi
    torch.testing.assert_close(torch.stack([a.sin(), a.cos()], -1).view(4, -1)[:, :W], ref.sinusoid(pos, W), rtol=0, atol=1e-9)


def test_normed_caches_and_sizes():
    cfg = NORMED["padded"]
    m = HybridDecoder(cfg, "cpu", seed=None, max_model_len=64)
    runs = HybridCache(m, 5, 3).runs
    S, ring = runs[0]
    assert S.shape == (3, 96) and S.dtype == torch.float32 and ring.shape == (3, 9, 96)
    (k, v), (S, ring) = runs[1]
    assert k.shape == (5, 1, BLOCK_SIZE, 64) and v.shape == (5, 1, 32, BLOCK_SIZE)
    assert S.shape == (3, 6, 40, 72) and S.dtype == torch.float32 and ring.shape == (3, 7, 6 * 72 + 2 * 3 * 40)
    flat = [t for r in (runs[0], *runs[1], *runs[2]) for t in r]
    assert m.row_bytes() == sum(t.numel() * t.itemsize for t in flat if t.shape[0] == 3) // 3
    assert m.block_bytes() == sum(t.numel() * t.itemsize for t in flat if t.shape[0] == 5) // 5


def test_normed_sizes_outside_the_design_are_refused():
    build = lambda *layers, **kw: HybridDecoder(dict(normed_config(list(layers)), **kw), "cpu", seed=None, max_model_len=8)  # noqa: E731
    for bad in (rglru(width=60, blocks=7), side(attend(heads=3, kv_heads=2)), side(right=ssd(heads=3, groups=2)),
                side(right=ssd(norm_groups=7))):
        with pytest.raises(ValueError):
            build(bad)
    with pytest.raises(ValueError, match="looped"):
        build(rglru(), loop={"start": 0, "stop": 1, "times": 2})
    with pytest.raises(ValueError, match="side by side"):
        build(side(), architecture="Lipedra")


@pytest.mark.parametrize("lens,per_run", [([1, 3, 40, 200, 129], 6), ([64] * 3, 64), ([8192], 64), ([5, 1000] + [700] * 5, 32), ([100], 4096)])
def test_walk_plan_covers_every_chunk_once(lens, per_run):
    first = sum(1 for n in lens if n < 32)
    tok = sum(lens[:first])
    chunk, runs, pick, chain = mixers.walk_plan(lens, first, tok, per_run)
    ref_chunk, ends = mixers.chunk_plan(lens, first, tok)
    assert (chunk[:, :3] == ref_chunk[:, :3]).all()
    covered, by_seq = [], {}
    for r, (a, n, seq, kind) in enumerate(runs.tolist()):
        assert n > 0 and {int(c) for c in chunk[a:a + n, 2]} == {seq}
        covered += range(a, a + n)
        assert set(chunk[a:a + n, 3].tolist()) == {r}
        by_seq.setdefault(seq, []).append((r, kind))
    assert covered == list(range(len(chunk)))
    many = {s: rs for s, rs in by_seq.items() if len(rs) > 1}
    assert chain.tolist() == [[rs[0][0], len(rs)] for rs in many.values()]
    assert pick.tolist() == [r for rs in many.values() for r, _ in rs[:-1]]
    for rs in by_seq.values():
        assert [k for _, k in rs] == [(len(rs) > 1) + 2 * (i == len(rs) - 1) for i in range(len(rs))]


def test_normed_plans_and_window_tiles():
    m = HybridDecoder(NORMED["odd"], "cpu", seed=None, max_model_len=64)
    plan = m.plan([1, 2, 40], [3, 0, 7], 2)
    assert set(plan) == {("runs", 3), ("runs", 2), ("tiles", 37), ("tiles", 16), "runs", ("walk", 3), ("walk", 4)}
    chunk, runs, seq_runs = plan[("runs", 3)]  # short portions too
    assert chunk.tolist() == [[0, 1, 0, 0], [1, 2, 1, 1], [3, 40, 2, 2]] and seq_runs.tolist() == [0, 1, 2, 3]
    assert runs.tolist() == [[0, 1, 0, 2], [1, 1, 1, 2], [2, 1, 2, 2]]
    assert plan[("tiles", 16)][0].tolist() == [[3, 40, 7, 2]] and plan[("walk", 3)][1].tolist() == [[0, 1, 2, 2]]
    assert set(m.plan([1, 2], [3, 0], 2)) == {("runs", 3), ("runs", 2)}
    tiles = mixers.tile_plan([300, 200], [0, 1000], 0, 0, 128)
    assert sorted(tiles[:, 0].tolist()) == [0, 128, 256, 300, 428]
    keys = [t[1] + min(t[2], 128) for t in tiles.tolist()]
    assert keys == sorted(keys, reverse=True)
    assert ModelRunner(m, 4, 6).buckets == [2, 4, 6]
