"""The Makisun design through the engine's own model, cache manager, step function and scheduler on the host: the
kernel operations are replaced by their plain PyTorch stand-ins (tests/emu_ops.py), the expected values come from the
plain implementation in tests/plain_makisun.py.  A difference here is a fault of the configuration, the parts, the
cache, the state or the batch."""
import copy
import json

import pytest
import torch

import helpers
import makisun_cases as cases
import plain_makisun as plain
from emu_ops import EmuOps

TOL = 2e-5      # float32 storage of activations against float64


@pytest.fixture(autouse=True)
def host_ops():
    from tempura_amd.kernels import ops
    ops.set_backend(EmuOps())
    yield
    ops.set_backend(None)


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("makisun")
    return {name: cases.write_model(name, str(root / name)) for name in cases.CASES}


def _runner(folder, max_tokens, page_size=16, max_requests=4):
    from tempura_amd.engine.loading import load_model
    from tempura_amd.engine.runner import ModelRunner
    model = load_model(folder, "float32", "cpu")
    return ModelRunner(model, page_size, (max_tokens + page_size - 1) // page_size, max_requests=max_requests)


def _plain(name):
    return cases.config_json(name), cases.make_weights(name)


# ---- configuration ------------------------------------------------------------------------------
def test_config_reads_every_size_and_writes_it_back():
    from tempura_amd.config import ConfigError, MakisunConfig
    from tempura_amd.parts.inventory import expected_weights
    for name in cases.CASES:
        d = cases.config_json(name)
        cfg = MakisunConfig.from_dict(d)
        assert MakisunConfig.from_json(cfg.to_json()) == cfg
        assert json.loads(cfg.to_json()) == d
        want = {k: tuple(v.shape) for k, v in cases.make_weights(name).items()}
        got = {k: tuple(v.shape) for k, v in expected_weights(cfg.build_spec()).items()}
        assert set(got) == set(want)
        # (the ranks of the decays' projections are the tensors' own)
        assert all(len(got[k]) == len(want[k]) and all(a in (None, b) for a, b in zip(got[k], want[k])) for k in want)
        free = [k for k in got if None in got[k]]
        assert free and all(k.rsplit(".", 1)[1] in ("w1", "w2", "a1", "a2") for k in free)
        assert cfg.num_parameters() == sum(v.numel() for k, v in cases.make_weights(name).items() if k not in free)
    for change in (lambda c: c["layers"][0].__setitem__("type", "attention"),
                   lambda c: c["layers"][0]["mixer"].pop("heads"),
                   lambda c: c["layers"][1]["mixer"].pop("left"),
                   lambda c: c["layers"][1]["mixer"].pop("right_scale"),
                   lambda c: c["layers"][1]["mixer"]["left"].__setitem__("kv_heads", 3),
                   lambda c: c["layers"][1]["mixer"]["left"].pop("scale"),
                   lambda c: c["layers"][1]["mixer"]["left"]["rot"].__setitem__("dims", 14),      # wider than the head
                   lambda c: c["layers"][1]["mixer"]["left"]["rot"].__setitem__("dims", 5),
                   lambda c: c["layers"][1]["mixer"]["left"]["mask"].__setitem__("size", 0),
                   lambda c: c["layers"][1]["mixer"]["right"].__setitem__("tau", 0),
                   lambda c: c["layers"][1]["mlp"]["router"].__setitem__("top", 7),
                   lambda c: c["layers"][1]["mlp"].__setitem__("kind", "gated"),
                   lambda c: c.__setitem__("layers", [])):
        bad = cases.config_json("mix")
        change(bad)
        with pytest.raises(ConfigError):
            MakisunConfig.from_dict(bad)


def test_sizes_the_configuration_leaves_out():
    """Without `vdim` values are as wide as keys, without `kv_heads` every head has its own, without `rot.dims` the whole
    head turns, without `mask` every earlier key is seen."""
    from tempura_amd.config import MakisunConfig
    d = cases.config_json("one")
    for key in ("vdim", "kv_heads", "mask"):
        del d["layers"][2]["mixer"]["left"][key]
    del d["layers"][2]["mixer"]["right"]["vdim"]
    del d["layers"][0]["mixer"]["left"]["rot"]["dims"]
    cfg = MakisunConfig.from_dict(d)
    a, r = cfg.layers[2].mixer.left, cfg.layers[2].mixer.right
    assert (a.vdim, a.kv_heads, a.window, r.vdim, cfg.layers[0].mixer.left.rot.dims) == (6, 3, None, 3, 20)


def test_registry_chooses_the_design_by_config_json(dirs):
    from tempura_amd.config import MakisunConfig, load_config
    assert isinstance(load_config(dirs["one"]), MakisunConfig)


def test_a_checkpoint_with_a_wrong_tensor_is_refused(dirs, tmp_path):
    from tempura_amd.engine.loading import load_model
    from tempura_amd.weights import WeightsError
    W = cases.make_weights("mix")
    W["l0.mix.u"] = W["l0.mix.u"].reshape(-1)                  # heads x dim, not one row
    del W["l0.mix.mu.w"]
    del W["l1.mlp.shared.down"]
    W["l4.ls2"] = W["l1.ls2"]                                  # that layer has no feed-forward
    cases.write_model("mix", str(tmp_path / "bad"), weights=W)
    with pytest.raises(WeightsError) as e:
        load_model(str(tmp_path / "bad"), "float32", "cpu")
    assert {"l0.mix.mu.w", "l1.mlp.shared.down"} <= set(e.value.missing) and "l0.mix.u" in e.value.wrong_shape
    assert e.value.unexpected == ["l4.ls2"]
    W = cases.make_weights("mix")
    W["l0.mix.w1"] = W["l0.mix.w1"][:3]
    cases.write_model("mix", str(tmp_path / "rank"), weights=W)
    with pytest.raises(ValueError, match="rank"):
        load_model(str(tmp_path / "rank"), "float32", "cpu")


def test_caches_groups_and_states_of_a_model(dirs):
    runner = _runner(dirs["mix"], 64)
    groups = {(g.kind, g.window, g.num_kv_heads, g.head_dim, getattr(g, "value_dim", g.head_dim)) for g in runner.model.cache_groups}
    assert groups == {("window", 9, 2, 12, 10), ("full", None, 1, 8, 14)}
    # a recurrence's state and, behind it, the row before; two mixers side by side keep the recurrence's state only
    assert [runner.pools.state[i].shape[1] for i in range(5)] == [3 * 100 + 48, 3 * 6 * 14, 2 * 256 + 48, 2 * 12 * 5, 4 * 49 + 48]
    from tempura_amd.config import load_config
    assert load_config(dirs["mix"]).state_bytes_per_request() == 4 * sum(runner.pools.state[i].shape[1] for i in range(5))


# ---- mechanisms alone, against the plain functions ----------------------------------------------
@pytest.mark.parametrize("name", ["mix", "one"])
def test_each_part_alone_matches_its_plain_function(dirs, name):
    import makisun_mechanisms
    makisun_mechanisms.check(dirs[name], name, "cpu", TOL)


def test_each_part_alone_in_bfloat16(dirs, tmp_path):
    """The parts as the bfloat16 engine builds them: padded key sizes, the squared ReLU in the experts' up product."""
    import makisun_mechanisms
    cfg = cases.config_json("wide", every_expert=True)
    folder = cases.write_model("wide", str(tmp_path / "wide"), config=cfg)
    makisun_mechanisms.check(folder, "wide", "cpu", 6e-2, dtype="bfloat16", cfg=cfg)
    from tempura_amd.engine.loading import load_model
    model = load_model(folder, "bfloat16", "cpu")
    assert [(g.head_dim, getattr(g, "value_dim", g.head_dim)) for g in model.cache_groups] == [(64, 64), (32, 32), (128, 128)]
    assert model.layers[1].ffn.fused_relu2 and model.layers[1].ffn.shared_relu2 and not model.layers[2].ffn.fused_relu2
    assert model.layers[0].mixer.input_dtype == torch.float32 and model.layers[1].mixer.input_dtype is None


def test_every_mechanism_matters_to_the_logits(monkeypatch):
    """The premise of every comparison of logits here: with any one mechanism left out or done otherwise, the plain
    implementation's own logits change far beyond the bounds."""
    cfg, W = _plain("mix")
    toks = cases.tokens("mix", 40, 4)
    ref = plain.forward(cfg, W, toks)

    def differs(what, weights=W, config=cfg):
        assert plain.logit_error(plain.forward(config, weights, toks), ref) > 0.02, what

    for suffix in (".mu.r", ".mu.k", ".mu.v", ".mu.g", ".mu.w", ".w0", ".w1", ".w2", ".mix.u", ".mix.norm", ".mix.g", ".left.g", ".left.q.norm",
                   ".left.k.norm", ".right.g", ".right.a1", ".right.a2", ".right.a2.b", ".right.norm", ".norm1", ".norm2", ".ls1", ".ls2",
                   ".router.b", ".shared.down"):
        differs(suffix, {k: (v * 0.5 if k.endswith(suffix) else v) for k, v in W.items()})
    for change in (lambda m: m["left"].pop("mask", None), lambda m: m["left"].update(scale=m["left"]["scale"] * 0.7),
                   lambda m: m["left"]["rot"].update(dims=m["left"]["rot"]["dims"] - 2), lambda m: m["left"]["rot"].update(base=20.0),
                   lambda m: m["right"].update(tau=m["right"]["tau"] * 2), lambda m: m.update(left_scale=0.9), lambda m: m.update(right_scale=0.9)):
        c = copy.deepcopy(cfg)
        for layer in c["layers"]:
            if layer["type"] == "parallel":
                change(layer["mixer"])
        differs("constant", config=c)
    c = copy.deepcopy(cfg)
    c["embedding"]["scale"] = 2.0
    differs("embedding scale", config=c)
    wkv_chain, over_rms = plain.wkv_chain, plain.over_rms
    for name, other in (("shifted", lambda u: torch.zeros_like(u)),                                       # no row before
                        ("gelu_erf", torch.relu), ("relu_squared", lambda z: torch.clamp(z, min=0.0)),
                        ("over_rms", lambda x, eps: over_rms(x, 0.05)),
                        ("wkv_chain", lambda r, k, v, w, u: plain.gla_chain(r, k, v, w)),                  # read behind the update, no bonus
                        ("gla_chain", lambda q, k, v, w: wkv_chain(q, k, v, w, torch.ones(k.shape[1:])))):  # read in front of the decay
        with monkeypatch.context() as mp:
            mp.setattr(plain, name, other)
            differs(name)


def test_a_window_counts_the_token_itself():
    m = plain.visible(12, 5)
    assert m[4].nonzero().reshape(-1).tolist() == [0, 1, 2, 3, 4] and m[5].nonzero().reshape(-1).tolist() == [1, 2, 3, 4, 5]


# ---- the model through the step function --------------------------------------------------------
@pytest.mark.parametrize("name", ["mix", "one"])
@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions", "mixed"])
def test_every_cutting_matches_plain(dirs, name, mode):
    cfg, W = _plain(name)
    reqs = cases.requests(name)
    lengths = cases.LENGTHS[name]
    if mode == "mixed":
        max_tokens = sum(sorted(helpers.roundup(n, 64) for n in lengths.values())[-2:]) + 64
        steps = helpers.schedule_mixed(lengths, max_tokens, seed=11)
    else:
        max_tokens = max(helpers.roundup(n, 64) for n in lengths.values())
        steps = {"whole": helpers.schedule_whole, "bulk_tail": lambda l: helpers.schedule_bulk_tail(l, tail=12),
                 "portions": lambda l: helpers.schedule_portions(l, sizes=(7, 2, 16, 3, 2, 5, 2, 9, 2, 17))}[mode](lengths)
    runner = _runner(dirs[name], max_tokens)
    got = helpers.run_schedule(runner, reqs, steps)
    for rid, toks in reqs.items():
        bad = helpers.first_difference(got[rid], plain.forward(cfg, W, toks), TOL)
        assert bad is None, f"{name}/{mode}: request {rid} first differs at position {bad}"
    assert not runner.cache.live_requests()
    assert runner.cache.free_pages() == [p.num_pages for p in runner.cache.pools]


def test_residual_after_every_layer_matches_plain(dirs):
    from tempura_amd.engine.runner import StepEntry
    cfg, W = _plain("mix")
    toks = cases.tokens("mix", 19, 7)
    want = []
    plain.forward(cfg, W, toks, want)
    runner = _runner(dirs["mix"], 64)
    seen = {}
    runner.model.observer = lambda i, h: seen.__setitem__(i, h.double().clone())
    runner.add_request("r")
    runner.step([StepEntry("r", toks, [])])
    assert len(want) == 5
    for i, ref in enumerate(want):
        assert float((seen[i + 1] - ref).abs().max() / ref.abs().max()) < TOL, f"after layer {i}"


def test_slots_and_pages_are_used_again(dirs):
    """Two slots and a pool of six pages for five requests one after the other and side by side: a slot's and a page's last
    owner must leave nothing behind (states, the row before, keys)."""
    from tempura_amd.engine.runner import StepEntry
    cfg, W = _plain("mix")
    runner = _runner(dirs["mix"], 96, max_requests=2)
    reqs = cases.requests("mix")
    order = ["m2", "m1", "m4", "m0", "m5"]
    for k in range(0, len(order), 2):
        pair = order[k: k + 2]
        for rid in pair:
            runner.add_request(rid)
        done = {rid: 0 for rid in pair}
        got = {rid: [] for rid in pair}
        while any(done[r] < len(reqs[r]) for r in pair):
            batch = []
            for rid in pair:
                c = min(5, len(reqs[rid]) - done[rid])
                if c > 0:
                    batch.append(StepEntry(rid, reqs[rid][done[rid]: done[rid] + c], list(range(c))))
                    done[rid] += c
            logits = runner.step(batch)
            row = 0
            for e in batch:
                got[e.rid].append(logits[row: row + len(e.tokens)].clone())
                row += len(e.tokens)
        for rid in pair:
            runner.end_request(rid)
            assert helpers.first_difference(torch.cat(got[rid]), plain.forward(cfg, W, reqs[rid]), TOL) is None, rid


@pytest.mark.parametrize("window", [5, 16, 17, 33])
def test_the_edges_of_the_window(tmp_path, window):
    """Windows shorter than a page, of exactly one page, one more, two pages and one: a prompt in portions that end at and
    beside page and window borders, then decoding across more borders, with queries so large that a softmax rests on one
    or two keys.  The premise is checked first: the plain implementation with a window one longer or one shorter gives
    other logits."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("mix")
    cfg["layers"] = [cfg["layers"][1], cfg["layers"][0]]
    cfg["layers"][0]["mixer"]["left"]["mask"] = {"size": window}
    W = cases.make_weights("mix", sharp=8.0, cfg=cfg)
    folder = cases.write_model("mix", str(tmp_path / "sharp"), weights=W, config=cfg)
    toks = cases.tokens("mix", 90, 5)
    ref = plain.forward(cfg, W, toks)
    for other in (window - 1, window + 1):
        c2 = copy.deepcopy(cfg)
        c2["layers"][0]["mixer"]["left"]["mask"]["size"] = other
        assert plain.logit_error(plain.forward(c2, W, toks), ref) > 0.05, other
    runner = _runner(folder, 128)
    runner.add_request("r")
    rows, at = [], 0
    for c in (16, 1, 14, 2, 7, 10):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]))
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]) for t in toks[at:]]
    assert plain.logit_error(torch.cat(rows), ref) < 1e-4
    # the pages behind the window went back to the pool while the request was live
    assert 8 - runner.cache.free_pages()[0] <= (window + 15) // 16 + 1


def test_a_far_token_decides(tmp_path):
    """Slow decays: what a token 250 positions back has left in the states shows in the logits; sharp queries over an
    attention without a window.  A prompt cut anywhere, then decoding.  The premise first: another token there gives other
    logits at the end, with the attention taken out as well."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("mix")
    cfg["layers"] = [cfg["layers"][0], cfg["layers"][3], cfg["layers"][2]]
    W = cases.make_weights("mix", sharp=8.0, slow=5.0, cfg=cfg)
    folder = cases.write_model("mix", str(tmp_path / "far"), weights=W, config=cfg)
    toks = cases.tokens("mix", 260, 17)
    ref = plain.forward(cfg, W, toks)
    other = [toks[0], (toks[1] + 1) % 90] + toks[2:]
    alone = copy.deepcopy(cfg)
    alone["layers"][1]["mixer"]["left_scale"] = 0.0
    assert plain.logit_error(plain.forward(alone, W, other)[-5:], plain.forward(alone, W, toks)[-5:]) > 0.01
    runner = _runner(folder, 320)
    runner.add_request("r")
    rows, at = [], 0
    for c in (110, 2, 61, 50, 7):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]))
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]) for t in toks[at:]]
    assert plain.logit_error(torch.cat(rows), ref) < 1e-4


def test_first_tokens_and_single_token_requests(dirs):
    """From the very first token on (no row before, an empty state), one token a step, then the same slot and pages for
    another request."""
    from tempura_amd.engine.runner import StepEntry
    for name in ("mix", "one"):
        cfg, W = _plain(name)
        runner = _runner(dirs[name], 64, max_requests=1)
        toks = cases.tokens(name, 6, 9)
        ref = plain.forward(cfg, W, toks)
        runner.add_request("x")
        rows = [runner.step([StepEntry("x", [t], [0])]) for t in toks]
        assert plain.logit_error(torch.cat(rows), ref) < 1e-4, name
        runner.end_request("x")
        runner.add_request("y")
        assert plain.logit_error(runner.step([StepEntry("y", toks[:3], [0, 1, 2])]), ref[:3]) < 1e-4, name


def test_a_request_that_sits_steps_out_keeps_its_state(dirs):
    from tempura_amd.engine.runner import StepEntry
    cfg, W = _plain("mix")
    a, b = cases.tokens("mix", 20, 31), cases.tokens("mix", 24, 32)
    runner = _runner(dirs["mix"], 128)
    runner.add_request("a")
    rows = [runner.step([StepEntry("a", a[:9], list(range(9)))])]
    runner.add_request("b")
    for i in range(0, 24, 6):
        runner.step([StepEntry("b", b[i: i + 6], [])])
    rows.append(runner.step([StepEntry("a", a[9:], list(range(11)))]))
    assert plain.logit_error(torch.cat(rows), plain.forward(cfg, W, a)) < 1e-4


def test_long_decoding(dirs):
    """A short prompt, then 120 tokens one by one."""
    from tempura_amd.engine.runner import StepEntry
    cfg, W = _plain("mix")
    toks = cases.tokens("mix", 125, 13)
    ref = plain.forward(cfg, W, toks)
    runner = _runner(dirs["mix"], 128)
    runner.add_request("r")
    rows = [runner.step([StepEntry("r", toks[:5], list(range(5)))])]
    rows += [runner.step([StepEntry("r", [t], [0])]) for t in toks[5:]]
    assert plain.logit_error(torch.cat(rows), ref) < 1e-4


def test_a_norm_per_head_follows_the_rotation_in_the_plain_attention_part():
    """The ordinary attention part with a norm per head AND a rotation of halves: the norm's weight is ordered like the heads
    whose elements were brought side by side."""
    from tempura_amd.cache import LayerCache
    from tempura_amd.config.spec import PartSpec
    from tempura_amd.parts import build_part
    g = torch.Generator().manual_seed(1)
    H, G, D, width, T = 4, 2, 6, 20, 13
    names = {"q": (H * D, width), "k": (G * D, width), "v": (G * D, width), "o": (width, H * D), "q.norm": (D,), "k.norm": (D,)}
    W = {n: torch.randn(*s, generator=g) for n, s in names.items()}
    part = build_part("mixer", PartSpec("attention", {
        "num_heads": H, "num_kv_heads": G, "head_dim": D, "scale": 0.3, "window": 7, "qk_norm": {"eps": 1e-6},
        "position": PartSpec("rope", {"head_dim": D, "rotary_dim": 4, "theta": 40.0})},
        {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}), width, torch.float32, "cpu")
    part.load_weights(lambda n: W[n])
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32)

    class Ctx:
        positions, token_req, cu_seqlens, context_lens = torch.arange(T, dtype=torch.int32), torch.zeros(T, dtype=torch.int32), i32(0, T), i32(T)
        block_tables, slot_mapping, shared = [i32(0).view(1, 1)], [torch.arange(T, dtype=torch.int32)], {}
        max_q_len, max_context_len, num_single, num_tokens = T, T, 0, T
    x = torch.randn(T, width, generator=g)
    cache = LayerCache(0, {"k": torch.zeros(2, G, 16, D), "v": torch.zeros(2, G, D, 16)}, True, 16, None)
    y = part.forward(x, Ctx, cache, None)
    d = {"p." + k: v.double() for k, v in W.items()}
    d["p.g"] = torch.zeros(H, width, dtype=torch.float64)      # (a gate of one half, undone below)
    c = {"heads": H, "kv_heads": G, "dim": D, "vdim": D, "scale": 0.3, "mask": {"size": 7}, "rot": {"dims": 4, "base": 40.0}}
    ref = 2.0 * plain.left(x.double(), d, "p", c, 1e-6)
    assert float((y.double() - ref).abs().max() / ref.abs().max()) < TOL


# ---- generation through the engine's entry point and scheduler ----------------------------------
@pytest.mark.parametrize("name", ["mix", "one"])
def test_engine_generates_what_plain_greedy_generates(dirs, name):
    from tempura_amd.engine import Engine
    from tempura_amd.sampling import SamplingParams
    cfg, W = _plain(name)
    prompts = [cases.tokens(name, n, 20 + i) for i, n in enumerate((3, 18, 9))]
    eng = Engine(dirs[name], dtype="float32", page_size=16, kv_pages=12, max_batch_size=2, max_num_batched_tokens=16,
                 prefill_chunk_size=7, device="cpu", use_graph=False)
    outs = eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=6))
    for p, o in zip(prompts, outs):
        assert o == plain.greedy(cfg, W, p, 6)


@pytest.mark.parametrize("kind", ["wkv", "parallel"])
def test_models_of_one_mixer_alone(tmp_path, kind):
    """Recurrences alone (a model that has no paged cache) and branches alone, through the scheduler."""
    from tempura_amd.engine import Engine
    from tempura_amd.sampling import SamplingParams
    cfg = cases.config_json("mix")
    cfg["layers"] = [layer for layer in cfg["layers"] if layer["type"] == kind]
    W = cases.make_weights("mix", 3, cfg=cfg)
    eng = Engine(cases.write_model("mix", str(tmp_path / kind), weights=W, config=cfg), dtype="float32", page_size=16, kv_pages=12, max_batch_size=2,
                 max_num_batched_tokens=16, prefill_chunk_size=7, device="cpu", use_graph=False)
    assert (len(eng.runner.model.cache_groups) == 0) == (kind == "wkv")
    prompts = [cases.tokens("mix", n, 40 + i) for i, n in enumerate((19, 2, 8))]
    for p, o in zip(prompts, eng.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=5))):
        assert o == plain.greedy(cfg, W, p, 5)


def test_command_line_inspects_and_writes_random_folders(dirs, tmp_path, capsys):
    """`tempura inspect` on a folder of the design, and `tempura random-model --config-json` for it (which needs the ranks
    that a checkpoint would say)."""
    from tempura_amd.cli import main
    from tempura_amd.engine.loading import load_model
    assert main(["inspect", dirs["mix"]]) == 0
    text = capsys.readouterr().out
    assert "Makisun" in text and "wkv 3 heads of 10; feed-forward 40" in text
    assert "window 9, 8 rotated, gate per head + 1.2 x gated linear attention 3 heads of 6, values of 14, tau 8" in text
    d = cases.config_json("one")
    for layer in d["layers"]:
        (layer["mixer"] if layer["type"] == "wkv" else layer["mixer"]["right"])["decay_rank"] = 4
    path = tmp_path / "c.json"
    path.write_text(json.dumps(d))
    assert main(["random-model", "--config-json", str(path), "--out", str(tmp_path / "rnd"), "--std", "0.3"]) == 0
    model = load_model(str(tmp_path / "rnd"), "float32", "cpu")
    assert model.layers[1].mixer.w2_t.shape == (4, 9) and model.layers[0].mixer.branches[1].a2_t.shape == (4, 7)
    assert torch.equal(model.layers[0].closing["mixer"], torch.ones(32))
