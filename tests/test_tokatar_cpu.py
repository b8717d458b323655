"""The Tokatar design through the engine's own model, cache manager, step function and scheduler on the host: the
kernel operations are replaced by their plain PyTorch stand-ins (tests/emu_ops.py), the expected values come from the
plain implementation in tests/plain_tokatar.py.  A difference here is a fault of the configuration, the parts, the
cache or the batch."""
import copy
import json

import pytest
import torch

import helpers
import plain_tokatar as plain
import tokatar_cases as cases
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
    root = tmp_path_factory.mktemp("tokatar")
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
    from tempura_amd.config import ConfigError, TokatarConfig
    from tempura_amd.parts.inventory import expected_weights
    for name in cases.CASES:
        d = cases.config_json(name)
        cfg = TokatarConfig.from_dict(d)
        assert TokatarConfig.from_json(cfg.to_json()) == cfg
        assert json.loads(cfg.to_json()) == d
        want = {k: tuple(v.shape) for k, v in cases.make_weights(name).items()}
        got = {k: tuple(v.shape) for k, v in expected_weights(cfg.build_spec()).items()}
        assert got == want
        assert cfg.num_parameters() == sum(v.numel() for v in cases.make_weights(name).values())
    for change in (lambda c: c["layers"][0].__setitem__("type", "attention_3"),
                   lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 3),
                   lambda c: c["layers"][0]["mixer"].pop("rot"),
                   lambda c: c["layers"][0]["mixer"].pop("scale"),
                   lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 14),      # wider than the head
                   lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 5),
                   lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("original"),
                   lambda c: c["layers"][0]["mixer"]["mask"].__setitem__("size", 0),
                   lambda c: c["layers"][2]["mixer"].pop("rot_dim"),
                   lambda c: c["layers"][2]["mixer"]["rot"].__setitem__("dims", 2),        # not the rotated part
                   lambda c: c["layers"][0]["mlp"].__setitem__("kind", "moe"),
                   lambda c: c.__setitem__("layers", [])):
        bad = cases.config_json("mix")
        change(bad)
        with pytest.raises(ConfigError):
            TokatarConfig.from_dict(bad)


def test_registry_chooses_the_design_by_config_json(dirs):
    from tempura_amd.config import TokatarConfig, load_config
    assert isinstance(load_config(dirs["one"]), TokatarConfig)


def test_a_checkpoint_with_a_wrong_tensor_is_refused(dirs, tmp_path):
    from tempura_amd.engine.loading import load_model
    from tempura_amd.weights import WeightsError
    W = cases.make_weights("mix")
    W["l0.norm1"] = torch.ones(48, dtype=torch.bfloat16)       # one number, not one per channel
    del W["l1.mix.v.b"]
    del W["l2.ls1"]
    W["l2.ls2"] = W["l1.ls2"]                                  # that layer has no feed-forward
    cases.write_model("mix", str(tmp_path / "bad"), weights=W)
    with pytest.raises(WeightsError) as e:
        load_model(str(tmp_path / "bad"), "float32", "cpu")
    assert {"l1.mix.v.b", "l2.ls1"} <= set(e.value.missing) and "l0.norm1" in e.value.wrong_shape
    assert e.value.unexpected == ["l2.ls2"]


def test_caches_and_groups_of_a_model(dirs):
    runner = _runner(dirs["mix"], 64)
    groups = {(g.kind, g.window, g.num_kv_heads, g.head_dim, getattr(g, "value_dim", g.head_dim)) for g in runner.model.cache_groups}
    # a latent layer holds one key of [rotated | latent] and one latent, whatever its heads
    assert groups == {("chunk", 9, 2, 12, 10), ("chunk", 21, 2, 10, 6), ("full", None, 1, 24, 20), ("full", None, 1, 8, 12),
                      ("full", None, 1, 16, 10), ("full", None, 2, 8, 8)}
    assert not runner.pools.state


def test_frequencies_of_every_kind():
    """The scaled rotation of the first case keeps, blends and divides frequencies; layouts differ in which elements
    turn together."""
    from tempura_amd.parts.rope import paired_order, rotary_inv_freq
    rot = cases.CASES["mix"]["layers"][0]["mixer"]["rot"]
    s = rot["scaling"]
    plainf, base = plain.key_frequencies(rot), plain.frequencies(rot["dims"], rot["base"])
    ratio = (plainf / base).tolist()
    assert ratio[0] == 1.0 and abs(ratio[-1] - 1.0 / s["factor"]) < 1e-12 and any(0.26 < r < 0.99 for r in ratio)
    got = rotary_inv_freq(12, rot["base"], {"rope_type": "llama3", "factor": s["factor"], "low_freq_factor": s["low"],
                                            "high_freq_factor": s["high"], "original_max_position_embeddings": s["original"]}, rot["dims"])
    assert torch.allclose(got, plainf, rtol=1e-14)
    assert paired_order(6, 4, "halves").tolist() == [0, 2, 1, 3, 4, 5] and paired_order(6, 4, "neighbours") is None


def test_turned_values_in_halves_give_what_plain_gives():
    """The attention part also takes values (and keys) whose pairs are halves: against the plain functions."""
    from tempura_amd.config.spec import PartSpec
    from tempura_amd.parts import build_part
    from tempura_amd.cache import LayerCache
    g = torch.Generator().manual_seed(1)
    H, G, D, E, width, T = 4, 2, 6, 10, 20, 13
    names = {"q": (H * D, width), "k": (G * D, width), "v": (G * E, width), "o": (width, H * E), "g": (H * E, width),
             "q.b": (H * D,), "k.b": (G * D,), "v.b": (G * E,), "q.norm": (H * D,), "k.norm": (G * D,)}
    W = {n: torch.randn(*s, generator=g) for n, s in names.items()}
    rope = lambda n: PartSpec("rope", {"head_dim": n, "rotary_dim": n, "theta": 40.0, "layout": "halves"})
    part = build_part("mixer", PartSpec("attention", {
        "num_heads": H, "num_kv_heads": G, "head_dim": D, "value_dim": E, "scale": 0.3, "chunk": 7, "gate": True, "bias": True,
        "qk_norm": {"eps": 1e-6, "over": "projection"}, "position": rope(D), "value_position": rope(E)},
        {"q": "q", "k": "k", "v": "v", "o": "o", "gate": "g", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "q_norm": "q.norm",
         "k_norm": "k.norm"}), width, torch.float32, "cpu")
    part.load_weights(lambda n: W[n])
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32)

    class Ctx:
        positions, token_req, cu_seqlens, context_lens = torch.arange(T, dtype=torch.int32), torch.zeros(T, dtype=torch.int32), i32(0, T), i32(T)
        block_tables, slot_mapping, shared = [i32(0).view(1, 1)], [torch.arange(T, dtype=torch.int32)], {}
        max_q_len, max_context_len, num_single, num_tokens = T, T, 0, T
    x = torch.randn(T, width, generator=g)
    cache = LayerCache(0, {"k": torch.zeros(2, G, 16, D), "v": torch.zeros(2, G, E, 16)}, True, 16, None)
    y = part.forward(x, Ctx, cache, None)
    d = {k: v.double() for k, v in W.items()}
    u = x.double()
    q = plain.over_rms(u @ d["q"].T + d["q.b"], 1e-6) * d["q.norm"]
    k = plain.over_rms(u @ d["k"].T + d["k.b"], 1e-6) * d["k.norm"]
    v = (u @ d["v"].T + d["v.b"]).reshape(T, G, E)
    f, fv = plain.frequencies(D, 40.0), plain.frequencies(E, 40.0)
    o = plain.attend(plain.turn(q.reshape(T, H, D), f, "halves"), plain.turn(k.reshape(T, G, D), f, "halves"), plain.turn(v, fv, "halves"),
                     0.3, plain.visible(T, 7))
    o = plain.turn(o, fv, "halves", -1.0).reshape(T, H * E) * torch.sigmoid(u @ d["g"].T)
    ref = o @ d["o"].T
    assert float((y.double() - ref).abs().max() / ref.abs().max()) < TOL


# ---- mechanisms alone, against the plain functions ----------------------------------------------
@pytest.mark.parametrize("name", ["mix", "one"])
def test_each_part_alone_matches_its_plain_function(dirs, name):
    import tokatar_mechanisms
    tokatar_mechanisms.check(dirs[name], name, "cpu", TOL)


@pytest.mark.parametrize("name", ["wide", "deep"])
def test_each_part_alone_in_bfloat16(dirs, name):
    """The parts as the bfloat16 engine builds them: padded cache sizes, the activation in the product's epilogue, the
    latent's maps as products per head (and folded where that is cheaper)."""
    import tokatar_mechanisms
    tokatar_mechanisms.check(dirs[name], name, "cpu", 6e-2, dtype="bfloat16")


def test_the_latent_maps_are_folded_where_that_is_cheaper(dirs):
    from tempura_amd.engine.loading import load_model
    kinds = lambda name, dtype: [b.mixer.folded for b in load_model(dirs[name], dtype, "cpu").layers if hasattr(b.mixer, "folded")]
    assert kinds("deep", "bfloat16") == [False] * 3 and kinds("deep", "float32") == [True] * 3
    assert kinds("mix", "bfloat16") == [True, True]      # (heads of ten and eight elements: no product per head)
    model = load_model(dirs["deep"], "bfloat16", "cpu")
    assert [(g.head_dim, g.value_dim) for g in model.cache_groups] == [(288, 256), (320, 256), (576, 512)]


def test_every_mechanism_matters_to_the_logits(monkeypatch):
    """The premise of every comparison of logits here: with any one mechanism left out or done otherwise, the plain
    implementation's own logits change far beyond the bounds."""
    cfg, W = _plain("mix")
    toks = cases.tokens("mix", 40, 4)
    ref = plain.forward(cfg, W, toks)
    over_rms, turn, softmax_plus, stretched = plain.over_rms, plain.turn, plain.softmax_plus, plain.stretched

    def differs(what, weights=W, config=cfg):
        assert plain.logit_error(plain.forward(config, weights, toks), ref) > 0.02, what

    for suffix in (".rg1.b", ".rg2.b", ".mix.q.b", ".mix.k.b", ".mix.v.b", ".ls1", ".ls2", ".q.norm", ".k.norm", ".dkv.norm", ".norm1", ".norm1b",
                   ".norm2b", ".mix.g", ".mix.uk"):
        changed = {k: (v * 0.5 if k.endswith(suffix) else v) for k, v in W.items()}
        differs(suffix, changed)
    for key in ("softcap", "mask"):
        c = copy.deepcopy(cfg)
        for layer in c["layers"]:
            layer["mixer"].pop(key, None)
        differs(key, config=c)
    c = copy.deepcopy(cfg)
    c["embedding"]["scale"] = 2.0
    differs("embedding scale", config=c)
    monkeypatch.setattr(plain, "stretched", lambda f, *a: f)
    differs("frequency scaling")
    monkeypatch.setattr(plain, "stretched", stretched)
    monkeypatch.setattr(plain, "softmax_plus", lambda s, m, extra: softmax_plus(s, m, 0.0))
    differs("one in the denominator")
    monkeypatch.setattr(plain, "softmax_plus", softmax_plus)
    monkeypatch.setattr(plain, "turn", lambda x, f, layout, sign=1.0: x if sign < 0 else turn(x, f, layout, sign))
    differs("outputs turned back")
    monkeypatch.setattr(plain, "turn", lambda x, f, layout, sign=1.0: turn(x, f, "halves", sign))
    differs("pairs of neighbours")
    monkeypatch.setattr(plain, "turn", turn)
    # a norm per head instead of over the whole projection
    monkeypatch.setattr(plain, "over_rms", lambda x, eps: over_rms(x.reshape(x.shape[0], -1, 10), eps).reshape(x.shape)
                        if x.shape[-1] in (40, 20) and x.dim() == 2 else over_rms(x, eps))
    differs("norm over the whole projection")


def test_a_chunk_starts_at_position_zero_of_the_request():
    m = plain.visible(12, 5)
    assert m[4].nonzero().reshape(-1).tolist() == [0, 1, 2, 3, 4] and m[5].nonzero().reshape(-1).tolist() == [5]
    assert m[11].nonzero().reshape(-1).tolist() == [10, 11]


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
    assert len(want) == 6
    for i, ref in enumerate(want):
        assert float((seen[i + 1] - ref).abs().max() / ref.abs().max()) < TOL, f"after layer {i}"


def test_slots_and_pages_are_used_again(dirs):
    """Two slots and a pool of six pages for five requests one after the other and side by side: a page's last owner must
    leave nothing behind (keys, values turned by another position, latents)."""
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


@pytest.mark.parametrize("chunk", [5, 16, 17, 33, 20])
@pytest.mark.parametrize("layer", [0, 1])
def test_the_edges_of_the_chunks(tmp_path, chunk, layer):
    """Chunks shorter than a page, of exactly one page, one more, two pages and one: a prompt in portions that end at and
    beside page and chunk borders, then decoding across more borders, with queries so large that a softmax rests on one
    or two keys of its chunk.  The premise is checked first: the plain implementation with a chunk one longer or one
    shorter, or with a window of the same length, gives other logits."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("mix")
    cfg["layers"] = cfg["layers"][layer: layer + 1] + cfg["layers"][2:3]
    cfg["layers"][0]["mixer"].update({"mask": {"size": chunk}})
    if layer == 0:
        cfg["layers"][0]["mixer"]["softcap"] = 25.0
    W = cases.make_weights("mix", sharp=8.0, cfg=cfg)
    folder = cases.write_model("mix", str(tmp_path / "sharp"), weights=W, config=cfg)
    toks = cases.tokens("mix", 90, 5)
    ref = plain.forward(cfg, W, toks)
    for other in (chunk - 1, chunk + 1):
        c2 = copy.deepcopy(cfg)
        c2["layers"][0]["mixer"]["mask"]["size"] = other
        assert plain.logit_error(plain.forward(c2, W, toks), ref) > 0.05, other
    runner = _runner(folder, 128)
    runner.add_request("r")
    rows, at = [], 0
    for c in (16, 1, 14, 2, 7, 10):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]))
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]) for t in toks[at:]]
    assert plain.logit_error(torch.cat(rows), ref) < 1e-4
    # the pages of finished chunks went back to the pool while the request was live
    g = [i for i, s in enumerate(runner.model.cache_groups) if s.kind == "chunk"][0]
    assert 8 - runner.cache.free_pages()[g] <= (chunk + 15) // 16 + 1


def test_a_far_key_decides(tmp_path):
    """Sharp queries over the cached latents and over an attention without chunks, hundreds of tokens back, in prompts cut
    anywhere and in decoding."""
    from tempura_amd.engine.runner import StepEntry
    cfg = cases.config_json("mix")
    cfg["layers"] = cfg["layers"][2:4]
    W = cases.make_weights("mix", sharp=8.0, cfg=cfg)
    folder = cases.write_model("mix", str(tmp_path / "far"), weights=W, config=cfg)
    toks = cases.tokens("mix", 260, 17)
    ref = plain.forward(cfg, W, toks)
    runner = _runner(folder, 320)
    runner.add_request("r")
    rows, at = [], 0
    for c in (110, 2, 61, 50, 7):
        rows.append(runner.step([StepEntry("r", toks[at: at + c], list(range(c)))]))
        at += c
    rows += [runner.step([StepEntry("r", [t], [0])]) for t in toks[at:]]
    assert plain.logit_error(torch.cat(rows), ref) < 1e-4


def test_first_tokens_and_single_token_requests(dirs):
    """From the very first token on, one token a step, then the same pages for another request."""
    from tempura_amd.engine.runner import StepEntry
    for name in ("mix", "one"):
        cfg, W = _plain(name)
        runner = _runner(dirs[name], 64)
        toks = cases.tokens(name, 6, 9)
        ref = plain.forward(cfg, W, toks)
        runner.add_request("x")
        rows = [runner.step([StepEntry("x", [t], [0])]) for t in toks]
        assert plain.logit_error(torch.cat(rows), ref) < 1e-4, name
        runner.end_request("x")
        runner.add_request("y")
        assert plain.logit_error(runner.step([StepEntry("y", toks[:3], [0, 1, 2])]), ref[:3]) < 1e-4, name


def test_long_decoding_passes_over_many_chunks(dirs):
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


def test_a_gate_whose_part_takes_no_side_rows_is_a_product_of_its_own():
    """The sandwich block's gate beside a part that does not know of side rows (a gated feed-forward)."""
    from tempura_amd.config.spec import LayerSpec, PartSpec
    from tempura_amd.parts.block import SandwichBlock
    g = torch.Generator().manual_seed(3)
    norm = lambda n: PartSpec("rmsnorm", {"eps": 1e-6, "scalar": True}, {"weight": n})
    spec = LayerSpec("sandwich", {
        "mixer_norm": norm("n1"), "mixer": PartSpec("attention", {"num_heads": 2, "num_kv_heads": 2, "head_dim": 4, "scale": 0.5,
                                                                   "position": PartSpec("none")}, {"q": "q", "k": "k", "v": "v", "o": "o"}),
        "mixer_post_norm": norm("n1b"), "ffn_norm": norm("n2"), "ffn": PartSpec("gated", {"intermediate_size": 16},
                                                                               {"gate": "fg", "up": "fu", "down": "fd"}),
        "ffn_post_norm": norm("n2b"), "ffn_gate": PartSpec("input_sigmoid", {}, {"weight": "r", "bias": "rb"})})
    shapes = {k: v.shape for k, v in SandwichBlock.expected_weights(spec, 8).items()}
    assert shapes["r"] == (8, 8) and shapes["n1"] == ()
    W = {k: torch.randn(list(s), generator=g) for k, s in shapes.items()}
    block = SandwichBlock(spec, 8, torch.float32, "cpu")
    block.load_weights(lambda n: W[n])
    d = {k: v.double() for k, v in W.items()}
    x = torch.randn(5, 8, generator=g)
    u = plain.scalar_norm(x.double(), d["n2"], 1e-6)
    y = (plain_silu(u @ d["fg"].T) * (u @ d["fu"].T)) @ d["fd"].T
    want = x.double() + plain.scalar_norm(y * plain.stream_gate(u, d["r"], d["rb"]), d["n2b"], 1e-6)
    h = x.clone()
    x2 = block.ffn_norm.forward(h)
    block._close(h, x2, block._run(block.ffn, x2, None, None, 5, "cpu"), "ffn", None)
    assert float((h.double() - want).abs().max() / want.abs().max()) < TOL


def plain_silu(z):
    return z * torch.sigmoid(z)


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


def test_command_line_inspects_and_writes_random_folders(dirs, tmp_path, capsys):
    """`tempura inspect` on a folder of the design, and `tempura random-model --config-json` for it."""
    from tempura_amd.cli import main
    from tempura_amd.engine.loading import load_model
    assert main(["inspect", dirs["mix"]]) == 0
    text = capsys.readouterr().out
    assert "Tokatar" in text and "chunks of 9, 8 rotated, scores capped at 2" in text and "latent 20, gate per head" in text
    path = tmp_path / "c.json"
    path.write_text(json.dumps(cases.config_json("one")))
    assert main(["random-model", "--config-json", str(path), "--out", str(tmp_path / "rnd"), "--std", "0.3"]) == 0
    model = load_model(str(tmp_path / "rnd"), "float32", "cpu")
    assert model.layers[2].mixer.inner == 8 and model.final_norm.weight.shape == (32,)
    assert torch.equal(model.layers[0].closing["mixer"], torch.ones(32))


def test_sizes_the_configuration_leaves_out():
    """Without `vdim` values are as wide as keys, without `kv_heads` every head has its own, without `rot.dims` the whole
    head turns."""
    from tempura_amd.config import TokatarConfig
    d = cases.config_json("one")
    for key in ("vdim", "kv_heads"):
        del d["layers"][1]["mixer"][key]
    del d["layers"][0]["mixer"]["rot"]["dims"]
    cfg = TokatarConfig.from_dict(d)
    assert (cfg.layers[1].mixer.vdim, cfg.layers[1].mixer.kv_heads, cfg.layers[0].mixer.rot.dims) == (6, 3, 20)
