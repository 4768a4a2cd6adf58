"""Lurepel on the CPU: the configuration and its manifest, the plain implementation's mechanisms against closed forms, mistakes
planted in it that the test models must show, and the engine's own logic (chunks, slots used again, portions, batches,
generation) with the kernel library replaced by the torch double, against the plain implementation."""

import copy
import math

import numpy as np
import pytest

import beholdd
import lurepel_models as lm
import plain_lurepel as plain
import schedules
from beholdd.config import ConfigError, LurepelConfig
from beholdd.engine import Engine, StepEntry
from beholdd.parts import RotaryFrequencies
from beholdd.registry import configuration_of
from kernel_emulation import TorchKernels


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name, seed=5):
        if (name, seed) not in made:
            config = lm.CONFIGS[name]
            made[(name, seed)] = lm.write_model(tmp_path_factory.mktemp(f"lurepel_{name}_{seed}"), config, lm.random_weights(config, seed))
        return made[(name, seed)]

    return get


def make_engine(folder, dtype="float32", max_tokens=1024, **kw):
    return Engine(folder, dtype=dtype, max_tokens=max_tokens, device="cpu", kernels=TorchKernels(), **kw)


# ---- configuration -----------------------------------------------------------------------------------------

def test_every_constant_comes_from_the_file():
    config = LurepelConfig.from_dict(lm.MIXED)
    assert (config.vocab, config.hidden, config.rms_eps, config.max_position) == (97, 64, 1e-5, None)
    first, second, third = (layer.mixer for layer in config.layers[:3])
    assert (first.heads, first.kv_heads, first.dim, first.scale, first.chunk) == (4, 2, 32, 0.3, 70)
    assert (first.rot_dims, first.rot_base, first.rot_slowed) == (16, 500.0, (4.0, 1.0, 4.0, 64.0))
    assert (second.chunk, second.rot_dims, second.rot_slowed) == (0, 16, None)
    assert (third.chunk, third.rot_dims) == (64, 0)
    experts = config.layers[0].mlp
    assert (experts.experts, experts.identity, experts.top, experts.expert_ff) == (6, 2, 3, 32)
    assert config.layers[1].mlp is None and config.layers[2].mlp.ff == 80
    assert [kinds.feed_forward for kinds in config.layer_kinds()] == ["routed_identity_experts", "none", "geglu_tanh", "routed_identity_experts"]
    assert config.schedule() == [(0, 0), (1, 1), (2, 2), (3, 3)]
    assert LurepelConfig.from_dict(lm.ODD).layers[0].mlp.identity == 0


@pytest.mark.parametrize("change,message", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
    (lambda c: c["layers"][0].update(type="convolution"), "not implemented"),
    (lambda c: c["layers"][2]["mlp"].update(kind="routed"), "not implemented"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "group"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=16), "vdim"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=34), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=15), "pairs"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("high"), "high"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(low=5.0), "low"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "top"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "expert"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_a_configuration_that_lacks_or_overreaches_is_refused(change, message):
    config = copy.deepcopy(lm.MIXED)
    change(config)
    with pytest.raises(ConfigError, match=message):
        LurepelConfig.from_dict(config)


@pytest.mark.parametrize("name", sorted(lm.CONFIGS))
def test_the_manifest_is_what_the_configuration_implies(name):
    config = lm.CONFIGS[name]
    entry = beholdd.resolve_architecture(config)
    model = entry.build(configuration_of(entry, config))
    assert {spec.name: tuple(spec.shape) for spec in model.tensor_specs()} == lm.tensor_shapes(config)


def test_a_checkpoint_with_other_tensors_is_refused(tmp_path):
    weights = lm.random_weights(lm.ODD, 1)
    weights["l0.mix.v"] = weights.pop("l0.mix.k")
    folder = lm.write_model(tmp_path / "odd", lm.ODD, weights)
    with pytest.raises(beholdd.WeightError) as caught:
        make_engine(folder)
    assert caught.value.missing == ["l0.mix.k"] and caught.value.unexpected == ["l0.mix.v"]


def test_the_frequencies_are_the_plain_ones():
    for rot in [lm.rotation(16, 500.0), lm.rotation(64, 1e5, (8.0, 1.0, 4.0, 512)), lm.rotation(8, 10.0, (16.0, 2.0, 2.0, 16)),
                lm.rotation(32, 3000.0, (3.0, 0.0, 7.0, 100))]:
        slowed = tuple(rot["scaling"][k] for k in ("factor", "low", "high", "original")) if "scaling" in rot else None
        if slowed and slowed[1] == 0.0:
            rot = dict(rot, scaling=dict(rot["scaling"], low=1e-12))         # the plain form divides by it
        got = RotaryFrequencies(rot["dims"], rot["base"], slowed=slowed).values()
        assert np.abs(got / plain.frequencies(rot) - 1).max() < 1e-9
    with pytest.raises(ValueError, match="not both"):
        RotaryFrequencies(8, 100.0, stretch=(2.0, 16, 4.0, 1.0), slowed=(2.0, 1.0, 4.0, 16))


# ---- the plain implementation's mechanisms against closed forms --------------------------------------------

def test_plain_rotation_turns_neighbours_and_slows_long_waves():
    x = np.zeros((1, 1, 8))
    x[0, 0, 2], x[0, 0, 7] = 1.0, 5.0
    out = plain.turn(x, [3], {"dims": 6, "base": 100.0})
    angle = 3 * 100.0 ** (-2.0 / 6)
    want = np.zeros(8)
    want[2], want[3], want[7] = np.cos(angle), np.sin(angle), 5.0       # dimension 2 pairs with 3; 6 and 7 pass
    assert np.abs(out[0, 0] - want).max() < 1e-12
    # waves of 2 pi base^(i/4) positions; slowed by 4: as they are up to 64 / 4 positions, four times slower beyond 64 / 1
    rot = lm.rotation(8, 256.0, (4.0, 1.0, 4.0, 64))
    bare = np.array([1.0, 0.25, 0.0625, 0.015625])
    waves = 2 * math.pi / bare                                          # 6.3, 25.1, 100.5, 402.1
    got = plain.frequencies(rot)
    share = (64 / waves[1] - 1.0) / 3.0
    assert got[0] == 1.0 and abs(got[1] - ((1 - share) * 0.0625 + share * 0.25)) < 1e-15
    assert abs(got[2] - 0.0625 / 4) < 1e-15 and abs(got[3] - 0.015625 / 4) < 1e-15
    # scores depend on distances alone, with the slow pairs too
    rng = np.random.default_rng(0)
    q, k = rng.standard_normal((5, 1, 8)), rng.standard_normal((5, 1, 8))
    near = plain.turn(q, range(5), rot)[:, 0] @ plain.turn(k, range(5), rot)[:, 0].T
    far = plain.turn(q, range(900, 905), rot)[:, 0] @ plain.turn(k, range(900, 905), rot)[:, 0].T
    assert np.abs(near - far).max() < 1e-9
    # a turn keeps a head's length: unit length before it or after it is one thing
    assert np.abs(plain.unit(plain.turn(q, range(5), rot), 1e-5) - plain.turn(plain.unit(q, 1e-5), range(5), rot)).max() < 1e-12


def test_plain_softmax_holds_one_more_term():
    rng = np.random.default_rng(1)
    scores = rng.standard_normal((4, 4)) * 3
    visible = np.tril(np.ones((4, 4), bool))
    got = plain.softmax_with_one_more(scores, visible)
    for i in range(4):
        e = np.exp(scores[i, :i + 1])
        assert np.abs(got[i, :i + 1] - e / (1 + e.sum())).max() < 1e-14 and (got[i, i + 1:] == 0).all()
    assert np.abs(plain.softmax_with_one_more(np.full((1, 1), -800.0), np.ones((1, 1), bool))).max() < 1e-300


def test_plain_chunks_are_counted_from_the_first_position():
    table = plain.seen(7, 3)
    assert table.astype(int).tolist() == [[1, 0, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0, 0], [0, 0, 0, 1, 0, 0, 0],
                                          [0, 0, 0, 1, 1, 0, 0], [0, 0, 0, 1, 1, 1, 0], [0, 0, 0, 0, 0, 0, 1]]
    assert (plain.seen(5, 0) == np.tril(np.ones((5, 5), bool))).all()
    assert plain.seen(3, 4, first_position=3).astype(int).tolist() == [[1, 0, 0], [0, 1, 0], [0, 1, 1]]      # 3 | 4 5


def test_plain_attention_of_a_first_token():
    """It sees itself and the one more term: gate * e^s / (1 + e^s) * its own raw key, s = scale * |u(q)| |u(k)| cos."""
    rng = np.random.default_rng(2)
    m = {"heads": 2, "kv_heads": 1, "dim": 6, "scale": 0.7, "rot": {"dims": 4, "base": 50.0}, "mask": {"size": 4}}
    w = {"m.q": rng.standard_normal((12, 8)), "m.k": rng.standard_normal((6, 8)), "m.g": rng.standard_normal((2, 8)), "m.o": rng.standard_normal((8, 12))}
    h = rng.standard_normal((5, 8))
    got = plain.attention(h, w, "m.", m, 1e-5)
    for t in (0, 4):                                       # position 4 opens the second chunk
        k = w["m.k"] @ h[t]
        heads = []
        for head in range(2):
            q = w["m.q"][6 * head:6 * head + 6] @ h[t]
            s = 0.7 * (q @ k) / np.sqrt(((q ** 2).mean() + 1e-5) * ((k ** 2).mean() + 1e-5))      # both turned alike: nothing changes
            heads.append(k / (1 + np.exp(-s)) / (1 + np.exp(-(w["m.g"][head] @ h[t]))))
        want = w["m.o"] @ np.concatenate(heads)
        assert np.abs(got[t] - want).max() < 1e-12 * np.abs(want).max(), t
    # the same tokens further on in a sequence, at the same places of their chunks
    moved = plain.attention(h[:4], w, "m.", m, 1e-5, first_position=36)
    assert np.abs(moved - got[:4]).max() < 1e-10


def test_plain_experts_choose_by_corrected_scores_and_weigh_by_bare_ones():
    rng = np.random.default_rng(4)
    width, ff = 6, 4
    w = {"m.router": rng.standard_normal((4, width)), "m.correction": np.array([0.0, 0.9, 0.0, 0.0])}
    for e in range(3):
        w.update({f"m.e{e}.gate": rng.standard_normal((ff, width)), f"m.e{e}.up": rng.standard_normal((ff, width)),
                  f"m.e{e}.down": rng.standard_normal((width, ff))})
    h = rng.standard_normal((9, width))
    chosen, shares = plain.route(h, w, "m.", 2)
    z = h @ w["m.router"].T
    s = np.exp(z) / np.exp(z).sum(-1, keepdims=True)
    assert (chosen == 1).any(axis=-1).mean() > 0.9                            # the correction brings expert 1 in nearly everywhere ...
    assert np.abs(shares - np.take_along_axis(s, chosen, -1)).max() < 1e-14    # ... with its bare share, and nothing is renormed
    assert plain.route(np.zeros((1, width)), dict(w, **{"m.correction": np.zeros(4)}), "m.", 2)[0].tolist() == [[0, 1]]      # ties
    got = plain.experts(h, w, "m.", {"router": {"experts": 3, "identity": 1, "top": 2}})
    want = np.zeros_like(h)
    for t in range(9):
        for e, share in zip(chosen[t], shares[t]):
            g, u = (w[f"m.e{e}.{name}"] @ h[t] for name in ("gate", "up")) if e < 3 else (None, None)
            want[t] += share * (h[t] if e == 3 else w[f"m.e{e}.down"] @ (g / (1 + np.exp(-g)) * u))
    assert np.abs(got - want).max() < 1e-12 and (chosen == 3).any()


def test_plain_dense_gate():
    w = {"m.gate": np.array([[1.0]]), "m.up": np.array([[2.0]]), "m.down": np.array([[1.0]])}
    got = plain.dense(np.array([[1.5]]), w, "m.")[0, 0]
    assert abs(got - 0.75 * (1 + math.tanh(math.sqrt(2 / math.pi) * (1.5 + 0.044715 * 1.5 ** 3))) * 3.0) < 1e-12


def planted(monkeypatch, name):
    """A mistake in the plain implementation: what the model would be without one of its mechanisms, or with it a little off."""
    real = {key: getattr(plain, key) for key in ("softmax_with_one_more", "frequencies", "seen", "route", "unit", "turn", "gelu", "experts", "attention")}
    if name == "no sink":
        monkeypatch.setattr(plain, "softmax_with_one_more", lambda s, v: plain.softmax(np.where(v, s, -np.inf)))
    elif name == "plain frequencies":
        monkeypatch.setattr(plain, "frequencies", lambda rot: real["frequencies"]({k: rot[k] for k in ("dims", "base")}))
    elif name == "chunks one longer":
        monkeypatch.setattr(plain, "seen", lambda t, c, f=0: real["seen"](t, c + 1 if c else 0, f))
    elif name == "no chunks":
        monkeypatch.setattr(plain, "seen", lambda t, c, f=0: real["seen"](t, 0, f))
    elif name == "values normed":
        monkeypatch.setattr(plain, "attend", lambda q, k, v, *rest: attend(q, k, k, *rest))
    elif name == "split halves":
        def halves(x, positions, rot):
            d = int(rot["dims"])
            order = np.arange(d).reshape(2, d // 2).T.reshape(-1)
            y = plain.f64(x).copy()
            y[..., :d] = y[..., order]
            y = real["turn"](y, positions, rot)
            out = y.copy()
            out[..., order] = y[..., :d]
            return out
        monkeypatch.setattr(plain, "turn", halves)
    elif name == "corrected weights":
        def corrected(h, w, p, top):
            chosen, shares = real["route"](h, w, p, top)
            return chosen, shares + plain.f64(w[p + "correction"])[chosen]
        monkeypatch.setattr(plain, "route", corrected)
    elif name == "uncorrected choice":
        monkeypatch.setattr(plain, "route", lambda h, w, p, top: real["route"](h, dict(w, **{p + "correction": np.zeros(len(w[p + "correction"]))}), p, top))
    elif name == "softmax without identity experts":
        def fewer(h, w, p, mlp):
            n = mlp["router"]["experts"]
            return real["experts"](h, dict(w, **{p + "router": w[p + "router"][:n], p + "correction": w[p + "correction"][:n]}), p,
                                   {"router": {"experts": n, "top": min(n, mlp["router"]["top"])}})
        monkeypatch.setattr(plain, "experts", fewer)
    elif name == "another gate":
        monkeypatch.setattr(plain, "gelu", plain.silu)
    elif name == "no gates":
        monkeypatch.setattr(plain, "attention", lambda h, w, p, *rest: real["attention"](h, dict(w, **{p + "g": np.zeros_like(w[p + "g"])}), p, *rest))
    else:
        raise AssertionError(name)


attend = plain.attend


@pytest.mark.parametrize("name", ["no sink", "plain frequencies", "chunks one longer", "no chunks", "values normed", "split halves",
                                  "corrected weights", "uncorrected choice", "softmax without identity experts", "another gate",
                                  "no gates"])
def test_the_test_models_show_a_planted_mistake(monkeypatch, name):
    """Every mechanism moves the logits of a test model by far more than the tests' tolerances: a kernel that leaves it out, or
    puts it a little off, cannot pass them.  (One factor on all of a token's shares, as renorming them would put there, is not
    among them: the norm behind the experts takes it out again.  The routing is held to the shares themselves further down and on
    the GPU.)"""
    config = lm.MIXED
    weights = lm.random_weights(config, 5)
    tokens = schedules.random_requests(config["vocab"], [150], seed=3)[0]
    right = plain.forward(config, weights, tokens)
    planted(monkeypatch, name)
    wrong = plain.forward(config, weights, tokens)
    assert np.abs(wrong - right).max() > 0.05 * np.abs(right).max()


# ---- the engine's logic with the torch double ----------------------------------------------------------------

@pytest.mark.parametrize("name,lengths", [("mixed", [5, 70, 17, 131]), ("plain", [1, 23, 66]), ("odd", [3, 64, 65, 9]), ("wide", [40, 7, 140])])
def test_every_cut_matches_the_plain_implementation(folders, name, lengths):
    folder = folders(name)
    config, weights = plain.load(folder)
    requests = schedules.random_requests(config["vocab"], lengths, seed=3)
    expected = [plain.forward(config, weights, r) for r in requests]
    engine = make_engine(folder)
    for label, got in (("whole", schedules.whole(engine, requests)),
                       ("tail", schedules.tail_one_by_one(engine, requests, tail=12)),
                       ("batches", schedules.batches(engine, requests, batch_size=3)),
                       ("portions", schedules.portions(engine, requests))):
        for i, (g, e) in enumerate(zip(got, expected)):
            assert g.shape == e.shape, (label, i)
            assert schedules.relative_error(g, e) < 1e-4, (label, i, schedules.relative_error(g, e))
    engine.cache.check_invariants()
    assert engine.cache.live_slots() == []
    assert engine.cache.free_page_count() == engine.cache.n_pages


def test_the_residual_after_every_layer(folders):
    folder = folders("mixed")
    config, weights = plain.load(folder)
    tokens = schedules.random_requests(config["vocab"], [21], seed=12)[0]
    want = []
    plain.forward(config, weights, tokens, residuals=want)
    engine = make_engine(folder)
    seen = []
    for block in engine.model.own_blocks():
        real = block.forward

        def spy(ctx, hidden, cache, prepared=None, next_block=None, real=real):
            result = real(ctx, hidden, cache, prepared, next_block)
            seen.append(hidden.clone().numpy())
            return result

        block.forward = spy
    slot = engine.alloc_slot()
    engine.step([StepEntry(slot, tokens, [])])
    assert len(seen) == len(want) == 4
    for layer, (g, e) in enumerate(zip(seen, want)):
        assert np.abs(g - e).max() < 1e-5 * np.abs(e).max(), layer


def test_layers_cache_their_own_heads_and_give_pages_back_behind_a_chunk(folders):
    folder = folders("mixed")
    config, weights = plain.load(folder)
    engine = make_engine(folder)
    needs = engine.model.entry_needs
    assert [(n.kv_heads, n.head_dim, n.window) for n in (needs[i] for i in range(4))] == [(2, 32, 70), (1, 32, 0), (2, 64, 64), (3, 64, 33)]
    tokens = schedules.random_requests(config["vocab"], [300], seed=2)[0]
    slot = engine.alloc_slot()
    engine.step([StepEntry(slot, tokens[:290], [])])
    held = {g.need.window: sum(page >= 0 for page in g.pages_of[slot]) for g in engine.cache.groups}
    assert held[0] == 5 and all(count <= 2 for window, count in held.items() if window)
    got = np.concatenate([engine.step([StepEntry(slot, [t], [0])]).numpy() for t in tokens[290:]])
    assert schedules.relative_error(got, plain.forward(config, weights, tokens)[290:]) < 1e-4
    engine.cache.check_invariants()


def test_a_slot_that_is_used_again_starts_from_nothing(folders):
    folder = folders("wide")
    config, weights = plain.load(folder)
    first, second = schedules.random_requests(config["vocab"], [80, 30], seed=8)
    engine = make_engine(folder, max_tokens=128, max_slots=1)
    slot = engine.alloc_slot()
    engine.step([StepEntry(slot, first, [])])
    engine.free_slot(slot)
    again = engine.alloc_slot()
    assert again == slot
    got = engine.step([StepEntry(again, second, list(range(len(second))))]).numpy()
    assert schedules.relative_error(got, plain.forward(config, weights, second)) < 1e-4


def test_a_step_whose_choices_are_all_identity_experts(tmp_path):
    """Corrections that put the experts without matrices ahead everywhere: prompts (whose experts run as products over gathered
    rows) and decode steps have no expert's rows to compute."""
    for ff, width in ((64, 64), (20, 36)):
        config = {"architecture": "Lurepel", "vocab": 50, "width": width, "norm": {"eps": 1e-5},
                  "layers": [lm.attention(2, 1, 16, 0.3, dims=8, mlp=lm.moe(2, 2, ff, identity=3)), lm.attention(2, 1, 16, 0.3, mlp=lm.dense(40))]}
        weights = lm.random_weights(config, 3)
        weights["l0.mlp.correction"][:] = [-4, -4, 0, 0.5, 0.25]
        folder = lm.write_model(tmp_path / f"identity{ff}", config, weights)
        requests = schedules.random_requests(50, [70, 3], seed=1)
        engine = make_engine(folder)
        for label, got in (("whole", schedules.whole(engine, requests)), ("tail", schedules.tail_one_by_one(engine, requests, tail=5))):
            for g, r in zip(got, requests):
                assert schedules.relative_error(g, plain.forward(config, weights, r)) < 1e-4, label


def test_greedy_generation_through_the_engine(folders):
    folder = folders("mixed")
    config, weights = plain.load(folder)
    prompts = schedules.random_requests(config["vocab"], [1, 9, 30], seed=6)
    engine = make_engine(folder)
    results = engine.generate(prompts, max_new_tokens=[6, 8, 5])
    for prompt, result, n_new in zip(prompts, results, [6, 8, 5]):
        want = plain.greedy(config, weights, prompt, n_new)
        assert result.token_ids == want, (result.token_ids, want)
    assert len({token for r in results for token in r.token_ids}) >= 4       # the continuations vary
    engine.cache.check_invariants()
    assert engine.cache.live_slots() == []


def test_prompts_longer_than_a_step_go_through_in_portions(folders):
    folder = folders("odd")
    config, weights = plain.load(folder)
    prompts = schedules.random_requests(config["vocab"], [50, 3, 21], seed=9)
    engine = make_engine(folder, max_rows_per_step=8)
    results = engine.generate(prompts, max_new_tokens=4)
    for prompt, result in zip(prompts, results):
        assert result.token_ids == plain.greedy(config, weights, prompt, 4)


@pytest.mark.parametrize("seed", range(8))
def test_drawn_configurations_on_the_torch_double(seed, tmp_path):
    """Sizes, counts, constants and layer orders that nobody picked: whole prompts, a tail token by token, a batch."""
    config = lm.drawn_config(seed)
    folder = lm.write_model(tmp_path / "drawn", config, lm.random_weights(config, seed, gain=0.7))
    _, weights = plain.load(folder)
    requests = schedules.random_requests(config["vocab"], [1, 19, 70], seed=seed)
    expected = [plain.forward(config, weights, r) for r in requests]
    engine = make_engine(folder)
    for label, got in (("whole", schedules.whole(engine, requests)), ("tail", schedules.tail_one_by_one(engine, requests, tail=5)),
                       ("batches", schedules.batches(engine, requests, batch_size=3))):
        for i, (g, e) in enumerate(zip(got, expected)):
            assert schedules.relative_error(g, e) < 1e-4, (config, label, i, schedules.relative_error(g, e))


def test_the_command_line_plans_the_bytes_of_this_design_without_a_gpu(folders):
    import io
    from beholdd import cli
    out = io.StringIO()
    code = cli.main(["generate", "--model", folders("mixed"), "--prompt-ids", "1,2,3", "--max-new-tokens", "70", "--dtype", "bfloat16",
                     "--plan-only"], out=out)
    text = out.getvalue()
    assert code == 0, text
    assert "keys/values of 1 layers (2 heads x 32, window 70)" in text and "keys/values of 1 layers (1 heads x 32)" in text
    assert "not counted" not in text          # every part says what a step of its allocates


def test_a_walk_over_a_stretch_of_keys_is_planned_for_as_many_pages_as_its_rows_can_touch():
    from beholdd.kernels.library import KernelSizes
    page = KernelSizes.PAGE
    for span in (1, 2, 63, 64, 65, 70, 128, 1000):
        for rows in (1, 16):
            most = max((start + span - 1 + rows - 1) // page - start // page + 1 for start in range(2 * page))
            assert KernelSizes.furthest(10 ** 6, window=span) // page + 1 >= most, (span, rows)
        assert KernelSizes.furthest(10 ** 6, chunk=span) == KernelSizes.furthest(10 ** 6, window=span)
    assert KernelSizes.furthest(40, window=1000) == 40 and KernelSizes.furthest(4000) == 4000
