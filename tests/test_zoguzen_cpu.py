"""Zoguzen on the CPU: configuration, the model's description, and the engine's own logic (pages shared between layers, state
slots, batches, portions, scheduler) with the plain kernels of tests/reference_ops.py in place of the HIP library, against the
plain implementation of tests/plain_zoguzen.py; and that plain implementation's mechanisms one by one."""
import copy

import numpy as np
import pytest
import torch

import plain_zoguzen as pz
import trace_tools as tt
import zoguzen_configs as zc
from reference_ops import ReferenceOps
from fllm_amd import Engine, SamplingParams
from fllm_amd.config.spec import ConfigError
from fllm_amd.engine import ModelRunner, StepEntry
from fllm_amd.registry import model_spec_from_config
from fllm_amd.weights.loader import WeightsError, check_tensors
from fllm_amd.weights.random_init import random_tensors


def make_runner(cfg, tensors, page_size, max_tokens, **kw):
    _, spec = model_spec_from_config(cfg)
    return ModelRunner(spec, dict(tensors), dtype="float32", device="cpu", page_size=page_size, max_tokens=max_tokens,
                       **{"max_requests": 4, "max_context": 512, "ops": ReferenceOps(), **kw})


def runner_for(name, max_tokens, seed=3, **kw):
    cfg = zc.CONFIGS[name]
    tensors = zc.weights(cfg, seed)
    return cfg, zc.to_float64(tensors), make_runner(cfg, tensors, zc.PAGE_SIZES[name], max_tokens, **kw)


def near(got, want, tol=3e-5):
    assert np.abs(got - want).max() <= tol * np.abs(want).max()


# ---- the plain implementation's mechanisms, each alone ----------------------------------------------------------------
def test_plain_layer_norm_takes_the_mean_off_and_no_bias_back_on():
    x = np.array([[1.0, 3.0, 5.0, 7.0]])
    out = pz.layer_norm(x, np.array([1.0, 1.0, 2.0, 1.0]), 0.0)
    assert np.allclose(out, np.array([[-3.0, -1.0, 2.0, 3.0]]) / np.sqrt(5.0))
    assert np.allclose(pz.layer_norm(x + 100.0, np.ones(4), 1e-5), pz.layer_norm(x, np.ones(4), 1e-5))


def test_plain_shift_moves_towards_the_token_before_and_the_first_towards_nothing():
    h = np.array([[1.0, 2.0], [3.0, 4.0], [5.0, 8.0]])
    out = pz.token_shift(h, np.array([0.0, 0.5]))
    assert np.allclose(out, [[1.0, 1.0], [3.0, 3.0], [5.0, 6.0]])


def test_plain_convolution_reads_back_as_far_as_its_taps_and_zeros_before_the_start():
    u = np.zeros((6, 1))
    u[2, 0] = 1.0
    taps = np.array([[7.0, 5.0, 3.0]])               # the last tap meets the newest value
    assert np.allclose(pz.causal_conv(u, taps)[:, 0], [0, 0, 3, 5, 7, 0])
    assert np.allclose(pz.causal_conv(np.ones((4, 1)), taps)[:, 0], [3, 8, 15, 15])


def test_plain_rotation_turns_neighbouring_lanes_and_leaves_the_rest():
    x = np.zeros((3, 1, 6))
    x[:, 0, 2], x[:, 0, 5] = 1.0, 7.0
    out = pz.rotate(x, {"dims": 4, "base": 10.0}, [0, 1, 2])
    a = np.array([0, 1, 2]) * 10.0 ** (-2 / 4)
    assert np.allclose(out[:, 0, 2], np.cos(a)) and np.allclose(out[:, 0, 3], np.sin(a))      # lane 2 turns into lane 3
    assert np.allclose(out[:, 0, :2], 0) and np.allclose(out[:, 0, 4:], x[:, 0, 4:])


def test_plain_wave_scaling_keeps_short_waves_divides_long_ones_and_blends_between():
    scaling = dict(zip(("factor", "low", "high", "original"), zc.WAVES))
    f = pz.frequencies({"dims": 16, "base": 100.0})
    g = pz.frequencies({"dims": 16, "base": 100.0, "scaling": scaling})
    wave = 2 * np.pi / f
    kept, divided = wave < 32 / 4.0, wave > 32 / 1.0
    between = ~kept & ~divided
    assert kept.any() and divided.any() and between.any()
    assert np.allclose(g[kept], f[kept]) and np.allclose(g[divided], f[divided] / 4.0)
    s = (32 / wave[between] - 1.0) / 3.0
    assert np.allclose(g[between], (1 - s) * f[between] / 4 + s * f[between])


def test_plain_masks_at_their_edges():
    c = pz.sees_chunk(9, 4)
    assert [list(np.nonzero(c[i])[0]) for i in (0, 3, 4, 8)] == [[0], [0, 1, 2, 3], [4], [8]]
    w = pz.sees_window_and_first(9, 3, 2)
    assert [list(np.nonzero(w[i])[0]) for i in (0, 2, 3, 4, 8)] == [[0], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 6, 7, 8]]
    assert list(np.nonzero(pz.sees_window_and_first(9, 3, 0)[8])[0]) == [6, 7, 8]


def test_plain_sink_cap_and_mixed_weights():
    T, H = 3, 2
    q, k, v = np.zeros((T, H, 2)), np.zeros((T, 2, 2)), np.zeros((T, 2, 1))
    v[:, 0, 0], v[:, 1, 0] = 1.0, 10.0
    share = np.array([1 / 2, 2 / 3, 3 / 4])                    # n keys of score 0 and the sink: n / (n + 1)
    out = pz.sink_talking_attention(q, k, v, 1.0, 5.0, pz.sees_chunk(T, 8), np.eye(2))
    assert np.allclose(out[:, 0, 0], share) and np.allclose(out[:, 1, 0], 10 * share)
    talk = np.array([[0.5, 2.0], [-1.0, 0.0]])                 # head 0 applies 2.5 times the weight, to its own values
    out = pz.sink_talking_attention(q, k, v, 1.0, 5.0, pz.sees_chunk(T, 8), talk)
    assert np.allclose(out[:, 0, 0], 2.5 * share) and np.allclose(out[:, 1, 0], -10 * share)
    loud = pz.sink_talking_attention(np.full((1, 1, 1), 50.0), np.full((1, 1, 1), 50.0), np.ones((1, 1, 1)), 1.0, 3.0, pz.sees_chunk(1, 8), np.eye(1))
    assert np.isclose(loud[0, 0, 0], np.exp(3.0) / (1 + np.exp(3.0)))      # 2500 is capped to 3


def test_plain_gated_recurrence_is_a_sum_over_products_of_decays():
    rng = np.random.default_rng(0)
    T, H, d, dv = 6, 2, 3, 4
    q, k, v = rng.normal(size=(T, H, d)), rng.normal(size=(T, H, d)), rng.normal(size=(T, H, dv))
    alpha = rng.uniform(0.2, 1.0, (T, H, d))
    got = pz.gated_recurrence(q, k, v, alpha)
    for t in range(T):
        for h in range(H):
            want = sum((q[t, h] * k[s, h] * np.prod(alpha[s + 1:t + 1, h], axis=0)).sum() * v[s, h] for s in range(t + 1))
            assert np.allclose(got[t, h], want)


def test_plain_min_recurrence_candidates_and_gates():
    z = np.array([[1.0, 0.0, 0.25], [1.0, 0.0, 0.25]])
    u = np.array([[2.0, 3.0, 0.0], [-1.0, 3.0, 4.0]])
    out = pz.min_recurrence(z, u)
    assert np.allclose(out[0], [2.5, 0.0, 0.125])              # open gate takes the candidate, shut gate nothing, u = 0 gives 1/2
    assert np.allclose(out[1], [1 / (1 + np.e), 0.0, 0.75 * 0.125 + 0.25 * 4.5])


def test_plain_router_weighs_by_the_picked_logits_alone():
    z = np.array([[1.0, 4.0, 2.0, 3.0]])
    ids, w = pz.route(np.eye(4)[:1], np.concatenate([z.T, np.zeros((4, 3))], axis=1), 2)
    assert ids.tolist() == [[1, 3]] and np.allclose(w, [[np.e / (1 + np.e), 1 / (1 + np.e)]])


# ---- configuration and description ------------------------------------------------------------------------------------
def test_the_description_names_the_parts():
    typed, spec = model_spec_from_config(zc.A)
    assert spec.architecture == "zoguzen" and [(e.layer, e.reads_cache_of) for e in spec.run_order] == [(0, None), (1, None), (2, 0), (3, None)]
    assert all(layer.mixer.kind == "conv_input" and layer.mixer["form"] == "shift" and layer.block.kind == "parallel" for layer in spec.layers)
    inner = [layer.mixer["inner"] for layer in spec.layers]
    assert [p.kind for p in inner] == ["conv_attention", "mixer_pair", "conv_attention", "min_gru"]
    assert inner[0]["chunk"] == 12 and inner[0]["softcap"] == 6.0 and inner[0]["sink"] == "zero" and inner[0]["mix_weights"]
    assert inner[0]["own_keys"] and not inner[2]["own_keys"] and set(inner[2].tensors) == {"q", "q_bias", "q_conv", "q_norm", "talk", "o"}
    left, right = inner[1]["left"], inner[1]["right"]
    assert left["window"] == 7 and left["keep_first"] == 3 and left["output_gate"] and left["position"]["scaling"] == "llama3"
    assert left["position"]["pairing"] == "interleaved" and left.get("qk_norm_eps") is None and not left.get("mix_weights")
    assert right.kind == "gated_linear" and right["tau"] == 4.0 and right["query_scale"] == 12 ** -0.5
    assert inner[1]["left_scale"] == inner[1]["right_scale"] == 0.5 and inner[1]["out_norm_eps"] == 1e-5
    assert spec.layers[2].feed_forward is None and "l2.norm2" in spec.ignorable_tensors
    ff = spec.layers[3].feed_forward
    assert ff["experts"] == 6 and ff["top"] == 3 and ff["score"] == "softmax" and ff["renormalize"] and ff["weight_on"] == "output"
    assert spec.layers[3].extras["after"][1]["layer"] == 3 and spec.head["softcap"] == 12.0 and spec.final_norm.kind == "layer"


def test_readers_share_the_pages_of_their_source_and_every_layer_has_its_state():
    _, _, r = runner_for("C", 64)
    b = r.model.bindings
    assert b[0].writes and not b[2].writes and not b[3].writes
    assert b[0].k_pages.data_ptr() == b[2].k_pages.data_ptr() == b[3].k_pages.data_ptr() and b[0].group == b[2].group
    assert b[1].k_pages.data_ptr() != b[0].k_pages.data_ptr()
    assert set(b[0].state) == {"", "conv_inputs"} and b[0].state[""].shape == (4, 3, 3 * 10 + 10 + 6) and b[0].state["conv_inputs"].shape == (4, 1, 52)
    assert b[2].state[""].shape == (4, 3, 30) and b[3].state[""].shape == (4, 1, 30)              # queries alone pass a reader's convolution
    assert set(b[1].state) == {"left.", "right.", "conv_inputs"} and b[1].state["right."].shape == (4, 3, 9, 7)
    _, _, a = runner_for("B", 64)
    assert a.model.bindings[0].group == -1 and a.model.bindings[0].state[""].shape == (4, 7)
    assert set(a.model.bindings[1].state) == {"conv_inputs"}                                      # one tap keeps nothing


@pytest.mark.parametrize("change,match", [
    (lambda c: c["layers"][0].__setitem__("type", "lightning"), "no mixer of this design"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "dense"), "no feed-forward of this design"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 3), "not a multiple"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("conv", 0), "positive"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("conv", 17), "more than 16"),
    (lambda c: c["layers"][0]["mixer"].pop("mask"), "requires layers\\[0\\].mixer.mask"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 2), "no layer before this one"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 1), "without keys and values of its own"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("vdim", 16), "that layer holds"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].__setitem__("keep_first", -1), "negative"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].__setitem__("dims", 7), "even and at most dim"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].__setitem__("high", 1.0), "above low"),
    (lambda c: c["layers"][1]["mixer"]["right"].__setitem__("tau", 0.0), "positive"),
    (lambda c: c["layers"][3]["mixer"].pop("width"), "requires layers\\[3\\].mixer.width"),
    (lambda c: c["layers"][3]["mlp"]["router"].__setitem__("top", 7), "more than the 6 experts"),
    (lambda c: c.pop("token_side"), "requires token_side"),
    (lambda c: c.__setitem__("logit_softcap", 0.0), "positive"),
    (lambda c: c["norm"].__setitem__("eps", 0), "positive"),
])
def test_configurations_that_are_refused(change, match):
    cfg = copy.deepcopy(zc.A)
    change(cfg)
    with pytest.raises(ConfigError, match=match):
        model_spec_from_config(cfg)


def test_the_loader_names_what_does_not_fit_and_takes_any_rank():
    _, spec = model_spec_from_config(zc.A)
    shapes = {n: tuple(t.shape) for n, t in zc.weights(zc.A, 1).items()}
    check_tensors(spec, shapes)
    check_tensors(spec, {n: tuple(t.shape) for n, t in zc.weights(zc.A, 1, rank=11).items()})
    broken = dict(shapes)
    del broken["l0.mix.talk"]
    del broken["l1.mix.right.out"]
    broken["l2.mix.k"] = (32, 48)                    # a reader has no keys of its own
    broken["side.embed"] = (90, 24)                  # one part a layer is missing
    with pytest.raises(WeightsError) as err:
        check_tensors(spec, broken)
    assert err.value.missing == ["l0.mix.talk", "l1.mix.right.out"] and err.value.unexpected == ["l2.mix.k"]
    assert [w[0] for w in err.value.wrong_shape] == ["side.embed"]
    made = random_tensors(spec, 0, torch.float32)
    assert made["l1.mix.right.a1"].shape == (16, 48)


# ---- the engine's logic -------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name,lengths", [("A", [5, 30, 61]), ("B", [45, 2]), ("C", [9, 50]), ("D", [70, 37])])
@pytest.mark.parametrize("family", ["whole", "last", "portions", "mixed"])
def test_every_way_of_cutting_gives_the_plain_logits(tmp_path, name, lengths, family):
    vocab = zc.CONFIGS[name]["vocab"]
    requests = {f"r{i}": zc.random_ids(n, vocab, 70 + i) for i, n in enumerate(lengths)}
    steps = {"whole": tt.whole, "last": lambda r: tt.last_tokens_one_by_one(r, 19), "portions": tt.portions,
             "mixed": lambda r: tt.mixed(r, seed=4, decode_tail=6, refeed=["r0"])}[family](requests)
    steps = tt.number(steps)
    cfg, w64, runner = runner_for(name, tt.live_tokens_bound(steps, round_to=zc.PAGE_SIZES[name]))
    given_up = {}
    got = tt.run_in_process(runner, steps, vocab, str(tmp_path), given_up)
    for rid, feedings in given_up.items():          # ended half way and fed again: other pages, a cleared slot, the same logits
        near(feedings[0], got[rid][:len(feedings[0])], 1e-5)
    for rid, toks in requests.items():
        near(got[rid], pz.forward(cfg, w64, toks))
    runner.cache.check_invariants()
    assert all(p.available == p.num_pages for p in runner.cache.pools)


def test_portions_of_two_tokens_and_of_one():
    for name in ("A", "C"):
        cfg, w64, runner = runner_for(name, 64)
        toks = zc.random_ids(41, cfg["vocab"], 6)
        got = [runner.step([StepEntry("a", toks[i:i + 2], list(range(len(toks[i:i + 2]))))]).numpy() for i in range(0, 41, 2)]
        near(np.concatenate(got), pz.forward(cfg, w64, toks))


def test_the_residual_stream_after_every_layer():
    cfg, w64, runner = runner_for("C", 64)
    seen = []
    for block in runner.model.blocks:
        def wrapped(ctx, x, binding, _inner=block.forward):
            _inner(ctx, x, binding)
            seen.append(x.clone().numpy())
        block.forward = wrapped
    toks = zc.random_ids(29, cfg["vocab"], 5)
    runner.step([StepEntry("a", toks, [])])
    want, _ = pz.layer_outputs(cfg, w64, toks)
    assert len(seen) == len(want) == 5
    for got, ref in zip(seen, want):
        near(got, ref, 2e-5)


@pytest.mark.parametrize("far", [0, 2, 3, 4, 11, 12, 16, 17, 18, 23])
def test_one_loud_token_around_the_edges(far):
    """A, pages of 8.  The last query sits at position 23: its chunk of 12 begins at 12, the reader's chunk of 9 at 18, the window of
    7 at 17, and the first 3 tokens are kept.  One token's embedding stands out, its key with it; whether it is seen shows, fed as
    one prompt and decoded token by token."""
    cfg, tensors = zc.A, zc.weights(zc.A, 9)
    toks = [3 + t % 80 for t in zc.random_ids(24, 90, 77)]
    toks[far] = 1
    tensors["embed"][1] *= 8.0
    w64 = zc.to_float64(tensors)
    want = pz.forward(cfg, w64, toks)
    r = make_runner(cfg, tensors, 8, 64)
    near(r.step([StepEntry("a", toks, list(range(24)))]).numpy(), want)
    r.free_request("a")
    got = [r.step([StepEntry("b", toks[:10], list(range(10)))]).numpy()] + [r.step([StepEntry("b", [t], [0])]).numpy() for t in toks[10:]]
    near(np.concatenate(got), want)


def test_a_slot_and_pages_that_are_used_again_start_clean():
    cfg, w64, runner = runner_for("A", 64)
    first, second = zc.random_ids(40, cfg["vocab"], 1), zc.random_ids(27, cfg["vocab"], 2)
    runner.step([StepEntry("a", first, [])])
    slot, pages = runner.cache.slot("a"), list(runner.cache.table("a", 0))
    runner.free_request("a")
    got = runner.step([StepEntry("b", second, list(range(27)))]).numpy()
    assert runner.cache.slot("b") == slot and set(runner.cache.table("b", 0)) <= set(pages)
    near(got, pz.forward(cfg, w64, second))


def test_long_decoding_from_the_first_token():
    for name in ("B", "A"):
        cfg, w64, runner = runner_for(name, 128)
        toks = zc.random_ids(80, cfg["vocab"], 8)
        near(np.concatenate([runner.step([StepEntry("a", [t], [0])]).numpy() for t in toks]), pz.forward(cfg, w64, toks))


def test_batches_of_unequal_requests_agree_with_each_alone():
    cfg, w64, runner = runner_for("A", 192)
    a, b, c = (zc.random_ids(n, cfg["vocab"], 40 + n) for n in (37, 2, 21))
    runner.step([StepEntry("a", a[:30], []), StepEntry("c", c[:20], [])])
    got = runner.step([StepEntry("a", a[30:], list(range(7))), StepEntry("b", b, [0, 1]), StepEntry("c", c[20:], [0])]).numpy()
    near(got, np.concatenate([pz.forward(cfg, w64, a)[30:], pz.forward(cfg, w64, b), pz.forward(cfg, w64, c)[20:]]))


@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_scheduler(tmp_path, name):
    cfg = zc.CONFIGS[name]
    tensors = zc.weights(cfg, 11)
    folder = zc.write_model(str(tmp_path / "m"), cfg, tensors)
    prompts = [zc.random_ids(n, cfg["vocab"], 20 + n) for n in (3, 26, 41)]
    w64 = zc.to_float64(tensors)
    want = []
    for p in prompts:
        toks = list(p)
        for _ in range(8):
            toks.append(int(np.argmax(pz.forward(cfg, w64, toks)[-1])))
        want.append(toks[len(p):])
    for opts in (dict(num_blocks=64), dict(num_blocks=12, max_batched_tokens=12)):       # roomy; few pages and small portions
        engine = Engine(folder, dtype="float32", device="cpu", ctx=256, max_seqs=3, block_size=zc.PAGE_SIZES[name],
                        ops=ReferenceOps(), **{"max_batched_tokens": 32, **opts})
        assert engine.generate(prompts, SamplingParams(max_tokens=8)) == want
        engine.runner.cache.check_invariants()
