"""Mutedra as data: which parts each layer has and what its tensors are called.

A layer is the "sandwich" arrangement, x += norm1b(mixer(norm1(x))), then, where the layer has a feed-forward,
x += norm2b(ff(norm2(x))); the norms are "dynamic_tanh". The mixer is

  "attention": the part "attention" without a norm or a rotation, with a window that keeps the first keys, a learned
      bias by distance and a one in the softmax's denominator;
  "latent_attention": the part "latent_attention" with queries from a latent of their own and no rotated part;
  "latent_attention_2": the same with a rotated part (neighbouring pairs), a sink a head and a gate a head.

The feed-forward is "swiglu" with relu. The configuration's loop is a matter of the schedule: it names the looped
layers once a pass, every run with a cache entry of its own, and marks where a pass starts ("step_and_embedding"
says what joins the stream there). The embedding's rows are scaled, the head is a matrix of its own whose logits are
capped. Tensors are stored under short names: `l<i>.norm1` (with `.alpha` and `.b` beside it) and so on,
`l<i>.mix.<name>`, `l<i>.mlp.<name>`, `embed`, `loop.step`, `final.norm`, `head`.
"""
from ..config import register_architecture
from ..config.mutedra import MutedraConfig
from ..parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def _attention(cfg, m, p):
    return PartSpec("attention", {"hidden_size": cfg.hidden_size, "num_heads": m.heads, "num_kv_heads": m.kv_heads,
                                  "head_dim": m.dim, "value_dim": m.vdim, "eps": cfg.norm_eps, "position": PartSpec("none"),
                                  "names": {k: p + k for k in ("q", "k", "v", "o", "rel")}, "qk_norm": False,
                                  "scale": m.scale, "window": m.window, "keep_first": m.keep_first,
                                  "distance_bias": (m.bias_max,), "sink": "unit"})


def _latent(cfg, m, p, rotated=None):
    names = {"dq": p + "dq", "dq_norm": p + "dq.norm", "uq": p + "uq", "dkv": p + "dkv", "dkv_norm": p + "dkv.norm",
             "uk": p + "uk", "uv": p + "uv", "o": p + "o"}
    position, rot_dim = PartSpec("none"), 0
    if rotated is not None:
        names.update(sink=p + "sink", g=p + "g")
        # the angles are computed from the positions, so no table bounds them; the part puts the rotated rows of its
        # projections into the order in which a rotation of halves turns what were neighbours
        rot_dim = rotated.rot_dim
        position = PartSpec("rope", {"theta": rotated.rot_base, "rotary_dims": rot_dim,
                                     "max_positions": cfg.max_position_embeddings, "tables": False})
    return PartSpec("latent_attention", {"hidden_size": cfg.hidden_size, "heads": m.heads, "dim": m.dim, "rot_dim": rot_dim,
                                         "vdim": m.vdim, "kv_rank": m.kv_rank, "q_rank": m.q_rank, "scale": m.scale,
                                         "eps": cfg.norm_eps, "position": position, "names": names, "gate": "head",
                                         "pairs": True, "sink": rotated is not None})


MIXER_SPECS = {"attention": _attention, "latent_attention": _latent,
               "latent_attention_2": lambda cfg, m, p: _latent(cfg, m.latent, p, rotated=m)}


def _norm(cfg, weight):
    return PartSpec("dynamic_tanh", {"size": cfg.hidden_size, "weight": weight, "eps": cfg.norm_eps})


def _schedule(cfg):
    n, loop = len(cfg.layers), cfg.loop
    if loop is None:
        return [ScheduleEntry(i) for i in range(n)]
    passes = [ScheduleEntry(i, starts_pass=t if i == loop.start else None)
              for t in range(loop.times) for i in range(loop.start, loop.stop)]
    return [ScheduleEntry(i) for i in range(loop.start)] + passes + [ScheduleEntry(i) for i in range(loop.stop, n)]


def build_spec(cfg):
    layers = []
    for i, layer in enumerate(cfg.layers):
        norms = {"before_mixer": _norm(cfg, f"l{i}.norm1"), "after_mixer": _norm(cfg, f"l{i}.norm1b")}
        ffn = None
        if layer.ff is not None:
            norms.update(before_ff=_norm(cfg, f"l{i}.norm2"), after_ff=_norm(cfg, f"l{i}.norm2b"))
            ffn = PartSpec("swiglu", {"hidden_size": cfg.hidden_size, "intermediate_size": layer.ff, "activation": "relu",
                                      "names": {k: f"l{i}.mlp.{k}" for k in ("gate", "up", "down")}})
        mixer = MIXER_SPECS[layer.type](cfg, layer.mixer, f"l{i}.mix.")
        layers.append(LayerSpec(PartSpec("sandwich"), mixer, ffn, norms))
    pass_input = None
    if cfg.loop is not None:
        pass_input = PartSpec("step_and_embedding", {"hidden_size": cfg.hidden_size, "passes": cfg.loop.times, "weight": "loop.step"})
    return ModelSpec(
        hidden_size=cfg.hidden_size, vocab_size=cfg.vocab_size, max_positions=cfg.max_position_embeddings,
        embedding=PartSpec("table", {"vocab_size": cfg.vocab_size, "hidden_size": cfg.hidden_size, "weight": "embed",
                                     "scale": cfg.embedding_scale}),
        layers=layers, schedule=_schedule(cfg), final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear", {"vocab_size": cfg.vocab_size, "hidden_size": cfg.hidden_size, "weight": "head",
                                 "tied_to_embedding": False, "softcap": cfg.logit_softcap}),
        eos_token_id=cfg.eos_token_id, pass_input=pass_input)


ARCHITECTURE = register_architecture("Mutedra", MutedraConfig, build_spec, model_types=("mutedra",))
