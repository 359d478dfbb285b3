"""Figalorn as data: which parts each layer has and what its tensors are called.

A layer is the "prenorm" arrangement, x += mixer(norm1(x)), then, where the layer has a feed-forward,
x += ff(norm2(x)); the norms are RMS norms whose weights are stored around zero. The mixer is the part "attention",

  "attention": as the difference of two maps a head over the same values, with biases on q, k and v, neighbouring pairs
      that turn at rates scaled by their wavelength, keys seen within the query's own chunk of positions, and a gate an
      entry;
  "attention_2": with values that are the keys before norm and rotation, a norm a head whose weights all heads share,
      halves that turn at rates scaled by a ramp over the pairs, capped scores and a window.

The feed-forward is "up_down" with the exact gelu. The configuration's loop is a matter of the schedule: it names the
looped layers once a pass, every run with a cache entry of its own, and marks where a pass starts, the first one
included ("joined_projection" says what the stream becomes there). The head is a matrix of its own. Tensors are stored
under short names: `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.<name>`, `l<i>.mlp.<name>`, `embed`, `loop.in`, `final.norm`,
`head`.
"""
from ..config import register_architecture
from ..config.figalorn import FigalornConfig
from ..parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry


def _position(kind, rot):
    if rot is None:
        return PartSpec("none")
    scaling = None if rot.scaling is None else tuple(v for _, v in rot.scaling)
    return PartSpec(kind, {"theta": rot.base, "rotary_dims": rot.dims, "scaling": scaling})


def _attention(cfg, m, p, names, **more):
    return PartSpec("attention", {"hidden_size": cfg.hidden_size, "num_heads": m.heads, "num_kv_heads": m.kv_heads,
                                  "head_dim": m.dim, "value_dim": m.vdim, "eps": cfg.norm_eps, "scale": m.scale,
                                  "names": {k: p + v for k, v in names.items()}, **more})


def _difference(cfg, m, p):
    names = {k: k for k in ("q", "k", "v", "o", "g", "lq1", "lk1", "lq2", "lk2")}
    names.update(q_bias="q.b", k_bias="k.b", v_bias="v.b")
    return _attention(cfg, m, p, names, position=_position("rope_pairs", m.rot), qk_norm=False, bias="qkv", gate=True,
                      difference=m.diff, chunk=m.size)


def _key_value(cfg, m, p):
    names = {"q": "q", "k": "k", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm"}
    return _attention(cfg, m, p, names, position=_position("rope_halves", m.rot), qk_norm=True, keys_are_values=True,
                      softcap=m.softcap, window=m.size)


MIXER_SPECS = {"attention": _difference, "attention_2": _key_value}


def _norm(cfg, weight):
    return PartSpec("rmsnorm", {"size": cfg.hidden_size, "eps": cfg.norm_eps, "weight": weight, "offset": 1.0})


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
        norms = {"input": _norm(cfg, f"l{i}.norm1")}
        ffn = None
        if layer.ff is not None:
            norms["post_mixer"] = _norm(cfg, f"l{i}.norm2")
            ffn = PartSpec("up_down", {"hidden_size": cfg.hidden_size, "intermediate_size": layer.ff, "activation": "gelu",
                                       "names": {k: f"l{i}.mlp.{k}" for k in ("up", "down")}})
        layers.append(LayerSpec(PartSpec("prenorm"), MIXER_SPECS[layer.type](cfg, layer.mixer, f"l{i}.mix."), ffn, norms))
    pass_input = None
    if cfg.loop is not None:
        pass_input = PartSpec("joined_projection", {"hidden_size": cfg.hidden_size, "weight": "loop.in"})
    return ModelSpec(
        hidden_size=cfg.hidden_size, vocab_size=cfg.vocab_size, max_positions=cfg.max_position_embeddings,
        embedding=PartSpec("table", {"vocab_size": cfg.vocab_size, "hidden_size": cfg.hidden_size, "weight": "embed"}),
        layers=layers, schedule=_schedule(cfg), final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear", {"vocab_size": cfg.vocab_size, "hidden_size": cfg.hidden_size, "weight": "head",
                                 "tied_to_embedding": False}),
        eos_token_id=cfg.eos_token_id, pass_input=pass_input)


ARCHITECTURE = register_architecture("Figalorn", FigalornConfig, build_spec, model_types=("figalorn",))
