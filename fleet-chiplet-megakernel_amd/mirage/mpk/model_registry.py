"""Which graph-builder class serves which model name (reference: python/mirage/mpk/model_registry.py)."""
_MODEL_BUILDERS = {}


def register_model_builder(*names):
    """Class decorator.  Takes the model names one by one or as a single list / tuple / set of them.  Names a config.json
    calls its architecture by are registered the same way."""
    if len(names) == 1 and not isinstance(names[0], str):
        names = tuple(names[0])

    def bind(builder_cls):
        _MODEL_BUILDERS.update(dict.fromkeys(names, builder_cls))
        return builder_cls

    return bind


def get_builder(name: str):
    try:
        return _MODEL_BUILDERS[name]
    except KeyError:
        raise ValueError(f"no graph builder is registered for model {name!r} (known: {sorted(_MODEL_BUILDERS)})") from None


def model_name_of(config: dict) -> str:
    """The registered name a parsed config.json asks for: its "architecture", or the first known entry of the Hugging Face
    list "architectures"."""
    names = [config["architecture"]] if config.get("architecture") else list(config.get("architectures") or [])
    for name in names:
        if name in _MODEL_BUILDERS:
            return name
    raise ValueError(f"config.json names no known architecture: {names} (known: {sorted(_MODEL_BUILDERS)})")
