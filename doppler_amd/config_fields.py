"""Reading of a design's config.json: fields that must be there, fields that may, and nothing else."""


class ConfigError(ValueError):
    pass


def take(obj, where, required, optional=()):
    if not isinstance(obj, dict):
        raise ConfigError("%s must be an object, got %r" % (where, obj))
    unknown = sorted(set(obj) - set(required) - set(optional))
    if unknown:
        raise ConfigError("%s has keys this design does not have: %s" % (where, ", ".join(unknown)))
    missing = sorted(set(required) - set(obj))
    if missing:
        raise ConfigError("%s lacks %s" % (where, ", ".join(missing)))
    return obj


def count(obj, key, where, low=1):
    v = obj[key]
    if isinstance(v, bool) or not isinstance(v, int) or v < low:
        raise ConfigError("%s.%s must be an integer of at least %d, got %r" % (where, key, low, v))
    return v


def number(obj, key, where, positive=False):
    v = obj[key]
    if isinstance(v, bool) or not isinstance(v, (int, float)) or (positive and not v > 0):
        raise ConfigError("%s.%s must be a %snumber, got %r" % (where, key, "positive " if positive else "", v))
    return float(v)
