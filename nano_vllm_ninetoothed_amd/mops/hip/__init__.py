from . import ops, recurrent_ops  # noqa: F401
