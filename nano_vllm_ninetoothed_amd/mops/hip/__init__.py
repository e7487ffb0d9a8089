from . import attention_ops, mixture_ops, ops, recurrent_ops  # noqa: F401
