from . import dumovik, fanulix, karopel, kudurax, lotelix, qwen3, verorax  # noqa: F401  (register the built-in architectures)
