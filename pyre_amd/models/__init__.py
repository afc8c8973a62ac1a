"""Built-in architectures; importing this package registers them."""

from pyre_amd.models import durelix, mafurax, nurasun, pinozen, qwen2, rukosun, zorulix  # noqa: F401
