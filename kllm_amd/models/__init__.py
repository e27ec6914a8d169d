from . import llama  # registers "LlamaForCausalLM"
from . import nusilix  # registers "Nusilix"
from . import ribovik  # registers "Ribovik"
from . import natenex  # registers "Natenex"
from . import lugetar  # registers "Lugetar"
from . import puladra  # registers "Puladra"
from . import bevadra  # registers "Bevadra"

__all__ = ["llama", "nusilix", "ribovik", "natenex", "lugetar", "puladra", "bevadra"]
