import sys

from .replay import generate_main

sys.exit(generate_main())
