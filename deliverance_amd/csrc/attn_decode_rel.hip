// Decode attention with a bias by distance, a query temperature, chunks, a sink and a gate: the kernel of attn_decode.hip,
// compiled with these extras (see there).  Entry point: da_attn_decode_rel.
#define DEC_REL 1
#include "attn_decode.hip"
