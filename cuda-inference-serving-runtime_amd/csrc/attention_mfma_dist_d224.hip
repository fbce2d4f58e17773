// Matrix-core attention whose scores fall with the distance, heads of up to 224 coordinates (see attention_mfma.inc).
#define ATTN_DISTANCE
#define DPAD 224
#include "attention_mfma.inc"
