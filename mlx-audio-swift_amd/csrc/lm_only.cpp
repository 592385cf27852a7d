// lm_only.cpp - what libmi_speech_lm.so (make lm: the token engines alone, a fraction of the compile time) has in place of the codecs, the speech
// framing and the code-streaming GEMMs: entry points that refuse.  libmi_speech.so never links this file.
#include "kernels.h"
#include "lm_kernels.h"

[[noreturn]] static void absent() { throw MisError(MIS_ERR_NOT_INITIALIZED, "not in the language-model build of the library (libmi_speech_lm.so)"); }

void launch_orpheus_deinterleave(const int32_t*, int, int, int, int32_t*, int32_t*, int32_t*, int, hipStream_t) { absent(); }
void launch_orpheus_deinterleave_ragged(const int32_t*, int, const int32_t*, int, int32_t*, int32_t*, int32_t*, int, hipStream_t) { absent(); }
void launch_orpheus_parse_output(const int32_t*, const int32_t*, int, int, int32_t*, int32_t*, hipStream_t, const SpeechTokenIds*) { absent(); }
void snac_decode_device(mis_snac*, const int32_t* const*, int, int, const float* const*, int, uint64_t, const int32_t*, int64_t, float*, int64_t, hipStream_t) { absent(); }
int snac_device(const mis_snac*) { absent(); }
const mis_snac_config* snac_config(const mis_snac*) { absent(); }
extern "C" int64_t mis_snac_num_samples(const mis_snac*, int) { return 0; }
extern "C" int64_t mis_snac_noise_len(const mis_snac*, int, int) { return 0; }
void launch_gemm_skinny_q(int, int, int, int, const void*, const bf16_t*, const bf16_t*, void*, int, int, int, int, int, hipStream_t, const bf16_t*) { absent(); }
void launch_pack_qweight(int, const uint32_t*, const bf16_t*, const bf16_t*, void*, bf16_t*, int, int, int, int, hipStream_t) { absent(); }
