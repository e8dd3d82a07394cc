// What every resident decoder has whatever its layers are: the stream, the token and position
// buffers, the logits, the greedy arg-max state and the captured single-token step, with the two
// loops over them (decoder_eval, decoder_generate).  A model class derives from litenn_hip_model,
// keeps its own weights, caches and scratch, and supplies the pass over a run of tokens.
#pragma once

#include "common.hpp"

#include <string>
#include <vector>

struct litenn_hip_model
{
	int dev = 0;
	int vocab = 0;
	int context_length = 0;          // positions one sequence may hold
	int dtype = LITENN_F16;          // LITENN_F32: every operand of this model is 32-bit
	unsigned base_flags = 0;         // or-ed into the flags of every call
	const char* action = "HIP model"; // prefix of this model's error messages
	std::string architecture;
	hipStream_t stream = nullptr;
	size_t cap_tokens = 0;
	int32_t* d_tokens = nullptr;
	size_t cap_logit_rows = 0;
	float* logits = nullptr;
	void* argmax_scratch = nullptr; // per-chunk (value, index) pairs of the vocabulary arg-max
	int32_t* d_next = nullptr;      // token produced by the last arg-max
	int32_t* d_out = nullptr;       // generated tokens
	size_t cap_out = 0;
	int* d_counters = nullptr;      // {past, emitted, steps run}
	int* d_err = nullptr;
	std::vector<void*> owned;       // device buffers freed with the model
	int past = 0;
	bool state_lost = false;        // a pass failed half-way through a state that cannot be rolled back
	hipGraphExec_t step_exec = nullptr;
	hipGraph_t step_graph = nullptr;

	virtual ~litenn_hip_model();

	// 0, or non-zero with a message when a tensor is missing
	virtual int check_complete() = 0;
	// scratch for passes of up to `rows` tokens (logits and token ids are the base's)
	virtual int ensure_rows(size_t rows) = 0;
	// decisions that must be made before anything is queued or captured
	virtual void prepare() {}
	// the most tokens one pass may carry; longer prompts are fed in passes of this size
	virtual size_t pass_rows() const { return SIZE_MAX; }
	// true when a pass changes state that a repetition would change again
	virtual bool stateful() const { return false; }
	// Enqueues a pass over `rows` tokens whose ids are at `ids` (device), positions past .. past + rows - 1;
	// `past` is also in d_counters[0], and a captured pass (rows == 1) reads it only there.  The logits of
	// the last logit_rows (>= 1) rows go to `logits`.
	virtual void forward(const int32_t* ids, size_t rows, size_t logit_rows, unsigned flags, int past) = 0;
	// forgets a sequence's state beyond `past` (queued on the stream)
	virtual int reset_state() { return 0; }
	// A pass raised bit 2 of the error word (a bounded wait ran out).  True when the model has switched
	// to a form that cannot raise it and the pass may be repeated.
	virtual bool give_up_waiting() { return false; }
};

namespace litenn_hip
{
	// the base's buffers and stream; vocab, context_length, dev and action are set by the caller
	hipError_t decoder_init(litenn_hip_model* m);
	void decoder_drop_graph(litenn_hip_model* m);
	int decoder_reset(litenn_hip_model* m);
	// One run of tokens.  `want` lists n_want rows (each < rows) whose logits go to `out`
	// ([n_want, vocab]); null means every row.  last_logits (may be null) receives the last row's.
	int decoder_eval(litenn_hip_model* m, const int32_t* tokens, size_t rows, const int32_t* want, size_t n_want,
	                 float* out, float* last_logits, unsigned flags);
	int decoder_generate(litenn_hip_model* m, const int32_t* prompt, size_t n_prompt, size_t n_new, int32_t* out_tokens,
	                     unsigned flags, double* prefill_ms, double* decode_ms);
	// synchronises, destroys
	void decoder_free(litenn_hip_model* m);
} // namespace litenn_hip
