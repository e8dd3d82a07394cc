// The token loops shared by every decoder of the library (see decoder.hpp): evaluation of a run of
// tokens in passes, and the greedy loop that stays on the device, its single-token step captured
// once into a HIP graph whose replays read their position from device memory.
#include "decoder.hpp"

#include <algorithm>
#include <cstdlib>

namespace litenn_hip
{
	size_t argmax_step_scratch_bytes(size_t n);
	void launch_argmax_step(const float* x, size_t n, void* scratch, int32_t* next, int* counters, int past_inc,
	                        int32_t* out, hipStream_t s);

	namespace
	{
		// counters[0] = past length, counters[1] = tokens emitted so far, counters[2] = steps this model
		// has run (never reset: it names a step in the values its workgroups hand to each other)
		__global__ void set_counters_kernel(int* counters, int past, int emitted)
		{
			counters[0] = past;
			counters[1] = emitted;
			counters[2] += 1;
		}

		constexpr int kWaitRanOut = -2;

		int check_error_flag(litenn_hip_model* m)
		{
			int flag = 0;
			LITENN_HIP_TRY(m->action, hipMemcpyAsync(&flag, m->d_err, sizeof(int), hipMemcpyDeviceToHost, m->stream));
			LITENN_HIP_TRY(m->action, hipStreamSynchronize(m->stream));
			if (flag)
			{
				const int zero = 0;
				(void)hipMemcpy(m->d_err, &zero, sizeof(int), hipMemcpyHostToDevice);
				if (flag & 2)
				{
					return kWaitRanOut;
				}
				return fail(m->action, "GetRows index out of range");
			}
			return 0;
		}

		int ensure_base(litenn_hip_model* m, size_t rows, size_t logit_rows)
		{
			if (m->ensure_rows(rows) != 0)
			{
				return 1;
			}
			if (rows > m->cap_tokens)
			{
				if (m->d_tokens)
				{
					(void)hipFree(m->d_tokens);
					m->d_tokens = nullptr;
					m->cap_tokens = 0;
				}
				LITENN_HIP_TRY(m->action, hipMalloc(reinterpret_cast<void**>(&m->d_tokens), sizeof(int32_t) * rows));
				m->cap_tokens = rows;
			}
			if (logit_rows > m->cap_logit_rows)
			{
				decoder_drop_graph(m);
				if (m->logits)
				{
					(void)hipFree(m->logits);
					m->logits = nullptr;
					m->cap_logit_rows = 0;
				}
				LITENN_HIP_TRY(m->action, hipMalloc(reinterpret_cast<void**>(&m->logits),
				                                    sizeof(float) * logit_rows * static_cast<size_t>(m->vocab)));
				m->cap_logit_rows = logit_rows;
			}
			return 0;
		}

		int check_call(litenn_hip_model* m, const int32_t* tokens, size_t n, size_t positions)
		{
			if (m->state_lost)
			{
				return fail(m->action, "an earlier pass failed half-way: reset the model first");
			}
			if (static_cast<size_t>(m->past) + positions > static_cast<size_t>(m->context_length))
			{
				return fail(m->action, "context length exceeded");
			}
			if (m->check_complete() != 0)
			{
				return 1;
			}
			for (size_t i = 0; i < n; ++i)
			{
				if (tokens[i] < 0 || tokens[i] >= m->vocab)
				{
					return fail(m->action, "GetRows index out of range"); // Device.h:868-871
				}
			}
			return 0;
		}
	} // namespace

	hipError_t decoder_init(litenn_hip_model* m)
	{
		// Non-blocking: a stream that synchronises with the legacy default stream would, while its
		// decode step is being captured, make every default-stream call of another host thread fail
		// ("would make the legacy stream depend on a capturing blocking stream").
		hipError_t e = hipStreamCreateWithFlags(&m->stream, hipStreamNonBlocking);
		if (e != hipSuccess)
		{
			m->stream = nullptr;
			return e;
		}
		if ((e = hipMalloc(reinterpret_cast<void**>(&m->d_counters), 4 * sizeof(int))) != hipSuccess ||
		    (e = hipMalloc(reinterpret_cast<void**>(&m->d_err), sizeof(int))) != hipSuccess ||
		    (e = hipMalloc(reinterpret_cast<void**>(&m->d_next), sizeof(int32_t))) != hipSuccess ||
		    (e = hipMemsetAsync(m->d_counters, 0, 4 * sizeof(int), m->stream)) != hipSuccess ||
		    (e = hipMemsetAsync(m->d_err, 0, sizeof(int), m->stream)) != hipSuccess ||
		    (e = hipMemsetAsync(m->d_next, 0, sizeof(int32_t), m->stream)) != hipSuccess)
		{
			return e;
		}
		return hipMalloc(&m->argmax_scratch, argmax_step_scratch_bytes(static_cast<size_t>(m->vocab)));
	}

	void decoder_drop_graph(litenn_hip_model* m)
	{
		if (m->step_exec)
		{
			(void)hipGraphExecDestroy(m->step_exec);
			m->step_exec = nullptr;
		}
		if (m->step_graph)
		{
			(void)hipGraphDestroy(m->step_graph);
			m->step_graph = nullptr;
		}
	}

	int decoder_reset(litenn_hip_model* m)
	{
		DeviceGuard guard(m->dev);
		if (!guard.ok())
		{
			return fail_hip(m->action, guard.error());
		}
		if (m->reset_state() != 0)
		{
			return 1;
		}
		m->past = 0;
		m->state_lost = false;
		return 0;
	}

	int decoder_eval(litenn_hip_model* m, const int32_t* tokens, size_t rows, const int32_t* want, size_t n_want,
	                 float* out, float* last_logits, unsigned flags)
	{
		if (rows == 0)
		{
			return fail(m->action, "sequence length must be positive");
		}
		if (check_call(m, tokens, rows, rows) != 0)
		{
			return 1;
		}
		flags |= m->base_flags;
		// (row, place in out) in row order
		std::vector<std::pair<size_t, size_t>> picks;
		if (out)
		{
			const size_t n = want ? n_want : rows;
			picks.reserve(n);
			for (size_t i = 0; i < n; ++i)
			{
				if (want && (want[i] < 0 || static_cast<size_t>(want[i]) >= rows))
				{
					return fail(m->action, "a wanted row lies outside the run of tokens");
				}
				picks.emplace_back(want ? static_cast<size_t>(want[i]) : i, i);
			}
			std::sort(picks.begin(), picks.end());
		}
		DeviceGuard guard(m->dev);
		if (!guard.ok())
		{
			return fail_hip(m->action, guard.error());
		}
		hipStream_t s = m->stream;
		const size_t vocab = static_cast<size_t>(m->vocab);
		const size_t pass = std::min(rows, m->pass_rows());
		size_t next_pick = 0;
		for (size_t first = 0; first < rows; first += pass)
		{
			const size_t count = std::min(pass, rows - first);
			size_t pick_end = next_pick;
			while (pick_end < picks.size() && picks[pick_end].first < first + count)
			{
				++pick_end;
			}
			const size_t logit_rows = pick_end > next_pick ? first + count - picks[next_pick].first : 1;
			if (ensure_base(m, pass, logit_rows) != 0)
			{
				return 1;
			}
			m->prepare();
			const size_t first_logit = first + count - logit_rows; // row of the run that logits[0] belongs to
			for (int attempt = 0;; ++attempt)
			{
				m->state_lost = m->stateful(); // until the pass is known to have run
				LITENN_HIP_TRY(m->action, hipMemcpyAsync(m->d_tokens, tokens + first, sizeof(int32_t) * count,
				                                         hipMemcpyHostToDevice, s));
				set_counters_kernel<<<1, 1, 0, s>>>(m->d_counters, m->past, 0);
				m->forward(m->d_tokens, count, logit_rows, flags, m->past);
				LITENN_HIP_TRY(m->action, hipGetLastError());
				for (size_t i = next_pick; i < pick_end;)
				{
					// consecutive rows that land in consecutive places travel together
					size_t j = i + 1;
					while (j < pick_end && picks[j].first == picks[i].first + (j - i) && picks[j].second == picks[i].second + (j - i))
					{
						++j;
					}
					LITENN_HIP_TRY(m->action,
					               hipMemcpyAsync(out + picks[i].second * vocab, m->logits + (picks[i].first - first_logit) * vocab,
					                              sizeof(float) * vocab * (j - i), hipMemcpyDeviceToHost, s));
					i = j;
				}
				if (last_logits && first + count == rows)
				{
					LITENN_HIP_TRY(m->action, hipMemcpyAsync(last_logits, m->logits + (logit_rows - 1) * vocab,
					                                         sizeof(float) * vocab, hipMemcpyDeviceToHost, s));
				}
				const int rc = check_error_flag(m);
				if (rc == kWaitRanOut && attempt == 0 && m->give_up_waiting())
				{
					continue; // and once more through the other form
				}
				if (rc != 0)
				{
					return rc == kWaitRanOut ? fail(m->action, "a wait inside the decoder step ran out") : 1;
				}
				break;
			}
			m->state_lost = false;
			m->past += static_cast<int>(count);
			next_pick = pick_end;
		}
		return 0;
	}

	int decoder_generate(litenn_hip_model* m, const int32_t* prompt, size_t n_prompt, size_t n_new, int32_t* out_tokens,
	                     unsigned flags, double* prefill_ms, double* decode_ms)
	{
		if (n_prompt == 0 || n_new == 0)
		{
			return fail(m->action, "prompt and generation lengths must be positive");
		}
		if (check_call(m, prompt, n_prompt, n_prompt + n_new - 1) != 0)
		{
			return 1;
		}
		flags |= m->base_flags;
		DeviceGuard guard(m->dev);
		if (!guard.ok())
		{
			return fail_hip(m->action, guard.error());
		}
		const size_t pass = std::min(n_prompt, m->pass_rows());
		if (ensure_base(m, pass, 1) != 0)
		{
			return 1;
		}
		m->prepare();
		if (n_new > m->cap_out)
		{
			decoder_drop_graph(m);
			if (m->d_out)
			{
				(void)hipFree(m->d_out);
				m->d_out = nullptr;
				m->cap_out = 0;
			}
			LITENN_HIP_TRY(m->action, hipMalloc(reinterpret_cast<void**>(&m->d_out), sizeof(int32_t) * n_new));
			m->cap_out = n_new;
		}
		hipStream_t s = m->stream;
		// the events exist before any work is queued and are destroyed on every way out
		hipEvent_t ev[3] = { nullptr, nullptr, nullptr };
		auto cleanup = [&]() {
			for (hipEvent_t& e : ev)
			{
				if (e)
				{
					(void)hipEventDestroy(e);
					e = nullptr;
				}
			}
		};
		for (hipEvent_t& e : ev)
		{
			const hipError_t ce = hipEventCreate(&e);
			if (ce != hipSuccess)
			{
				e = nullptr;
				cleanup();
				return fail_hip(m->action, ce);
			}
		}
		// A failure part-way leaves `past` as it was: the rows a failed run appended lie beyond it, are
		// never read (every pass takes its position from `past`) and are overwritten by the next call;
		// a model with recurrent state asks for a reset instead.  The stream is drained first so that
		// nothing of the failed run is still in flight afterwards.
		m->state_lost = m->stateful();
#define GEN_TRY(expr)                                                                                                  \
	do                                                                                                                 \
	{                                                                                                                  \
		const hipError_t e_ = (expr);                                                                                  \
		if (e_ != hipSuccess)                                                                                          \
		{                                                                                                              \
			(void)hipStreamSynchronize(s);                                                                             \
			cleanup();                                                                                                 \
			return fail_hip(m->action, e_);                                                                            \
		}                                                                                                              \
	} while (0)

		// prompt: passes over n_prompt rows, logits of the last row only, first token from its arg-max
		for (size_t first = 0; first < n_prompt; first += pass)
		{
			const size_t count = std::min(pass, n_prompt - first);
			const int past = m->past + static_cast<int>(first);
			GEN_TRY(hipMemcpyAsync(m->d_tokens, prompt + first, sizeof(int32_t) * count, hipMemcpyHostToDevice, s));
			set_counters_kernel<<<1, 1, 0, s>>>(m->d_counters, past, 0);
			if (first == 0)
			{
				GEN_TRY(hipEventRecord(ev[0], s)); // the first pass's ids are on their way: the clock starts here
			}
			m->forward(m->d_tokens, count, 1, flags, past);
			if (first + count == n_prompt)
			{
				launch_argmax_step(m->logits, m->vocab, m->argmax_scratch, m->d_next, m->d_counters,
				                   static_cast<int>(count), m->d_out, s);
			}
		}
		GEN_TRY(hipEventRecord(ev[1], s));
		GEN_TRY(hipGetLastError());

		// single-token steps: embed d_next at position counters[0], arg-max, append.  The step is
		// captured once; every replay reads its position from device memory.
		const char* graph_env = getenv("LITENN_HIP_GRAPH");
		const bool use_graph = !(graph_env && graph_env[0] == '0');
		const int step_past = m->past + static_cast<int>(n_prompt);
		if (n_new > 1)
		{
			if (use_graph && !m->step_exec)
			{
				GEN_TRY(hipStreamSynchronize(s));
				hipError_t ce = hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal);
				if (ce == hipSuccess)
				{
					m->forward(m->d_next, 1, 1, flags, step_past);
					launch_argmax_step(m->logits, m->vocab, m->argmax_scratch, m->d_next, m->d_counters, 1, m->d_out, s);
					ce = hipStreamEndCapture(s, &m->step_graph);
				}
				if (ce == hipSuccess)
				{
					ce = hipGraphInstantiate(&m->step_exec, m->step_graph, nullptr, nullptr, 0);
				}
				if (ce != hipSuccess)
				{
					decoder_drop_graph(m);
					cleanup();
					return fail_hip(m->action, ce);
				}
			}
			for (size_t i = 1; i < n_new; ++i)
			{
				if (use_graph)
				{
					GEN_TRY(hipGraphLaunch(m->step_exec, s));
				}
				else
				{
					m->forward(m->d_next, 1, 1, flags, step_past + static_cast<int>(i) - 1);
					launch_argmax_step(m->logits, m->vocab, m->argmax_scratch, m->d_next, m->d_counters, 1, m->d_out, s);
				}
			}
		}
		GEN_TRY(hipEventRecord(ev[2], s));
		GEN_TRY(hipGetLastError());
		GEN_TRY(hipMemcpyAsync(out_tokens, m->d_out, sizeof(int32_t) * n_new, hipMemcpyDeviceToHost, s));
		int step_flag = 0;
		GEN_TRY(hipMemcpyAsync(&step_flag, m->d_err, sizeof(int), hipMemcpyDeviceToHost, s));
		GEN_TRY(hipStreamSynchronize(s));
		if ((step_flag & 2) && m->give_up_waiting())
		{
			// the tokens are void; once more, from the prompt, through the other form (`past` has not moved)
			const int zero = 0;
			GEN_TRY(hipMemcpy(m->d_err, &zero, sizeof(int), hipMemcpyHostToDevice));
			cleanup();
			return decoder_generate(m, prompt, n_prompt, n_new, out_tokens, flags, prefill_ms, decode_ms);
		}
		float ms = 0.0f;
		if (prefill_ms)
		{
			GEN_TRY(hipEventElapsedTime(&ms, ev[0], ev[1]));
			*prefill_ms = ms;
		}
		if (decode_ms)
		{
			GEN_TRY(hipEventElapsedTime(&ms, ev[1], ev[2]));
			*decode_ms = ms;
		}
		cleanup();
#undef GEN_TRY
		// the last emitted token has not been fed back: the caches hold prompt + (n_new - 1) rows
		m->past += static_cast<int>(n_prompt + n_new - 1);
		m->state_lost = false;
		return 0;
	}

	void decoder_free(litenn_hip_model* m)
	{
		DeviceGuard guard(m->dev);
		if (m->stream)
		{
			(void)hipStreamSynchronize(m->stream);
		}
		delete m;
	}
} // namespace litenn_hip

litenn_hip_model::~litenn_hip_model()
{
	litenn_hip::decoder_drop_graph(this);
	for (void* ptr : owned)
	{
		(void)hipFree(ptr);
	}
	void* singles[] = { d_tokens, logits, argmax_scratch, d_next, d_out, d_counters, d_err };
	for (void* ptr : singles)
	{
		if (ptr)
		{
			(void)hipFree(ptr);
		}
	}
	if (stream)
	{
		(void)hipStreamDestroy(stream);
	}
}

// ---- the model-agnostic entry points ---------------------------------------------------------

using namespace litenn_hip;

extern "C" int litenn_hip_model_free(litenn_hip_model* m)
{
	if (m)
	{
		decoder_free(m);
	}
	return 0;
}

extern "C" int litenn_hip_model_reset(litenn_hip_model* m)
{
	return m ? decoder_reset(m) : fail("HIP model", "null argument");
}

extern "C" int litenn_hip_model_past(const litenn_hip_model* m)
{
	return m ? m->past : -1;
}

extern "C" int litenn_hip_model_get_info(const litenn_hip_model* m, litenn_hip_model_info* out)
{
	if (!m || !out)
	{
		return fail("HIP model", "null argument");
	}
	out->architecture = m->architecture.c_str();
	out->vocab_size = m->vocab;
	out->context_length = m->context_length;
	out->dtype = m->dtype;
	return 0;
}

extern "C" int litenn_hip_model_eval(litenn_hip_model* m, const int32_t* tokens, size_t count, const int32_t* want,
                                     size_t n_want, float* logits, unsigned flags)
{
	if (!m || !tokens || (want && n_want && !logits))
	{
		return fail("HIP model", "null argument");
	}
	return decoder_eval(m, tokens, count, want, n_want, want && n_want == 0 ? nullptr : logits, nullptr, flags);
}

extern "C" int litenn_hip_model_generate(litenn_hip_model* m, const int32_t* prompt, size_t n_prompt, size_t n_new,
                                         int32_t* out_tokens, unsigned flags, double* prefill_ms, double* decode_ms)
{
	if (!m || !prompt || !out_tokens)
	{
		return fail("HIP model", "null argument");
	}
	return decoder_generate(m, prompt, n_prompt, n_new, out_tokens, flags, prefill_ms, decode_ms);
}
