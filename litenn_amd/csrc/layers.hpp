// Layer mechanisms of the layered decoder (see layers.hip): launchers over device buffers.  Rows of
// Float32 buffers are `ld*` elements apart; T below is the operand type, bfloat16 (raw bits) or float.
#pragma once

#include "dense.hpp"

namespace litenn_hip
{
	// position of row r: (dev ? *dev : 0) + add + r
	struct Position
	{
		const int* dev = nullptr;
		int add = 0;
	};

	// x[r] = table[ids[r]] (+ a sinusoidal position vector: sine on even entries, cosine on odd ones).
	// turns: [(width + 1) / 2] frequencies in turns per position, null without position vectors.
	void launch_embed_rows(const DenseMatrix& table, const int32_t* ids, int rows, const double* turns, Position pos,
	                       float* x, int* err, hipStream_t s);

	// Per row: v = x + norm(sub) sub_w (v = x without sub), v -> x_out if given, norm(v) norm_w -> out
	struct AddNorm
	{
		const float* x = nullptr;
		int ldx = 0;
		const float* sub = nullptr;
		int ldsub = 0;
		int sub_parts = 1; // sub is the sum of so many buffers, sub_stride floats apart
		size_t sub_stride = 0;
		const float* sub_w = nullptr;
		float* x_out = nullptr; // may be x; rows ldx apart
		const float* norm_w = nullptr;
		void* out = nullptr; // T
		int ldo = 0;
		int rows = 0, width = 0;
		float eps = 0.0f;
		bool f32 = false; // T = float
	};
	void launch_add_norm(const AddNorm& a, hipStream_t s);

	// ---- attention over a latent cache ------------------------------------------------------------
	// A cache holds one row per position in a ring of `ring` rows: position p lives in row p mod ring.
	struct LatentCache
	{
		void* rows = nullptr; // T [ring, pitch]
		int ring = 0, rank = 0, pitch = 0;
		bool f32 = false;
	};
	struct LatentShape
	{
		int heads = 0, dim = 0, vdim = 0;
		int window = 0;                // positions a query sees, itself included
		float scale = 1.0f;
		const float* sink = nullptr;   // [heads] or null: joins the denominator, unscaled, once
	};
	// norm(src[r]) norm_w -> the cache row of position pos + r
	void launch_latent_append(const float* src, int ld, const float* norm_w, float eps, int rows, Position pos,
	                          const LatentCache& cache, hipStream_t s);
	// The same attention for few rows without expanding the cache: queries are taken into the latent
	// space (W_uk^T q), attend to the cached rows themselves, and the result is taken through W_uv.
	struct LatentStep
	{
		LatentShape shape;
		LatentCache cache;
		DenseMatrix uk, uv;            // [heads dim, rank], [heads vdim, rank]
		const float* q = nullptr;      // [rows, ldq]
		int ldq = 0;
		const float* latent = nullptr; // un-normalised latents to append first, or null
		int ldl = 0;
		const float* latent_w = nullptr;
		float eps = 0.0f;
		const float* gate = nullptr;   // [rows, ldg] or null: times sigmoid(gate)
		int ldg = 0;
		void* out = nullptr;           // [rows, ldo], T
		int ldo = 0;
		bool out_f32 = true;
		int rows = 1;
		Position pos;
		float* absorbed = nullptr;     // scratch: rows heads pitch
		float* partial = nullptr;      // scratch: latent_step_partial_floats()
		int splits = 1;
	};
	int latent_step_splits(int heads, int rows, int window);
	size_t latent_step_partial_floats(int heads, int rows, int pitch, int splits);
	int latent_step_max_rank();
	void launch_latent_step(const LatentStep& a, hipStream_t s);
	// Expanded form for a prompt's rows: keys k[r] = kv[r, h dim ..], values kv[r, v_first + h vdim ..] of
	// positions key_base + r; query row i is position q_base + i.
	struct WindowAttn
	{
		LatentShape shape;
		const float* q = nullptr;
		int ldq = 0;
		const void* kv = nullptr; // T
		int ldkv = 0, v_first = 0;
		int keys = 0, key_base = 0, rows = 0, q_base = 0;
		const float* gate = nullptr;
		int ldg = 0;
		void* out = nullptr; // T
		int ldo = 0;
		bool f32 = false;
	};
	void launch_window_attn(const WindowAttn& a, hipStream_t s);

	// ---- gated linear attention -----------------------------------------------------------------
	struct GlaShape
	{
		int heads = 0, dim = 0, vdim = 0;
		float q_scale = 1.0f;
		float inv_tau = 1.0f;
	};
	__host__ __device__ inline int gla_state_pitch(int vdim) { return (vdim + 3) & ~3; }
	struct Gla
	{
		GlaShape shape;
		const float *q = nullptr, *k = nullptr, *v = nullptr, *gate = nullptr, *a1 = nullptr; // columns of one buffer
		int ld = 0;
		DenseMatrix a2;              // [heads dim, rank]
		const float* a2_bias = nullptr;
		float* state = nullptr;      // [heads, dim, gla_state_pitch(vdim)]
		int rows = 1;
		// one row: o [heads vdim] before the head norm
		float* o = nullptr;
		// many rows: head norm, silu gate -> out (T)
		const float* norm_w = nullptr;
		float eps = 0.0f;
		void* out = nullptr;
		int ldo = 0;
		bool f32 = false;
		float* log_decay = nullptr;    // scratch [rows, heads dim]
		float* chunk_states = nullptr; // scratch: gla_chunk_floats()
	};
	int gla_max_dim();
	int gla_max_vdim();
	size_t gla_chunk_floats(int rows, int heads, int dim, int vdim);
	void launch_gla_step(const Gla& a, hipStream_t s);
	void launch_gla_rows(const Gla& a, hipStream_t s);
} // namespace litenn_hip
