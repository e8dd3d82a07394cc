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

	// Per row: v = x + norm(sub) sub_w (v = x without sub), v -> x_out if given, norm(v) norm_w (v without norm_w) -> out
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
		int share = 1;                 // query heads that read the same key/value head (expanded form only)
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
	// Attention of a prompt's rows over keys and values as they are: head h reads k[r] = kv[r, g k_head ..] and
	// values kv[r, v_first + g v_head ..], g = h / share, of positions key_base + r; query row i is position
	// q_base + i.  Heads that start on whole 16-byte pieces run on the matrix cores; behind a head's last key
	// element there must then be finite numbers up to the end of its last piece.
	struct WindowAttn
	{
		LatentShape shape;
		const float* q = nullptr;
		int ldq = 0;
		const void* kv = nullptr; // T
		int ldkv = 0, v_first = 0;
		size_t k_head = 0, v_head = 0;
		int kv_first = 0, kv_ring = 0; // kv_ring > 0: key row r lives at (kv_first + r) modulo kv_ring, keys <= kv_ring
		int keys = 0, key_base = 0, rows = 0, q_base = 0;
		const float* gate = nullptr;
		int ldg = 0;
		float out_scale = 1.0f;
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

	// ---- attention whose query heads share key/value heads (mixers.hip) -----------------------------
	// Rotary positions on the first `dims` entries of a head: entry i is paired with entry i + dims / 2.
	struct Rotary
	{
		int dims = 0;
		const double* turns = nullptr; // [dims / 2] turns per position
	};
	// Per key/value head a ring of rows, one per position (position p in row p mod ring): the key, then the
	// value, each padded with zeros to whole 16-byte pieces (allocate zeroed; the padding is never written).
	struct HeadCache
	{
		void* rows = nullptr; // T [heads, ring, row_pitch]
		int ring = 0, heads = 0, dim = 0, vdim = 0;
		bool f32 = false;
		__host__ __device__ int key_pitch() const { return (dim + 7) & ~7; }
		__host__ __device__ int value_pitch() const { return (vdim + 7) & ~7; }
		__host__ __device__ int row_pitch() const { return key_pitch() + value_pitch(); }
		__host__ __device__ size_t head_stride() const { return static_cast<size_t>(ring) * row_pitch(); }
		size_t elements() const { return head_stride() * heads; }
	};
	// Queries and keys are normalised as whole projections (where norm weights are given), rotated, and keys
	// and values appended to the cache.
	struct GroupedAttn
	{
		int heads = 0;             // of queries; head h reads the cache's head h / (heads / cache.heads)
		int window = 0;            // positions a query sees, itself included
		float scale = 1.0f;
		Rotary rot;
		const float *q_norm = nullptr, *k_norm = nullptr; // [heads dim], [cache.heads dim], or both null
		float eps = 0.0f;
		HeadCache cache;
		// columns of one buffer; v may be k.  These and the norms start on 16-byte pieces and are readable up to whole ones.
		const float *q = nullptr, *k = nullptr, *v = nullptr;
		int ld = 0;
		int rows = 1;
		Position pos;
		// many rows
		float* q_out = nullptr;    // [rows, ldq]
		int ldq = 0;
		// one row
		float* partial = nullptr;  // scratch: grouped_step_partial_floats()
		int splits = 1;
	};
	int grouped_max_dim();
	void launch_grouped_append(const GroupedAttn& a, hipStream_t s);
	WindowAttn grouped_window(const GroupedAttn& a, int past); // the rest of a prompt's attention, for launch_window_attn
	int grouped_step_splits(int heads, int kv_heads, int dim, int vdim, int window);
	size_t grouped_step_partial_floats(int heads, int vdim, int splits);

	// ---- state-space recurrence with a decay per head (mixers.hip) -----------------------------------
	// S_t = exp(-exp(a_log) dt_t) S_(t-1) + dt_t B_t x_t^T, y_t = S_t^T C_t + d x_t, with dt = softplus(raw + dt_bias)
	// and x, B, C behind a causal convolution per channel and silu.  The last inputs of the convolution live in a
	// ring of `taps` rows (position p in row p mod taps).
	struct Ssm
	{
		int heads = 0, vdim = 0, state = 0, groups = 0, taps = 0;
		const float* conv_w = nullptr; // [taps, channels], the last row meets the current token
		const float *conv_b = nullptr, *dt_bias = nullptr, *a_log = nullptr, *d = nullptr;
		float* in = nullptr;           // [rows, ld]: z | x | B | C | dt
		int ld = 0;
		float* states = nullptr;       // [heads, state, ssm_state_pitch(vdim)]
		float* ring = nullptr;         // [taps, channels]
		int rows = 1;
		Position pos;
		// one row: y [heads vdim]
		float* y = nullptr;
		// many rows: y silu(z) takes the place of z
		float* xbc = nullptr;          // scratch [rows, ssm_ldx()]
		float* steps = nullptr;        // scratch [2, rows, heads]: dt, then log decays in units of log 2
		float* chunk_states = nullptr; // scratch: ssm_chunk_floats()
		__host__ __device__ int inner() const { return heads * vdim; }
		__host__ __device__ int channels() const { return heads * vdim + 2 * groups * state; }
		__host__ __device__ int ldx() const { return (channels() + 3) & ~3; }
		__host__ __device__ int columns() const { return inner() + channels() + heads; }
	};
	__host__ __device__ inline int ssm_state_pitch(int vdim) { return (vdim + 3) & ~3; }
	int ssm_max_state();
	size_t ssm_chunk_floats(int rows, const Ssm& shape);
	void launch_ssm_rows(const Ssm& a, hipStream_t s);

	// out = scale w norm(y silu(z)), in `parts` equal parts with a root mean square of their own (z null: y alone)
	struct GatedNorm
	{
		const float *y = nullptr, *z = nullptr;
		int ldy = 0, ldz = 0, width = 0, parts = 1;
		const float* norm_w = nullptr;
		float eps = 0.0f, scale = 1.0f;
		void* out = nullptr; // T
		int ldo = 0, rows = 1;
		bool f32 = true;     // T = float
	};
	void launch_gated_norm(const GatedNorm& a, hipStream_t s);

	// One token: the attention's splits and the recurrence, which depend on the same projections only, in one
	// launch; then what both still need (merge of the splits times out_scale, gated norm) in another.  Either may
	// be null.
	void launch_mixer_step(const GroupedAttn* attn, const Ssm* ssm, hipStream_t s);
	void launch_mixer_finish(const GroupedAttn* attn, float out_scale, float* out, const GatedNorm* norm, hipStream_t s);
} // namespace litenn_hip
