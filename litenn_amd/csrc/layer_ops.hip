// C ABI of the layered decoder's mechanisms as single operators (include/litenn_hip.h, group 2b).
#include "layers.hpp"

using namespace litenn_hip;

namespace
{
	constexpr size_t kMaxExtent = size_t{ 1 } << 28;

	bool extent_ok(size_t n) { return n > 0 && n <= kMaxExtent; }

	DenseMatrix dense_of(const void* w, size_t n, size_t k, size_t pitch)
	{
		DenseMatrix m;
		m.w = static_cast<const uint16_t*>(w);
		m.n = static_cast<int>(n);
		m.k = static_cast<int>(k);
		m.pitch = static_cast<int>(pitch);
		return m;
	}
} // namespace

#define LAYER_GUARD(action, dev)                                                                                       \
	DeviceGuard guard(dev);                                                                                            \
	if (!guard.ok())                                                                                                   \
	{                                                                                                                  \
		return fail_hip(action, guard.error());                                                                        \
	}

extern "C" int litenn_hip_linear_bf16(int dev, const void* w, size_t n, size_t k, size_t pitch, const void* x, int x_dtype,
                                      size_t m, void* y, const litenn_hip_exec* opts)
{
	const char* action = "HIP linear";
	if (m == 0 || n == 0)
	{
		return 0;
	}
	if (!w || !x || !y)
	{
		return fail(action, "null operand");
	}
	if (!extent_ok(n) || !extent_ok(k) || !extent_ok(m) || pitch != static_cast<size_t>(dense_pitch(static_cast<int>(k))))
	{
		return fail(action, "rows must be k rounded up to a multiple of 64 apart");
	}
	if (x_dtype != LITENN_F32 && x_dtype != LITENN_BF16)
	{
		return fail(action, "activations must be Float32 or BFloat16");
	}
	LAYER_GUARD(action, dev);
	if (m == 1 && x_dtype == LITENN_F32)
	{
		DenseRow r;
		r.w = dense_of(w, n, k, pitch);
		r.x = static_cast<const float*>(x);
		r.y = static_cast<float*>(y);
		if (launch_dense_row(r, stream_of(opts)))
		{
			return finish(action, opts);
		}
	}
	DenseRows d;
	d.w = dense_of(w, n, k, pitch);
	d.a = x;
	d.lda = static_cast<int>(pitch);
	d.m = static_cast<int>(m);
	d.c = y;
	d.ldc = static_cast<int>(n);
	d.f32 = x_dtype == LITENN_F32;
	launch_dense_rows(d, stream_of(opts));
	return finish(action, opts);
}

extern "C" int litenn_hip_window_attn(int dev, const void* q, const void* kv, int dtype, size_t m, size_t keys,
                                      size_t heads, size_t dim, size_t vdim, const litenn_hip_window_attn_opts* o,
                                      void* out, const litenn_hip_exec* opts)
{
	const char* action = "HIP window attention";
	if (!q || !kv || !out || !o)
	{
		return fail(action, "null operand");
	}
	if (!extent_ok(m) || !extent_ok(keys) || !extent_ok(heads) || heads > 32768 || !extent_ok(dim) || dim > 1024 ||
	    !extent_ok(vdim) || vdim > 1024 || !extent_ok(o->window) || o->key_position > kMaxExtent ||
	    o->query_position > kMaxExtent)
	{
		return fail(action, "extent out of range");
	}
	if (dtype != LITENN_F32 && dtype != LITENN_BF16)
	{
		return fail(action, "keys and values must be Float32 or BFloat16");
	}
	// every row sees at least one key: its own position is among them
	if (o->query_position < o->key_position || o->query_position + m > o->key_position + keys)
	{
		return fail(action, "the keys must hold every query's own position");
	}
	WindowAttn a;
	a.shape.heads = static_cast<int>(heads);
	a.shape.dim = static_cast<int>(dim);
	a.shape.vdim = static_cast<int>(vdim);
	a.shape.window = static_cast<int>(o->window);
	a.shape.scale = static_cast<float>(o->scale);
	a.shape.sink = static_cast<const float*>(o->sinks);
	a.q = static_cast<const float*>(q);
	a.ldq = static_cast<int>(heads * dim);
	a.kv = kv;
	a.ldkv = static_cast<int>(heads * (dim + vdim));
	a.v_first = static_cast<int>(heads * dim);
	a.k_head = dim;
	a.v_head = vdim;
	a.keys = static_cast<int>(keys);
	a.key_base = static_cast<int>(o->key_position);
	a.rows = static_cast<int>(m);
	a.q_base = static_cast<int>(o->query_position);
	a.gate = static_cast<const float*>(o->gate);
	a.ldg = static_cast<int>(heads * vdim);
	a.out = out;
	a.ldo = static_cast<int>(heads * vdim);
	a.f32 = dtype == LITENN_F32;
	LAYER_GUARD(action, dev);
	launch_window_attn(a, stream_of(opts));
	return finish(action, opts);
}

extern "C" size_t litenn_hip_gla_workspace_bytes(size_t m, size_t heads, size_t dim, size_t vdim)
{
	if (!extent_ok(m) || !extent_ok(heads) || !extent_ok(dim) || !extent_ok(vdim))
	{
		return 0;
	}
	return sizeof(float) * (((m * heads * dim + 3) & ~size_t{ 3 }) + gla_chunk_floats(static_cast<int>(m), static_cast<int>(heads),
	                                                                 static_cast<int>(dim), static_cast<int>(vdim)));
}

extern "C" int litenn_hip_gla(int dev, const litenn_hip_gla_args* p, size_t m, void* state, void* out, int out_dtype,
                              void* workspace, size_t workspace_bytes, const litenn_hip_exec* opts)
{
	const char* action = "HIP gated linear attention";
	if (!p || !state || !out || !p->q || !p->k || !p->v || !p->low || !p->decay_w || !p->decay_bias)
	{
		return fail(action, "null operand");
	}
	if (!extent_ok(m) || !extent_ok(p->heads) || p->heads > 32768 || !extent_ok(p->dim) ||
	    p->dim > static_cast<size_t>(gla_max_dim()) || !extent_ok(p->vdim) || p->vdim > static_cast<size_t>(gla_max_vdim()) ||
	    p->rank == 0 || p->rank > 512 || !extent_ok(p->ld) || !(p->tau > 0.0))
	{
		return fail(action, "extent out of range");
	}
	const bool step = !p->head_norm;
	if (step ? m != 1 || out_dtype != LITENN_F32 : !p->gate || (out_dtype != LITENN_F32 && out_dtype != LITENN_BF16))
	{
		return fail(action, "one row without the head norm gives Float32, rows with it need a gate and give Float32 or BFloat16");
	}
	if (!step && (!workspace || workspace_bytes < litenn_hip_gla_workspace_bytes(m, p->heads, p->dim, p->vdim)))
	{
		return fail(action, "workspace too small");
	}
	Gla g;
	g.shape.heads = static_cast<int>(p->heads);
	g.shape.dim = static_cast<int>(p->dim);
	g.shape.vdim = static_cast<int>(p->vdim);
	g.shape.q_scale = static_cast<float>(p->q_scale);
	g.shape.inv_tau = static_cast<float>(1.0 / p->tau);
	g.q = static_cast<const float*>(p->q);
	g.k = static_cast<const float*>(p->k);
	g.v = static_cast<const float*>(p->v);
	g.gate = static_cast<const float*>(p->gate);
	g.a1 = static_cast<const float*>(p->low);
	g.ld = static_cast<int>(p->ld);
	g.a2 = dense_of(p->decay_w, p->heads * p->dim, p->rank, static_cast<size_t>(dense_pitch(static_cast<int>(p->rank))));
	g.a2_bias = static_cast<const float*>(p->decay_bias);
	g.state = static_cast<float*>(state);
	g.rows = static_cast<int>(m);
	g.norm_w = static_cast<const float*>(p->head_norm);
	g.eps = static_cast<float>(p->eps);
	LAYER_GUARD(action, dev);
	if (step)
	{
		g.o = static_cast<float*>(out);
		launch_gla_step(g, stream_of(opts));
		return finish(action, opts);
	}
	g.out = out;
	g.ldo = static_cast<int>(p->heads * p->vdim);
	g.f32 = out_dtype == LITENN_F32;
	g.log_decay = static_cast<float*>(workspace);
	g.chunk_states = g.log_decay + ((m * p->heads * p->dim + 3) & ~size_t{ 3 });
	launch_gla_rows(g, stream_of(opts));
	return finish(action, opts);
}
