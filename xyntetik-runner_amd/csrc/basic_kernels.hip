// Element-wise and row-wise kernels of the forward pass, for float and bfloat16
// storage: embedding gather, RMSNorm, rotary position encoding fused with the
// write of keys and values into cache pages, SiLU-gate, residual add, fill.
// All arithmetic is 32-bit float; only loads and stores see the storage type.
#include "common.h"

// ---------------------------------------------------------------- embedding
// x[t] = table[id_t]; an id outside [0, V) reads row 0
// (src/model.c:6148-6162).
template <typename TW>
__global__ void k_embedding(float* __restrict__ out, const TW* __restrict__ table,
                            const int* __restrict__ ids, int E, int V, float scale) {
    int t = blockIdx.x;
    int id = ids[t];
    if (id < 0 || id >= V) id = 0;
    const TW* row = table + (size_t)id * E;
    float* o = out + (size_t)t * E;
    for (int i = threadIdx.x; i < E; i += blockDim.x) o[i] = ld<TW>(row, i) * scale;
}

// The same from a bfloat16 table in the matrix kernels' packed order (blocks of 16 rows x 32
// columns, 1 KB each, [row group][column block][row][column]): a model that ties its output
// head to the embedding then keeps the table once, in the order the head's product reads it.
__global__ void k_embedding_packed(float* __restrict__ out, const bf16_t* __restrict__ table,
                                   const int* __restrict__ ids, int E, int V, float scale) {
    int t = blockIdx.x;
    int id = ids[t];
    if (id < 0 || id >= V) id = 0;
    const size_t kblocks = (size_t)((E + 31) / 32);
    const bf16_t* grp = table + (size_t)(id >> 4) * kblocks * 512 + (id & 15) * 32;
    float* o = out + (size_t)t * E;
    for (int i = threadIdx.x; i < E; i += blockDim.x) o[i] = bf16_to_f32(grp[(size_t)(i >> 5) * 512 + (i & 31)]) * scale;
}

extern "C" int xr_embedding(float* out, const void* table, const int* ids, int T, int E, int V,
                            float scale, int table_dtype, int packed, hipStream_t stream) {
    XR_REQUIRE(T >= 0 && E > 0 && V > 0, "embedding: bad sizes T=%d E=%d V=%d", T, E, V);
    XR_REQUIRE(table_dtype == XR_F32 || table_dtype == XR_BF16, "embedding: bad dtype %d", table_dtype);
    XR_REQUIRE(!packed || table_dtype == XR_BF16, "embedding: a packed table is bfloat16");
    if (T == 0) return XR_OK;
    if (packed)
        k_embedding_packed<<<T, 256, 0, stream>>>(out, (const bf16_t*)table, ids, E, V, scale);
    else if (table_dtype == XR_F32)
        k_embedding<float><<<T, 256, 0, stream>>>(out, (const float*)table, ids, E, V, scale);
    else
        k_embedding<bf16_t><<<T, 256, 0, stream>>>(out, (const bf16_t*)table, ids, E, V, scale);
    XR_CHECK_LAUNCH("embedding");
    return XR_OK;
}

// ---------------------------------------------------------------- RMSNorm
// y_i = x_i * r * w_i with r = 1/sqrt(mean(x^2) + eps): eps inside the root, added to
// the mean; multiply order (x*r)*w (src/model.c:3386-3392).
template <typename TO, typename TW>
__global__ void k_rmsnorm(TO* __restrict__ out, const float* __restrict__ x, const TW* __restrict__ w,
                          const int* __restrict__ rows, int E, int ldx, float eps) {
    __shared__ float part[4];
    int r = blockIdx.x;
    int src = rows ? rows[r] : r;
    const float* xr = x + (size_t)src * ldx;
    float ss = 0.f;
    for (int i = threadIdx.x; i < E; i += blockDim.x) {
        float v = xr[i];
        ss += v * v;
    }
    ss = wave_sum(ss);
    int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    if (lane == 0) part[wave] = ss;
    __syncthreads();
    float tot = part[0] + part[1] + part[2] + part[3];
    float rinv = 1.0f / sqrtf(tot / (float)E + eps);
    TO* o = out + (size_t)r * E;
    if (w) {
        for (int i = threadIdx.x; i < E; i += blockDim.x) st<TO>(o, i, xr[i] * rinv * ld<TW>(w, i));
    } else {
        for (int i = threadIdx.x; i < E; i += blockDim.x) st<TO>(o, i, xr[i] * rinv);
    }
}

// Rows whose width is a multiple of 4 (up to 4 * 256 * RN_MAXV): every thread keeps its
// float4 pieces in registers between the sum and the scaling, and writes 4 values at a time.
#define RN_MAXV 8
template <typename TO> __device__ inline void st4(TO* p, size_t i, float a, float b, float c, float d);
template <> __device__ inline void st4<float>(float* p, size_t i, float a, float b, float c, float d) {
    *reinterpret_cast<float4*>(p + i) = make_float4(a, b, c, d);
}
template <> __device__ inline void st4<bf16_t>(bf16_t* p, size_t i, float a, float b, float c, float d) {
    uint2 w;
    w.x = (uint32_t)f32_to_bf16(a) | ((uint32_t)f32_to_bf16(b) << 16);
    w.y = (uint32_t)f32_to_bf16(c) | ((uint32_t)f32_to_bf16(d) << 16);
    *reinterpret_cast<uint2*>(p + i) = w;
}

template <typename TO, typename TW, int NV>
__global__ __launch_bounds__(256) void k_rmsnorm_v4(TO* __restrict__ out, const float* __restrict__ x,
                                                    const TW* __restrict__ w, const int* __restrict__ rows,
                                                    int E, int ldx, float eps) {
    __shared__ float part[4];
    const int r = blockIdx.x;
    const int src = rows ? rows[r] : r;
    const float4* xr = reinterpret_cast<const float4*>(x + (size_t)src * ldx);
    const int n4 = E >> 2;
    float4 v[NV];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = threadIdx.x + i * 256;
        v[i] = c < n4 ? xr[c] : make_float4(0.f, 0.f, 0.f, 0.f);
        ss += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
    }
    ss = wave_sum(ss);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float tot = part[0] + part[1] + part[2] + part[3];
    const float rinv = 1.0f / sqrtf(tot / (float)E + eps);
    TO* o = out + (size_t)r * E;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = threadIdx.x + i * 256;
        if (c >= n4) continue;
        float w0 = 1.f, w1 = 1.f, w2 = 1.f, w3 = 1.f;
        if (w) { w0 = ld<TW>(w, 4 * c); w1 = ld<TW>(w, 4 * c + 1); w2 = ld<TW>(w, 4 * c + 2); w3 = ld<TW>(w, 4 * c + 3); }
        st4<TO>(o, (size_t)4 * c, v[i].x * rinv * w0, v[i].y * rinv * w1, v[i].z * rinv * w2, v[i].w * rinv * w3);
    }
}

extern "C" int xr_rmsnorm(void* out, const float* x, const void* w, const int* rows, int R, int E,
                          int ldx, float eps, int out_dtype, int w_dtype, hipStream_t stream) {
    XR_REQUIRE(R >= 0 && E > 0 && ldx >= E, "rmsnorm: bad sizes R=%d E=%d ldx=%d", R, E, ldx);
    XR_REQUIRE(eps >= 0.f, "rmsnorm: eps %g is negative", eps);
    XR_REQUIRE((out_dtype == XR_F32 || out_dtype == XR_BF16) && (w_dtype == XR_F32 || w_dtype == XR_BF16),
               "rmsnorm: bad dtypes out=%d w=%d", out_dtype, w_dtype);
    if (R == 0) return XR_OK;
    const bool vec = E % 4 == 0 && ldx % 4 == 0 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)out % 16) == 0 &&
                     E <= 4 * 256 * RN_MAXV;
#define RN(TO, TW)                                                                                              \
    do {                                                                                                        \
        if (!vec) k_rmsnorm<TO, TW><<<R, 256, 0, stream>>>((TO*)out, x, (const TW*)w, rows, E, ldx, eps);        \
        else if (E <= 4 * 256 * 2) k_rmsnorm_v4<TO, TW, 2><<<R, 256, 0, stream>>>((TO*)out, x, (const TW*)w, rows, E, ldx, eps); \
        else if (E <= 4 * 256 * 4) k_rmsnorm_v4<TO, TW, 4><<<R, 256, 0, stream>>>((TO*)out, x, (const TW*)w, rows, E, ldx, eps); \
        else k_rmsnorm_v4<TO, TW, RN_MAXV><<<R, 256, 0, stream>>>((TO*)out, x, (const TW*)w, rows, E, ldx, eps); \
    } while (0)
    if (out_dtype == XR_F32 && w_dtype == XR_F32) RN(float, float);
    else if (out_dtype == XR_F32 && w_dtype == XR_BF16) RN(float, bf16_t);
    else if (out_dtype == XR_BF16 && w_dtype == XR_F32) RN(bf16_t, float);
    else RN(bf16_t, bf16_t);
#undef RN
    XR_CHECK_LAUNCH("rmsnorm");
    return XR_OK;
}

// ---------------------------------------------------------------- dynamic tanh ("DyT")
// A norm without statistics: y_i = tanh(alpha x_i) w_i + b_i, alpha one number, in 32-bit.  As nothing of
// the row enters an element's value, the kernel is element-wise, and one pass can do what lies between two
// sublayers of a layer whose sublayers are normed before and after:
//   x += mult * (tanh(alpha_p y) w_p + b_p)        (the sublayer's result y through its second norm)
//   h  = tanh(alpha_n x) w_n + b_n                 (the next sublayer's input)
// either half alone too.  `rows` selects rows of x for the second half alone (the final norm).
struct DytArgs {
    float* x;               // [T, ldx] 32-bit residual rows
    const void* y;          // [T, E] the sublayer's result, or null
    const float* w_p; const float* b_p; float alpha_p, mult;
    void* h;                // [R, E] out, or null
    const float* w_n; const float* b_n; float alpha_n;
    const int* rows;
    int E, ldx;
    size_t n;               // elements (groups of NV) in all
};

template <typename TY, typename TO, int NV>
__global__ __launch_bounds__(256) void k_dyt_step(DytArgs a) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= a.n) return;
    const int per_row = a.E / NV;
    const size_t r = i / per_row;
    const int c = (int)(i - r * per_row) * NV;
    const size_t src = a.rows ? (size_t)a.rows[r] : r;
    float* xp = a.x + src * a.ldx + c;
    float v[NV], wv[NV], bv[NV];
    // NV = 4: E, ldx and c are multiples of 4 and the tensors' starts are 16-byte aligned, so a lane's four
    // values are one load and one store
    if constexpr (NV == 4) {
        const float4 t = *reinterpret_cast<const float4*>(xp);
        v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
    } else {
#pragma unroll
        for (int k = 0; k < NV; ++k) v[k] = xp[k];
    }
    auto vec = [&](const float* p, float (&o)[NV]) {
        if constexpr (NV == 4) {
            const float4 t = *reinterpret_cast<const float4*>(p + c);
            o[0] = t.x; o[1] = t.y; o[2] = t.z; o[3] = t.w;
        } else {
#pragma unroll
            for (int k = 0; k < NV; ++k) o[k] = p[c + k];
        }
    };
    if (a.y) {
        float yv[NV];
        if constexpr (NV == 4 && sizeof(TY) == 4) {
            const float4 t = *reinterpret_cast<const float4*>((const float*)a.y + r * a.E + c);
            yv[0] = t.x; yv[1] = t.y; yv[2] = t.z; yv[3] = t.w;
        } else if constexpr (NV == 4) {
            const uint2 t = *reinterpret_cast<const uint2*>((const bf16_t*)a.y + r * a.E + c);
            yv[0] = __uint_as_float(t.x << 16); yv[1] = __uint_as_float(t.x & 0xffff0000u);
            yv[2] = __uint_as_float(t.y << 16); yv[3] = __uint_as_float(t.y & 0xffff0000u);
        } else {
#pragma unroll
            for (int k = 0; k < NV; ++k) yv[k] = ld<TY>((const TY*)a.y, r * a.E + c + k);
        }
        vec(a.w_p, wv); vec(a.b_p, bv);
#pragma unroll
        for (int k = 0; k < NV; ++k) v[k] = v[k] + a.mult * fmaf(tanhf(a.alpha_p * yv[k]), wv[k], bv[k]);
        if constexpr (NV == 4) *reinterpret_cast<float4*>(xp) = make_float4(v[0], v[1], v[2], v[3]);
        else {
#pragma unroll
            for (int k = 0; k < NV; ++k) xp[k] = v[k];
        }
    }
    if (a.h) {
        vec(a.w_n, wv); vec(a.b_n, bv);
        float o[NV];
#pragma unroll
        for (int k = 0; k < NV; ++k) o[k] = fmaf(tanhf(a.alpha_n * v[k]), wv[k], bv[k]);
        if constexpr (NV == 4 && sizeof(TO) == 4)
            *reinterpret_cast<float4*>((float*)a.h + r * a.E + c) = make_float4(o[0], o[1], o[2], o[3]);
        else if constexpr (NV == 4)
            *reinterpret_cast<uint2*>((bf16_t*)a.h + r * a.E + c) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
        else {
#pragma unroll
            for (int k = 0; k < NV; ++k) st<TO>((TO*)a.h, r * a.E + c + k, o[k]);
        }
    }
}

extern "C" int xr_dyt_step(float* x, const void* y, const float* w_p, const float* b_p, float alpha_p, float mult,
                           void* h, const float* w_n, const float* b_n, float alpha_n, const int* rows, int R, int E,
                           int ldx, int y_dtype, int h_dtype, hipStream_t stream) {
    XR_REQUIRE(R >= 0 && E > 0 && ldx >= E, "dyt: bad sizes R=%d E=%d ldx=%d", R, E, ldx);
    XR_REQUIRE(x != nullptr && (y != nullptr || h != nullptr), "dyt: nothing to do");
    XR_REQUIRE(!y || (w_p && b_p), "dyt: the norm of the sublayer's result needs its weight and bias");
    XR_REQUIRE(!h || (w_n && b_n), "dyt: the norm needs its weight and bias");
    XR_REQUIRE(!(y && rows), "dyt: a selection of rows goes with the norm alone");
    XR_REQUIRE((y_dtype == XR_F32 || y_dtype == XR_BF16) && (h_dtype == XR_F32 || h_dtype == XR_BF16),
               "dyt: bad dtypes y=%d h=%d", y_dtype, h_dtype);
    if (R == 0) return XR_OK;
    auto al16 = [](const void* p) { return p == nullptr || (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    const bool vec = E % 4 == 0 && ldx % 4 == 0 && al16(x) && al16(y) && al16(h) && al16(w_p) && al16(b_p) && al16(w_n) && al16(b_n);
    DytArgs a{x, y, w_p, b_p, alpha_p, mult, h, w_n, b_n, alpha_n, rows, E, ldx, (size_t)R * (E / (vec ? 4 : 1))};
    const unsigned blocks = (unsigned)((a.n + 255) / 256);
#define DY(TY, TO)                                                                  \
    do {                                                                            \
        if (vec) k_dyt_step<TY, TO, 4><<<blocks, 256, 0, stream>>>(a);              \
        else k_dyt_step<TY, TO, 1><<<blocks, 256, 0, stream>>>(a);                  \
    } while (0)
    if (y_dtype == XR_F32 && h_dtype == XR_F32) DY(float, float);
    else if (y_dtype == XR_F32) DY(float, bf16_t);
    else if (h_dtype == XR_F32) DY(bf16_t, float);
    else DY(bf16_t, bf16_t);
#undef DY
    XR_CHECK_LAUNCH("dyt_step");
    return XR_OK;
}

// ---------------------------------------------------------------- rotary + cache write
// Rotation of pair index j of a head by a = pos * inv_freq[j]:
//   (x0, x1) -> (x0*c - x1*s, x0*s + x1*c), c = cos(a)*mscale, s = sin(a)*mscale
// (src/model.c:3514-3532).  Half-split pairs (j, j + rot/2) are what
// un-permuted checkpoints need; interleaved pairs (2j, 2j+1) are the other option.
// Keys are cached rotated, values as they are (src/model.c:6300-6311).
// Cache layout per layer: K [page][kv_head][slot][d], V [page][kv_head][d][slot].
struct RopeArgs {
    const float* q_in;      // [T, in_stride] 32-bit
    const float* k_in;
    const float* v_in;
    int in_stride;
    void* q_out;            // [T, H*D] storage type
    void* k_cache;
    void* v_cache;
    const int* positions;   // [T]
    const int* req_of_token;// [T]
    const int* block_table; // [B, table_stride]
    int table_stride;
    const float* inv_freq;  // [rot/2] or null
    int T, H, Hk, D, rot, interleaved;
    float mscale;
    int page_shift, page_mask, page_size;
    int heads_per_block;
    int paired;             // queries and keys come in paired order (paired_col)
};

// 8 values of one channel at 8 consecutive positions of a page: 16 or 32 bytes side by side in
// the transposed value cache.
template <typename T> __device__ inline void store8(T* dst, const float* v);
template <> __device__ inline void store8<float>(float* dst, const float* v) {
    *reinterpret_cast<float4*>(dst) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(dst + 4) = make_float4(v[4], v[5], v[6], v[7]);
}
template <> __device__ inline void store8<bf16_t>(bf16_t* dst, const float* v) {
    *reinterpret_cast<uint4*>(dst) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                                                pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
}

// A workgroup takes a token and some of its heads (heads_per_block, a wave a head at a time):
// query heads are rotated into q_out, key heads rotated into their page, value heads written
// to theirs.  The cosines and sines of the token's angles are computed once per workgroup into
// LDS and serve every head (the exact cosf/sinf of 64 angles for each of 40 heads was what the
// kernel's time went to).  Values are cached transposed ([channel][position]), so a token
// alone writes one element every page_size: where the step brings the 8 positions of an
// aligned group of a page (prompt portions), the wave of the group's first token writes all 8
// side by side for each channel and the other seven leave their values to it.
template <typename T>
__global__ __launch_bounds__(256) void k_rope_kv_write(RopeArgs a) {
    __shared__ float cs[2][128];
    const int t = blockIdx.x;
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int pos = a.positions[t];
    const int D = a.D, half = a.rot >> 1;
    for (int j = threadIdx.x; j < half; j += 256) {
        const float ang = (float)pos * a.inv_freq[j];
        cs[0][j] = cosf(ang) * a.mscale;
        cs[1][j] = sinf(ang) * a.mscale;
    }
    __syncthreads();
    const int h_begin = blockIdx.y * a.heads_per_block;
    const int h_end = min(a.H + a.Hk, h_begin + a.heads_per_block);
    // query heads, four at a time per wave: the loads of all four are on their way before the
    // first is used (one head at a time, a wave waited out a memory latency per head)
    const int hq_end = min(h_end, a.H);
    for (int hb = h_begin + wave * 4; hb < hq_end; hb += 16) {
        const float* src[4];
        T* dst[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int hs = hb + u < hq_end ? hb + u : hb;
            src[u] = a.q_in + (size_t)t * a.in_stride + (size_t)hs * D;
            dst[u] = (T*)a.q_out + ((size_t)t * a.H + hs) * D;
        }
        for (int j = lane; j < half; j += 64) {
            const int i0 = a.interleaved ? 2 * j : j;
            const int i1 = a.interleaved ? 2 * j + 1 : j + half;
            const int c0 = a.paired ? paired_col(i0, a.rot) : i0, c1 = a.paired ? paired_col(i1, a.rot) : i1;
            float x0[4], x1[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) { x0[u] = src[u][c0]; x1[u] = src[u][c1]; }
            const float c = cs[0][j], sn = cs[1][j];
#pragma unroll
            for (int u = 0; u < 4; ++u)
                if (hb + u < hq_end) {
                    st<T>(dst[u], i0, x0[u] * c - x1[u] * sn);
                    st<T>(dst[u], i1, x0[u] * sn + x1[u] * c);
                }
        }
        for (int i = a.rot + lane; i < D; i += 64) {
            float x[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) x[u] = src[u][i];
#pragma unroll
            for (int u = 0; u < 4; ++u)
                if (hb + u < hq_end) st<T>(dst[u], i, x[u]);
        }
    }
    for (int hs = max(h_begin, a.H) + wave; hs < h_end; hs += 4) {
        const int kvh = hs - a.H;
        const int req = a.req_of_token[t];
        PageRef pr = page_of(a.block_table, a.table_stride, req, pos, a.page_shift, a.page_mask);
        const float* ks = a.k_in + (size_t)t * a.in_stride + (size_t)kvh * D;
        const float* vs = a.v_in + (size_t)t * a.in_stride + (size_t)kvh * D;
        T* kd = (T*)a.k_cache + (((size_t)pr.page * a.Hk + kvh) * a.page_size + pr.off) * D;
        T* vd = (T*)a.v_cache + ((size_t)pr.page * a.Hk + kvh) * D * a.page_size + pr.off;
        for (int j = lane; j < half; j += 64) {
            const int i0 = a.interleaved ? 2 * j : j;
            const int i1 = a.interleaved ? 2 * j + 1 : j + half;
            const float x0 = ks[a.paired ? paired_col(i0, a.rot) : i0], x1 = ks[a.paired ? paired_col(i1, a.rot) : i1];
            const float c = cs[0][j], sn = cs[1][j];
            st<T>(kd, i0, x0 * c - x1 * sn);
            st<T>(kd, i1, x0 * sn + x1 * c);
        }
        for (int i = a.rot + lane; i < D; i += 64) st<T>(kd, i, ks[i]);
        // the aligned group of 8 positions this token belongs to: whole in this step?  (A request's
        // tokens of a step are consecutive rows at consecutive positions.)
        const int lead = t - (pos & 7);
        const bool whole = a.page_size >= 8 && lead >= 0 && lead + 7 < a.T && a.req_of_token[lead] == req &&
                           a.req_of_token[lead + 7] == req && a.positions[lead] == pos - (pos & 7);
        if (!whole) {
            for (int i = lane; i < D; i += 64) st<T>(vd, (size_t)i * a.page_size, vs[i]);
        } else if ((pos & 7) == 0) {
            for (int i = lane; i < D; i += 64) {
                float v[8];
#pragma unroll
                for (int j = 0; j < 8; ++j) v[j] = vs[(size_t)j * a.in_stride + i];
                store8<T>(vd + (size_t)i * a.page_size, v);
            }
        }
    }
}

extern "C" int xr_rope_kv_write(const float* q_in, const float* k_in, const float* v_in, int in_stride,
                                void* q_out, void* k_cache, void* v_cache, const int* positions,
                                const int* req_of_token, const int* block_table, int table_stride,
                                const float* inv_freq, int T, int H, int Hk, int D, int rot,
                                int interleaved, float mscale, int page_size, int dtype, int paired,
                                hipStream_t stream) {
    XR_REQUIRE(T >= 0 && H >= 0 && Hk >= 0 && D > 0, "rope_kv_write: bad sizes T=%d H=%d Hk=%d D=%d", T, H, Hk, D);
    XR_REQUIRE(rot >= 0 && rot <= D && (rot % 2) == 0, "rope_kv_write: rotary width %d must be even and at most head_dim %d", rot, D);
    XR_REQUIRE(rot == 0 || inv_freq, "rope_kv_write: rotary width %d without a frequency table", rot);
    int shift = ilog2_exact(page_size);
    XR_REQUIRE(Hk == 0 || shift >= 0, "rope_kv_write: page size %d is not a power of two", page_size);
    XR_REQUIRE(Hk == 0 || (k_in && v_in && k_cache && v_cache && block_table && req_of_token),
               "rope_kv_write: keys and values to cache but a null operand");
    XR_REQUIRE(H == 0 || (q_in && q_out), "rope_kv_write: queries but a null operand");
    XR_REQUIRE(dtype == XR_F32 || dtype == XR_BF16, "rope_kv_write: bad dtype %d", dtype);
    if (T == 0 || H + Hk == 0) return XR_OK;
    RopeArgs a;
    a.q_in = q_in; a.k_in = k_in; a.v_in = v_in; a.in_stride = in_stride;
    a.q_out = q_out; a.k_cache = k_cache; a.v_cache = v_cache;
    a.positions = positions; a.req_of_token = req_of_token;
    a.block_table = block_table; a.table_stride = table_stride; a.inv_freq = inv_freq;
    a.T = T; a.H = H; a.Hk = Hk; a.D = D; a.rot = rot; a.interleaved = interleaved; a.mscale = mscale;
    a.page_shift = shift < 0 ? 0 : shift; a.page_mask = page_size - 1; a.page_size = page_size;
    XR_REQUIRE(rot <= 256, "rope_kv_write: rotary width %d exceeds 256", rot);
    XR_REQUIRE(!paired || (!interleaved && rot % 16 == 0), "rope_kv_write: paired order needs pairs (j, j + width/2) and a rotary width (%d) that is a multiple of 16", rot);
    a.paired = paired ? 1 : 0;
    // all heads of a token in one workgroup when there are tokens enough to fill the chip, else
    // fewer heads each, down to one a wave
    int groups = (1024 + T - 1) / T;
    const int max_groups = (H + Hk + 3) / 4;
    groups = groups < 1 ? 1 : (groups > max_groups ? max_groups : groups);
    a.heads_per_block = (H + Hk + groups - 1) / groups;
    dim3 grid(T, (H + Hk + a.heads_per_block - 1) / a.heads_per_block);
    if (dtype == XR_F32) k_rope_kv_write<float><<<grid, 256, 0, stream>>>(a);
    else k_rope_kv_write<bf16_t><<<grid, 256, 0, stream>>>(a);
    XR_CHECK_LAUNCH("rope_kv_write");
    return XR_OK;
}

// ---------------------------------------------------------------- norm over all heads + rotary + cache write
// The same for queries and keys that are normed over all their heads at once first (RMS, eps inside the root, a
// weight a channel of the whole projection): a workgroup takes a token, sums the squares of its queries and of its
// keys, and rotates what it scales.  Values come from rows of their own, which may be the keys' before norm and
// rotation; they are stored as above.  NW waves: 4 where there are tokens enough to fill the chip, 16 for the few of a
// decode step.  VEC: neighbouring pairs, head size, rotated part, widths and strides multiples of 4, bases on 16 bytes:
// a lane takes 4 channels (two pairs) of a head.
struct RowNormArgs {
    RopeArgs r;
    const float* wq;        // [H * D]
    const float* wk;        // [Hk * D]
    float eps;
};

template <typename T> __device__ inline void put4(T* p, float a, float b, float c, float d);
template <> __device__ inline void put4<float>(float* p, float a, float b, float c, float d) {
    *reinterpret_cast<float4*>(p) = make_float4(a, b, c, d);
}
template <> __device__ inline void put4<bf16_t>(bf16_t* p, float a, float b, float c, float d) {
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(a, b), pack_bf16x2(c, d));
}

template <typename T, int NW, bool VEC>
__global__ __launch_bounds__(64 * NW) void k_row_norm_rope_write(RowNormArgs n) {
    constexpr int NT = 64 * NW;
    __shared__ float cs[2][128];
    __shared__ float part[2][NW];
    const RopeArgs& a = n.r;
    const int t = blockIdx.x, tid = threadIdx.x;
    const int D = a.D, half = a.rot >> 1, Q = a.H * D, K = a.Hk * D;
    const float* qr = a.q_in + (size_t)t * a.in_stride;
    const float* kr = a.Hk ? a.k_in + (size_t)t * a.in_stride : qr;
    const int pos = a.positions[t];
    float sq = 0.f, sk = 0.f;
    if (VEC) {
        for (int i = tid * 4; i < Q; i += NT * 4) {
            const float4 x = *reinterpret_cast<const float4*>(qr + i);
            sq += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
        }
        for (int i = tid * 4; i < K; i += NT * 4) {
            const float4 x = *reinterpret_cast<const float4*>(kr + i);
            sk += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
        }
    } else {
        for (int i = tid; i < Q; i += NT) sq = fmaf(qr[i], qr[i], sq);
        for (int i = tid; i < K; i += NT) sk = fmaf(kr[i], kr[i], sk);
    }
    for (int j = tid; j < half; j += NT) {
        const float ang = (float)pos * a.inv_freq[j];
        cs[0][j] = cosf(ang) * a.mscale;
        cs[1][j] = sinf(ang) * a.mscale;
    }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((tid & 63) == 0) { part[0][tid >> 6] = sq; part[1][tid >> 6] = sk; }
    __syncthreads();
    sq = sk = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) { sq += part[0][w]; sk += part[1][w]; }
    const float rq = 1.0f / sqrtf(sq / (float)Q + n.eps);
    const float rk = K ? 1.0f / sqrtf(sk / (float)K + n.eps) : 0.f;
    PageRef pr{0, 0};
    int req = 0;
    if (K) {
        req = a.req_of_token[t];
        pr = page_of(a.block_table, a.table_stride, req, pos, a.page_shift, a.page_mask);
    }
    T* qo = (T*)a.q_out + (size_t)t * Q;
    // channel d of key head g of this token: kpage + g * (page_size * D) + d
    T* kpage = (T*)a.k_cache + ((size_t)pr.page * a.Hk * a.page_size + pr.off) * D;
    const int total = Q + K;
    if (VEC) {
        for (int i4 = tid * 4; i4 < total; i4 += NT * 4) {
            const bool is_q = i4 < Q;
            const int i = is_q ? i4 : i4 - Q;
            const int head = i / D, d = i - head * D;
            float4 x = *reinterpret_cast<const float4*>((is_q ? qr : kr) + i);
            const float4 w = *reinterpret_cast<const float4*>((is_q ? n.wq : n.wk) + i);
            const float f = is_q ? rq : rk;
            x.x *= f * w.x; x.y *= f * w.y; x.z *= f * w.z; x.w *= f * w.w;
            if (d < a.rot) {
                const int j = d >> 1;
                const float c0 = cs[0][j], s0 = cs[1][j], c1 = cs[0][j + 1], s1 = cs[1][j + 1];
                x = make_float4(x.x * c0 - x.y * s0, x.x * s0 + x.y * c0, x.z * c1 - x.w * s1, x.z * s1 + x.w * c1);
            }
            put4<T>(is_q ? qo + i : kpage + (size_t)head * a.page_size * D + d, x.x, x.y, x.z, x.w);
        }
    } else {
        for (int ii = tid; ii < total; ii += NT) {
            const bool is_q = ii < Q;
            const int i = is_q ? ii : ii - Q;
            const int head = i / D, d = i - head * D;
            const float* src = is_q ? qr : kr;
            const float* w = is_q ? n.wq : n.wk;
            const float f = is_q ? rq : rk;
            float y = src[i] * f * w[i];
            if (d < a.rot) {
                const int j = a.interleaved ? d >> 1 : (d < half ? d : d - half);
                const bool first = a.interleaved ? (d & 1) == 0 : d < half;
                const int o = i + (first ? 1 : -1) * (a.interleaved ? 1 : half);     // the pair's other channel
                const float z = src[o] * f * w[o];
                y = first ? y * cs[0][j] - z * cs[1][j] : z * cs[1][j] + y * cs[0][j];
            }
            st<T>(is_q ? qo : kpage + (size_t)head * a.page_size * D, is_q ? i : d, y);
        }
    }
    if (!K) return;
    // values: see k_rope_kv_write
    const float* vr = a.v_in + (size_t)t * a.in_stride;
    T* vpage = (T*)a.v_cache + (size_t)pr.page * K * a.page_size + pr.off;
    const int lead = t - (pos & 7);
    const bool whole = a.page_size >= 8 && lead >= 0 && lead + 7 < a.T && a.req_of_token[lead] == req &&
                       a.req_of_token[lead + 7] == req && a.positions[lead] == pos - (pos & 7);
    if (!whole) {
        for (int i = tid; i < K; i += NT) st<T>(vpage, (size_t)i * a.page_size, vr[i]);
    } else if ((pos & 7) == 0) {
        for (int i = tid; i < K; i += NT) {
            float v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = vr[(size_t)j * a.in_stride + i];
            store8<T>(vpage + (size_t)i * a.page_size, v);
        }
    }
}

extern "C" int xr_row_norm_rope_write(const float* q_in, const float* k_in, const float* v_in, int in_stride, const float* wq,
                                      const float* wk, float eps, void* q_out, void* k_cache, void* v_cache,
                                      const int* positions, const int* req_of_token, const int* block_table,
                                      int table_stride, const float* inv_freq, int T, int H, int Hk, int D, int rot,
                                      int interleaved, float mscale, int page_size, int dtype, hipStream_t stream) {
    XR_REQUIRE(T >= 0 && H > 0 && Hk >= 0 && D > 0, "row_norm_rope_write: bad sizes T=%d H=%d Hk=%d D=%d", T, H, Hk, D);
    XR_REQUIRE(rot >= 0 && rot <= D && (rot % 2) == 0 && rot <= 256, "row_norm_rope_write: rotary width %d must be even, at most head_dim %d and 256", rot, D);
    XR_REQUIRE(rot == 0 || inv_freq, "row_norm_rope_write: rotary width %d without a frequency table", rot);
    XR_REQUIRE(eps >= 0.f, "row_norm_rope_write: eps %g is negative", (double)eps);
    const int shift = ilog2_exact(page_size);
    XR_REQUIRE(Hk == 0 || shift >= 0, "row_norm_rope_write: page size %d is not a power of two", page_size);
    XR_REQUIRE(Hk == 0 || (k_in && v_in && wk && k_cache && v_cache && block_table && req_of_token),
               "row_norm_rope_write: keys and values to cache but a null operand");
    XR_REQUIRE(q_in && q_out && wq && positions, "row_norm_rope_write: an operand is missing");
    XR_REQUIRE(dtype == XR_F32 || dtype == XR_BF16, "row_norm_rope_write: bad dtype %d", dtype);
    if (T == 0) return XR_OK;
    RowNormArgs n;
    RopeArgs& a = n.r;
    a.q_in = q_in; a.k_in = k_in; a.v_in = v_in; a.in_stride = in_stride;
    a.q_out = q_out; a.k_cache = k_cache; a.v_cache = v_cache;
    a.positions = positions; a.req_of_token = req_of_token;
    a.block_table = block_table; a.table_stride = table_stride; a.inv_freq = inv_freq;
    a.T = T; a.H = H; a.Hk = Hk; a.D = D; a.rot = rot; a.interleaved = interleaved; a.mscale = mscale;
    a.page_shift = shift < 0 ? 0 : shift; a.page_mask = page_size - 1; a.page_size = page_size;
    a.heads_per_block = 0; a.paired = 0;
    n.wq = wq; n.wk = wk; n.eps = eps;
    auto on16 = [](const void* p) { return ((uintptr_t)p % 16) == 0; };
    const bool vec = (interleaved || rot == 0) && D % 4 == 0 && rot % 4 == 0 && in_stride % 4 == 0 && on16(q_in) && on16(k_in) &&
                     on16(wq) && on16(wk) && on16(q_out) && on16(k_cache);
    const bool few = T <= 128 && (H + Hk) * D >= 1024;
#define RNW(TT)                                                                                    \
    do {                                                                                            \
        if (vec && few) k_row_norm_rope_write<TT, 16, true><<<T, 1024, 0, stream>>>(n);             \
        else if (vec) k_row_norm_rope_write<TT, 4, true><<<T, 256, 0, stream>>>(n);                 \
        else if (few) k_row_norm_rope_write<TT, 16, false><<<T, 1024, 0, stream>>>(n);              \
        else k_row_norm_rope_write<TT, 4, false><<<T, 256, 0, stream>>>(n);                         \
    } while (0)
    if (dtype == XR_F32) RNW(float);
    else RNW(bf16_t);
#undef RNW
    XR_CHECK_LAUNCH("row_norm_rope_write");
    return XR_OK;
}

// The same head by head, for values of any size: every query and key head over its own root mean square (eps inside
// the root) times a weight of its channels that the heads share (absent: none), before the rotation or behind it, or no
// norm at all.  Queries go out, keys and values (Dv channels a head) to their pages.  A workgroup a token, a wave a head at
// a time: its lanes hold channels lane, lane + 64, .. and read a pair's other channel beside their own.
struct HeadNormArgs {
    RopeArgs r;
    const float* wq;        // [D] or null
    const float* wk;        // [D] or null
    float eps;
    int norm;               // HEAD_NORM_*
    int Dv;
};
#define HEAD_NORM_NONE 0
#define HEAD_NORM_BEFORE 1
#define HEAD_NORM_AFTER 2
#define HEAD_MAX_D 256
template <typename T, int NW>
__global__ __launch_bounds__(64 * NW) void k_head_norm_rope_write(HeadNormArgs n) {
    constexpr int NT = 64 * NW, NC = HEAD_MAX_D / 64;
    __shared__ float cs[2][HEAD_MAX_D / 2];
    const RopeArgs& a = n.r;
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int D = a.D, half = a.rot >> 1;
    const int pos = a.positions[t];
    for (int j = tid; j < half; j += NT) {
        const float ang = (float)pos * a.inv_freq[j];
        cs[0][j] = cosf(ang) * a.mscale;
        cs[1][j] = sinf(ang) * a.mscale;
    }
    __syncthreads();
    PageRef pr{0, 0};
    int req = 0;
    if (a.Hk) {
        req = a.req_of_token[t];
        pr = page_of(a.block_table, a.table_stride, req, pos, a.page_shift, a.page_mask);
    }
    for (int head = wave; head < a.H + a.Hk; head += NW) {
        const bool is_q = head < a.H;
        const float* src = (is_q ? a.q_in + (size_t)head * D : a.k_in + (size_t)(head - a.H) * D) + (size_t)t * a.in_stride;
        const float* w = is_q ? n.wq : n.wk;
        float x[NC], z[NC], wx[NC], wz[NC];
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
            const int d = lane + 64 * i;
            const bool ok = d < D, turns = d < a.rot;
            const int o = !turns ? d : a.interleaved ? d ^ 1 : (d < half ? d + half : d - half);      // the pair's other channel
            x[i] = ok ? src[d] : 0.f;
            z[i] = ok && turns ? src[o] : 0.f;
            wx[i] = ok && w ? w[d] : 1.f;
            wz[i] = ok && w && turns ? w[o] : 1.f;
            ss = fmaf(x[i], x[i], ss);
        }
        if (n.norm == HEAD_NORM_BEFORE) {
            const float f = 1.0f / sqrtf(wave_sum(ss) / (float)D + n.eps);
#pragma unroll
            for (int i = 0; i < NC; ++i) { x[i] *= f * wx[i]; z[i] *= f * wz[i]; }
        }
        ss = 0.f;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
            const int d = lane + 64 * i;
            if (d < a.rot) {
                const int j = a.interleaved ? d >> 1 : (d < half ? d : d - half);
                const bool first = a.interleaved ? (d & 1) == 0 : d < half;
                const float c = cs[0][j], s = cs[1][j];
                x[i] = first ? x[i] * c - z[i] * s : x[i] * c + z[i] * s;
            }
            ss = fmaf(x[i], x[i], ss);
        }
        if (n.norm == HEAD_NORM_AFTER) {
            const float f = 1.0f / sqrtf(wave_sum(ss) / (float)D + n.eps);
#pragma unroll
            for (int i = 0; i < NC; ++i) x[i] *= f * wx[i];
        }
        T* dst = is_q ? (T*)a.q_out + ((size_t)t * a.H + head) * D
                      : (T*)a.k_cache + (((size_t)pr.page * a.Hk + (head - a.H)) * a.page_size + pr.off) * D;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
            const int d = lane + 64 * i;
            if (d < D) st<T>(dst, d, x[i]);
        }
    }
    if (!a.Hk) return;
    // values: see k_rope_kv_write
    const int V = a.Hk * n.Dv;
    const float* vr = a.v_in + (size_t)t * a.in_stride;
    T* vpage = (T*)a.v_cache + (size_t)pr.page * V * a.page_size + pr.off;
    const int lead = t - (pos & 7);
    const bool whole = a.page_size >= 8 && lead >= 0 && lead + 7 < a.T && a.req_of_token[lead] == req &&
                       a.req_of_token[lead + 7] == req && a.positions[lead] == pos - (pos & 7);
    if (!whole) {
        for (int i = tid; i < V; i += NT) st<T>(vpage, (size_t)i * a.page_size, vr[i]);
    } else if ((pos & 7) == 0) {
        for (int i = tid; i < V; i += NT) {
            float v[8];
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = vr[(size_t)j * a.in_stride + i];
            store8<T>(vpage + (size_t)i * a.page_size, v);
        }
    }
}

extern "C" int xr_head_norm_rope_write(const float* q_in, const float* k_in, const float* v_in, int in_stride, const float* wq,
                                       const float* wk, float eps, int norm, void* q_out, void* k_cache, void* v_cache,
                                       const int* positions, const int* req_of_token, const int* block_table,
                                       int table_stride, const float* inv_freq, int T, int H, int Hk, int D, int Dv, int rot,
                                       int interleaved, float mscale, int page_size, int dtype, hipStream_t stream) {
    XR_REQUIRE(T >= 0 && H > 0 && Hk >= 0 && D > 0 && D <= HEAD_MAX_D && Dv > 0, "head_norm_rope_write: bad sizes T=%d H=%d Hk=%d D=%d Dv=%d", T, H, Hk, D, Dv);
    XR_REQUIRE(rot >= 0 && rot <= D && (rot % 2) == 0, "head_norm_rope_write: rotary width %d must be even and at most head_dim %d", rot, D);
    XR_REQUIRE(rot == 0 || inv_freq, "head_norm_rope_write: rotary width %d without a frequency table", rot);
    XR_REQUIRE(eps >= 0.f && norm >= HEAD_NORM_NONE && norm <= HEAD_NORM_AFTER, "head_norm_rope_write: eps %g, norm %d", (double)eps, norm);
    const int shift = ilog2_exact(page_size);
    XR_REQUIRE(Hk == 0 || shift >= 0, "head_norm_rope_write: page size %d is not a power of two", page_size);
    XR_REQUIRE(Hk == 0 || (k_in && v_in && k_cache && v_cache && block_table && req_of_token),
               "head_norm_rope_write: keys and values to cache but a null operand");
    XR_REQUIRE(q_in && q_out && positions, "head_norm_rope_write: an operand is missing");
    XR_REQUIRE(dtype == XR_F32 || dtype == XR_BF16, "head_norm_rope_write: bad dtype %d", dtype);
    if (T == 0) return XR_OK;
    HeadNormArgs n;
    RopeArgs& a = n.r;
    a.q_in = q_in; a.k_in = k_in; a.v_in = v_in; a.in_stride = in_stride;
    a.q_out = q_out; a.k_cache = k_cache; a.v_cache = v_cache;
    a.positions = positions; a.req_of_token = req_of_token;
    a.block_table = block_table; a.table_stride = table_stride; a.inv_freq = inv_freq;
    a.T = T; a.H = H; a.Hk = Hk; a.D = D; a.rot = rot; a.interleaved = interleaved; a.mscale = mscale;
    a.page_shift = shift < 0 ? 0 : shift; a.page_mask = page_size - 1; a.page_size = page_size;
    a.heads_per_block = 0; a.paired = 0;
    n.wq = wq; n.wk = wk; n.eps = eps; n.norm = norm; n.Dv = Dv;
    const bool few = T <= 128 && H + Hk > 4;
    if (dtype == XR_F32) {
        if (few) k_head_norm_rope_write<float, 16><<<T, 1024, 0, stream>>>(n);
        else k_head_norm_rope_write<float, 4><<<T, 256, 0, stream>>>(n);
    } else {
        if (few) k_head_norm_rope_write<bf16_t, 16><<<T, 1024, 0, stream>>>(n);
        else k_head_norm_rope_write<bf16_t, 4><<<T, 256, 0, stream>>>(n);
    }
    XR_CHECK_LAUNCH("head_norm_rope_write");
    return XR_OK;
}

// ---------------------------------------------------------------- gate
// h = act(g) * u; act = SiLU: g / (1 + exp(-g)) (src/model.c:4451-4452,
// src/kernels.cu:2868-2874).  gu row = [gate(F) | up(F)].
template <typename TI, typename TO>
__global__ void k_gate_mul(TO* __restrict__ out, const TI* __restrict__ gu, int F, int ld_gu, size_t n, int act, float param) {
    size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    size_t t = i / F;
    int c = (int)(i - t * F);
    float g = ld<TI>(gu, t * ld_gu + c);
    float u = ld<TI>(gu, t * ld_gu + F + c);
    st<TO>(out, i, gate_value<false>(act, param, g, u));
}

// dtype: of gu; out_dtype: of out (32-bit branches may leave as bfloat16)
extern "C" int xr_gate_mul(void* out, const void* gu, int T, int F, int ld_gu, int dtype, int out_dtype, int act, float param,
                           hipStream_t stream) {
    XR_REQUIRE(T >= 0 && F > 0 && ld_gu >= 2 * F, "gate_mul: bad sizes T=%d F=%d ld=%d", T, F, ld_gu);
    XR_REQUIRE(act >= 0 && act < XR_ACT_COUNT, "gate_mul: unknown activation code %d", act);
    size_t n = (size_t)T * F;
    if (n == 0) return XR_OK;
    unsigned blocks = (unsigned)((n + 255) / 256);
    if (dtype == XR_F32 && out_dtype == XR_F32) k_gate_mul<float, float><<<blocks, 256, 0, stream>>>((float*)out, (const float*)gu, F, ld_gu, n, act, param);
    else if (dtype == XR_F32 && out_dtype == XR_BF16) k_gate_mul<float, bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)out, (const float*)gu, F, ld_gu, n, act, param);
    else if (dtype == XR_BF16 && out_dtype == XR_BF16) k_gate_mul<bf16_t, bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)out, (const bf16_t*)gu, F, ld_gu, n, act, param);
    else { xr_set_error("gate_mul: bad dtypes %d -> %d", dtype, out_dtype); return XR_BAD_ARG; }
    XR_CHECK_LAUNCH("gate_mul");
    return XR_OK;
}

// ---------------------------------------------------------------- residual add
// x += scale * y (one rounding; with scale 1 the plain sum)
template <typename TY>
__global__ void k_add(float* __restrict__ x, const TY* __restrict__ y, size_t n, float scale) {
    size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) x[i] = fmaf(scale, ld<TY>(y, i), x[i]);
}

extern "C" int xr_add(float* x, const void* y, size_t n, int y_dtype, float scale, hipStream_t stream) {
    if (n == 0) return XR_OK;
    unsigned blocks = (unsigned)((n + 255) / 256);
    if (y_dtype == XR_F32) k_add<float><<<blocks, 256, 0, stream>>>(x, (const float*)y, n, scale);
    else if (y_dtype == XR_BF16) k_add<bf16_t><<<blocks, 256, 0, stream>>>(x, (const bf16_t*)y, n, scale);
    else { xr_set_error("add: bad dtype %d", y_dtype); return XR_BAD_ARG; }
    XR_CHECK_LAUNCH("add");
    return XR_OK;
}

// ---------------------------------------------------------------- fill (32-bit words)
__global__ void k_fill_rows(uint32_t* __restrict__ base, const int* __restrict__ rows, size_t row_words,
                            uint32_t value) {
    int r = rows ? rows[blockIdx.y] : blockIdx.y;
    if (r < 0) return;
    size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < row_words) base[(size_t)r * row_words + i] = value;
}

// Sets rows[r] (or rows 0..n_rows-1) of a [*, row_words] array of 32-bit words to `value`.
extern "C" int xr_fill_rows(void* base, const int* rows, int n_rows, size_t row_words, uint32_t value,
                            hipStream_t stream) {
    if (n_rows <= 0 || row_words == 0) return XR_OK;
    dim3 grid((unsigned)((row_words + 255) / 256), n_rows);
    k_fill_rows<<<grid, 256, 0, stream>>>((uint32_t*)base, rows, row_words, value);
    XR_CHECK_LAUNCH("fill_rows");
    return XR_OK;
}

// The same for many arrays at once (every state tensor of every layer when a request begins): array a
// has rows of row_words[a] words at bases[a]; one launch instead of one an array.
__global__ void k_fill_rows_many(uint32_t* const* __restrict__ bases, const size_t* __restrict__ row_words,
                                 const int* __restrict__ rows, uint32_t value) {
    const size_t words = row_words[blockIdx.z];
    const int r = rows[blockIdx.y];
    if (r < 0) return;
    uint32_t* row = bases[blockIdx.z] + (size_t)r * words;
    for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < words; i += (size_t)gridDim.x * blockDim.x) row[i] = value;
}

// bases, row_words: device arrays of n_arrays entries; rows: n_rows row numbers on the device.
extern "C" int xr_fill_rows_many(void* const* bases, const size_t* row_words, int n_arrays, size_t max_row_words,
                                 const int* rows, int n_rows, uint32_t value, hipStream_t stream) {
    if (n_arrays <= 0 || n_rows <= 0 || max_row_words == 0) return XR_OK;
    XR_REQUIRE(bases && row_words && rows, "fill_rows_many: an operand is missing");
    XR_REQUIRE(n_arrays <= 65535 && n_rows <= 65535, "fill_rows_many: %d arrays, %d rows (at most 65535 each)", n_arrays, n_rows);
    size_t blocks = (max_row_words + 255) / 256;
    if (blocks > 64) blocks = 64;           // longer rows: a block strides over its row
    dim3 grid((unsigned)blocks, n_rows, n_arrays);
    k_fill_rows_many<<<grid, 256, 0, stream>>>((uint32_t* const*)bases, row_words, rows, value);
    XR_CHECK_LAUNCH("fill_rows_many");
    return XR_OK;
}

// ---------------------------------------------------------------- dtype conversion
template <typename TI, typename TO>
__global__ void k_convert(TO* __restrict__ out, const TI* __restrict__ in, size_t n) {
    size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) st<TO>(out, i, ld<TI>(in, i));
}

extern "C" int xr_convert(void* out, const void* in, size_t n, int in_dtype, int out_dtype, hipStream_t stream) {
    if (n == 0) return XR_OK;
    unsigned blocks = (unsigned)((n + 255) / 256);
    if (in_dtype == XR_F32 && out_dtype == XR_BF16) k_convert<float, bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)out, (const float*)in, n);
    else if (in_dtype == XR_BF16 && out_dtype == XR_F32) k_convert<bf16_t, float><<<blocks, 256, 0, stream>>>((float*)out, (const bf16_t*)in, n);
    else if (in_dtype == XR_F32 && out_dtype == XR_F32) k_convert<float, float><<<blocks, 256, 0, stream>>>((float*)out, (const float*)in, n);
    else if (in_dtype == XR_BF16 && out_dtype == XR_BF16) k_convert<bf16_t, bf16_t><<<blocks, 256, 0, stream>>>((bf16_t*)out, (const bf16_t*)in, n);
    else { xr_set_error("convert: bad dtypes %d -> %d", in_dtype, out_dtype); return XR_BAD_ARG; }
    XR_CHECK_LAUNCH("convert");
    return XR_OK;
}

// ---------------------------------------------------------------- memory yardstick
// What the memory system delivers to a kernel that does nothing but read: every workgroup
// streams a range of its own with 16-byte loads marked as streaming, eight of them in flight
// a lane, and leaves the XOR of its words (so the loads cannot be dropped, and a test can
// check that every word was read once).  The benchmark reports a decode step's bytes per second
// as a fraction of this figure beside the fraction of the nominal peak.
typedef uint32_t xr_u32x4 __attribute__((ext_vector_type(4)));
__global__ __launch_bounds__(256) void k_stream_read(const xr_u32x4* __restrict__ src, size_t n16, uint32_t* __restrict__ sink) {
    const size_t per = (n16 + gridDim.x - 1) / gridDim.x;
    const size_t begin = (size_t)blockIdx.x * per;
    const size_t end = begin + per < n16 ? begin + per : n16;
    xr_u32x4 acc = {0u, 0u, 0u, 0u};
    size_t i = begin + threadIdx.x;
    for (; i + 7 * 256 < end; i += 8 * 256) {
        xr_u32x4 v[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = __builtin_nontemporal_load(src + i + u * 256);
#pragma unroll
        for (int u = 0; u < 8; ++u) acc ^= v[u];
    }
    for (; i < end; i += 256) acc ^= __builtin_nontemporal_load(src + i);
    uint32_t x = acc.x ^ acc.y ^ acc.z ^ acc.w;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) x ^= __shfl_xor(x, o, 64);
    __shared__ uint32_t part[4];
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = x;
    __syncthreads();
    if (threadIdx.x == 0) sink[blockIdx.x] = part[0] ^ part[1] ^ part[2] ^ part[3];
}

// sink: [blocks] words; the XOR of all of them is the XOR of the buffer's 32-bit words.
extern "C" int xr_stream_read(const void* src, size_t bytes, uint32_t* sink, int blocks, hipStream_t stream) {
    XR_REQUIRE(src && sink && blocks > 0 && blocks <= 65535, "stream_read: bad operands (%d workgroups)", blocks);
    XR_REQUIRE(bytes % 16 == 0 && ((uintptr_t)src % 16) == 0, "stream_read: the buffer must be a multiple of 16 bytes long and aligned so");
    k_stream_read<<<blocks, 256, 0, stream>>>((const xr_u32x4*)src, bytes / 16, sink);
    XR_CHECK_LAUNCH("stream_read");
    return XR_OK;
}
