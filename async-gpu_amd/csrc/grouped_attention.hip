// Grouped attention (grouped_attention.h).  The queries of all heads that share a key/value head, of all new tokens, are the
// columns of one matrix product: column c is token c / group, head c % group.  S^T = K Q^T and O^T = V^T P^T run on the matrix
// cores with an online softmax per column (query dimensions beyond the head are zero, value tiles beyond it are dropped), keys and (transposed) values straight from the cache.  The rows of a K tile are dealt
// so that the probabilities come out of the first product as the operand of the second, so nothing passes through the LDS
// until the waves of a workgroup merge.
//
// attend (decode, short portions, fp32 models): 16 columns per workgroup, keys split over workgroups and waves.  bf16 cache:
//   v_mfma_f32_16x16x32_bf16, queries and probabilities as two bf16 pieces (16 bits of mantissa); fp32 cache:
//   v_mfma_f32_16x16x4_f32.  A decode token's own key and value are the softmax's first state, straight from the projection (at
//   one position a rotation leaves the score of a query and a key alone), and the workgroup that starts with them writes them
//   to the cache.
// prompt (bf16): 32 columns per wave on v_mfma_f32_32x32x16_bf16.
#include <algorithm>

#include "grouped_attention.h"

namespace {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int kChunk = 32;       // keys per step of a wave
constexpr int kMaxSplits = 64;
constexpr int kPromptFrom = 16;  // new tokens per sequence from which bf16 models take the prompt kernel
constexpr float kMinusInf = -3.0e38f;

template <typename T>
__device__ __forceinline__ T to_cache(float v);
template <>
__device__ __forceinline__ float to_cache<float>(float v) { return v; }
template <>
__device__ __forceinline__ uint16_t to_cache<uint16_t>(float v) { return f32_to_bf16(v); }

// N consecutive dimensions from d0 on (both even) of a head's row, turned.  cs has at least one entry, even if nothing turns.
template <int N>
__device__ __forceinline__ void load_turned(const float *row, int d0, int rot_dims, const float2 *cs, float (&v)[N]) {
#pragma unroll
    for (int e = 0; e < N; e += 4) *(float4 *)&v[e] = *(const float4 *)(row + d0 + e);
#pragma unroll
    for (int e = 0; e < N; e += 2) {
        const bool turns = d0 + e < rot_dims;
        const float2 t = cs[turns ? (d0 + e) >> 1 : 0];
        const float c = turns ? t.x : 1.0f, n = turns ? t.y : 0.0f, a = v[e], b = v[e + 1];
        v[e] = a * c - b * n;
        v[e + 1] = b * c + a * n;
    }
}

// Sum or maximum over the four rows of 16 lanes, per column.
__device__ __forceinline__ float rows_max(float v) {
    auto s = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = fmaxf(__uint_as_float(s[0]), __uint_as_float(s[1]));
    s = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return fmaxf(__uint_as_float(s[0]), __uint_as_float(s[1]));
}
__device__ __forceinline__ float rows_sum(float v) {
    auto s = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    v = __uint_as_float(s[0]) + __uint_as_float(s[1]);
    s = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
    return __uint_as_float(s[0]) + __uint_as_float(s[1]);
}

// Exponentials and capped scores: next to bf16 keys the short forms (errors of some 1e-6), in fp32 models the accurate ones.
template <typename T>
__device__ __forceinline__ float exp_of(float x);
template <>
__device__ __forceinline__ float exp_of<float>(float x) { return expf(x); }
template <>
__device__ __forceinline__ float exp_of<uint16_t>(float x) { return __expf(x); }
template <typename T>
__device__ __forceinline__ float capped(float x, float cap);
template <>
__device__ __forceinline__ float capped<float>(float x, float cap) { return cap * tanhf(x / cap); }
template <>
__device__ __forceinline__ float capped<uint16_t>(float x, float cap) {  // cap tanh(x / cap) = cap - 2 cap / (exp(2 x / cap) + 1)
    return cap - 2.0f * cap * __builtin_amdgcn_rcpf(__expf(x * (2.0f * __builtin_amdgcn_rcpf(cap))) + 1.0f);
}

__device__ __forceinline__ void store4(const GroupedArgs &a, int row, int h, int vdimp, int dv, const float (&v)[4]) {
    float o[4] = {v[0], v[1], v[2], v[3]};
    if (a.gate) {
        const float4 g = *(const float4 *)(a.gate + (size_t)row * a.ld + h * vdimp + dv);
        o[0] *= sigmoid_dev(g.x);
        o[1] *= sigmoid_dev(g.y);
        o[2] *= sigmoid_dev(g.z);
        o[3] *= sigmoid_dev(g.w);
    }
    const size_t at = (size_t)row * a.ldo + h * vdimp + dv;
    if (a.out_bf16) {
        *(uint2 *)((uint16_t *)a.out + at) = make_uint2((uint32_t)f32_to_bf16(o[0]) | ((uint32_t)f32_to_bf16(o[1]) << 16),
                                                        (uint32_t)f32_to_bf16(o[2]) | ((uint32_t)f32_to_bf16(o[3]) << 16));
    } else {
        *(float4 *)((float *)a.out + at) = make_float4(o[0], o[1], o[2], o[3]);
    }
}

// One token's key and value of one head into the cache.
template <typename T>
__device__ __forceinline__ void write_token(const GroupedArgs &a, int dimp, int vdimp, int b, int kvh, int row, int p) {
    const GroupedShape &s = a.s;
    const int kvs = (a.positions + 31) / 32 * 32;
    const size_t hd = (size_t)b * s.kv_heads + kvh;
    T *kc = (T *)a.kcache + (hd * a.positions + p) * dimp, *vc = (T *)a.vcache + hd * vdimp * kvs + p;
    const float *k = a.k + (size_t)row * a.ld + kvh * dimp, *v = a.v + (size_t)row * a.ld + kvh * vdimp;
    const float2 *cs = a.rope + (size_t)p * (s.rot_dims >> 1);
    for (int d = threadIdx.x * 4; d < dimp; d += blockDim.x * 4) {
        float x[4];
        load_turned<4>(k, d, s.rot_dims, cs, x);
#pragma unroll
        for (int e = 0; e < 4; ++e) kc[d + e] = to_cache<T>(x[e]);
    }
    for (int e = threadIdx.x; e < vdimp; e += blockDim.x) vc[(size_t)e * kvs] = to_cache<T>(v[e]);
}

// grid (groups of 32 tokens, kv heads x (key, value), batch)
template <typename T>
__global__ __launch_bounds__(256) void grouped_append_kernel(GroupedArgs a, int dimp, int vdimp) {
    extern __shared__ float tile[];  // [32][vdimp + 1]
    const GroupedShape &s = a.s;
    const int t0 = blockIdx.x * 32, kvh = blockIdx.y >> 1, b = blockIdx.z, nt = min(32, a.new_len - t0), pos = *a.pos_dev;
    const int kvs = (a.positions + 31) / 32 * 32;
    const size_t hd = (size_t)b * s.kv_heads + kvh, row0 = (size_t)b * a.new_len + t0;
    if ((blockIdx.y & 1) == 0) {
        T *kc = (T *)a.kcache + (hd * a.positions + pos + t0) * dimp;
        const int quads = dimp >> 2, half = s.rot_dims >> 1;
#pragma unroll 4
        for (int i = threadIdx.x; i < nt * quads; i += 256) {
            const int t = i / quads, d = i % quads * 4;
            float x[4];
            load_turned<4>(a.k + (row0 + t) * a.ld + kvh * dimp, d, s.rot_dims, a.rope + (size_t)(pos + t0 + t) * half, x);
#pragma unroll
            for (int e = 0; e < 4; ++e) kc[(size_t)t * dimp + d + e] = to_cache<T>(x[e]);
        }
        return;
    }
    T *vc = (T *)a.vcache + hd * vdimp * kvs + pos + t0;
    const int quads = vdimp >> 2, t = threadIdx.x & 31;
#pragma unroll 4
    for (int i = threadIdx.x; i < nt * quads; i += 256) {
        const float4 v = *(const float4 *)(a.v + (row0 + i / quads) * a.ld + kvh * vdimp + i % quads * 4);
        float *to = tile + i / quads * (vdimp + 1) + i % quads * 4;
        to[0] = v.x;
        to[1] = v.y;
        to[2] = v.z;
        to[3] = v.w;
    }
    __syncthreads();
    if (t < nt) {
#pragma unroll 8
        for (int e = threadIdx.x >> 5; e < vdimp; e += 8) vc[(size_t)e * kvs + t] = to_cache<T>(tile[t * (vdimp + 1) + e]);
    }
}

// The columns of a 16-column block and the cached keys they see (one new token: all before it).
struct Columns {
    int t, h, row;       // of this lane's column
    int kv, chunks, per; // of the block
};
template <bool ONE>
__device__ __forceinline__ Columns columns_of(const GroupedArgs &a, int group, int kvh, int b, int c, int pos, int splits) {
    Columns x;
    const int nc = ONE ? group : a.new_len * group, cc = min(c, nc - 1);
    x.t = ONE ? 0 : cc / group;
    x.h = kvh * group + (ONE ? cc : cc % group);
    x.row = ONE ? b : b * a.new_len + x.t;
    x.kv = ONE ? pos : pos + min((c & ~15) + 15, nc - 1) / group + 1;
    x.chunks = (x.kv + kChunk - 1) / kChunk;
    x.per = max((x.chunks + splits - 1) / splits, 1);
    return x;
}

// What differs between the cache formats.  A chunk's scores are two tiles of 16 keys: register r of tile j in row g of 16
// lanes is key key_of(j, g, r).
template <typename T, int ND>
struct Product;

template <int ND>
struct Product<uint16_t, ND> {
    bf16x8 q[ND][2];
    __device__ __forceinline__ void load_query(const float *row, int rot_dims, const float2 *cs, int g, int nd) {
#pragma unroll
        for (int k = 0; k < ND; ++k) {
            float v[8];
            load_turned<8>(row, 32 * min(k, nd - 1) + 8 * g, rot_dims, cs, v);  // dimensions beyond the head are zero
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                q[k][0][e] = k < nd ? (__bf16)v[e] : (__bf16)0.0f;
                q[k][1][e] = k < nd ? (__bf16)(v[e] - (float)q[k][0][e]) : (__bf16)0.0f;
            }
        }
    }
    static __device__ __forceinline__ int row_key(int j, int i) { return 8 * (i >> 2) + 4 * j + (i & 3); }
    static __device__ __forceinline__ int key_of(int j, int g, int r) { return 8 * g + 4 * j + r; }
    struct Keys {
        bf16x8 k[ND];
    };
    static __device__ __forceinline__ Keys keys(const uint16_t *row, int g, int nd) {
        Keys x;
#pragma unroll
        for (int k = 0; k < ND; ++k)
            x.k[k] = *(const bf16x8 *)(row + 32 * min(k, nd - 1) + 8 * g);
        return x;
    }
    __device__ __forceinline__ f32x4 scores(const Keys &x) const {
        f32x4 hi = {0.0f, 0.0f, 0.0f, 0.0f}, lo = hi;
#pragma unroll
        for (int k = 0; k < ND; ++k) {
            lo = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x.k[k], q[k][1], lo, 0, 0, 0);
            hi = __builtin_amdgcn_mfma_f32_16x16x32_bf16(x.k[k], q[k][0], hi, 0, 0, 0);
        }
        return hi + lo;
    }
    struct Weights {
        bf16x8 hi, lo;
    };
    static __device__ __forceinline__ Weights weights(const float (&p)[2][4]) {
        Weights w;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float v = p[e >> 2][e & 3];
            w.hi[e] = (__bf16)v;
            w.lo[e] = (__bf16)(v - (float)w.hi[e]);
        }
        return w;
    }
    struct Values {
        bf16x8 v;
    };
    // 32 keys of one value dimension
    static __device__ __forceinline__ Values values(const uint16_t *p, int g) {
        Values x;
        x.v = *(const bf16x8 *)(p + 8 * g);
        return x;
    }
    // Only `left` of the keys are there: the others weigh nothing, but may hold anything.
    struct Mask {
        uint4 m;
    };
    static __device__ __forceinline__ Mask mask(int g, int left) {
        const int n = left - 8 * g;  // pairs of elements of this lane
        auto pair = [&](int e) { return n > 2 * e + 1 ? 0xffffffffu : (n > 2 * e ? 0xffffu : 0u); };
        return Mask{make_uint4(pair(0), pair(1), pair(2), pair(3))};
    }
    static __device__ __forceinline__ void cut(Values &x, const Mask &m) {
        const uint4 v = __builtin_bit_cast(uint4, x.v);
        x.v = __builtin_bit_cast(bf16x8, make_uint4(v.x & m.m.x, v.y & m.m.y, v.z & m.m.z, v.w & m.m.w));
    }
    static __device__ __forceinline__ f32x4 add(const Values &v, const Weights &w, f32x4 acc) {
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, w.lo, acc, 0, 0, 0);
        return __builtin_amdgcn_mfma_f32_16x16x32_bf16(v.v, w.hi, acc, 0, 0, 0);
    }
};

template <int ND>
struct Product<float, ND> {
    f32x4 q[ND][2];
    __device__ __forceinline__ void load_query(const float *row, int rot_dims, const float2 *cs, int g, int nd) {
#pragma unroll
        for (int k = 0; k < 2 * ND; ++k) {
            float v[4];
            load_turned<4>(row, 16 * min(k, 2 * nd - 1) + 4 * g, rot_dims, cs, v);
            q[k >> 1][k & 1] = k < 2 * nd ? f32x4{v[0], v[1], v[2], v[3]} : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        }
    }
    static __device__ __forceinline__ int row_key(int j, int i) { return 16 * j + i; }
    static __device__ __forceinline__ int key_of(int j, int g, int r) { return 16 * j + 4 * g + r; }
    struct Keys {
        f32x4 k[ND][2];
    };
    static __device__ __forceinline__ Keys keys(const float *row, int g, int nd) {
        Keys x;
#pragma unroll
        for (int k = 0; k < 2 * ND; ++k) x.k[k >> 1][k & 1] = *(const f32x4 *)(row + 16 * min(k, 2 * nd - 1) + 4 * g);
        return x;
    }
    __device__ __forceinline__ f32x4 scores(const Keys &x) const {
        f32x4 s = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int k = 0; k < 2 * ND; ++k)
#pragma unroll
            for (int e = 0; e < 4; ++e) s = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[k >> 1][k & 1][e], q[k >> 1][k & 1][e], s, 0, 0, 0);
        return s;
    }
    struct Weights {
        f32x4 p[2];
    };
    static __device__ __forceinline__ Weights weights(const float (&p)[2][4]) {
        Weights w;
#pragma unroll
        for (int j = 0; j < 2; ++j) w.p[j] = f32x4{p[j][0], p[j][1], p[j][2], p[j][3]};
        return w;
    }
    struct Values {
        f32x4 v[2];
    };
    static __device__ __forceinline__ Values values(const float *p, int g) {
        Values x;
#pragma unroll
        for (int j = 0; j < 2; ++j) x.v[j] = *(const f32x4 *)(p + 16 * j + 4 * g);
        return x;
    }
    struct Mask {
        int g, left;
    };
    static __device__ __forceinline__ Mask mask(int g, int left) { return Mask{g, left}; }
    static __device__ __forceinline__ void cut(Values &x, const Mask &m) {
#pragma unroll
        for (int e = 0; e < 8; ++e)
            if (16 * (e >> 2) + 4 * m.g + (e & 3) >= m.left) x.v[e >> 2][e & 3] = 0.0f;
    }
    static __device__ __forceinline__ f32x4 add(const Values &v, const Weights &w, f32x4 acc) {
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(v.v[j][e], w.p[j][e], acc, 0, 0, 0);
        return acc;
    }
};

// grid (splits * column blocks, kv heads, batch), four waves.  ND steps of 32 query dimensions, NV tiles of 16 value dimensions.
// ONE: one new token, whose key and value are not in the cache yet.
template <typename T, int ND, int NV, bool ONE>
__global__ __launch_bounds__(256) void grouped_attend_kernel(GroupedArgs a, int dimp, int vdimp, int splits) {
    __shared__ float sm[4][16], sl[4][16];
    constexpr int NM = NV < 8 ? NV : 8;  // value tiles merged at a time
    __shared__ __align__(16) f32x4 so[4][NM][64];
    const GroupedShape &s = a.s;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lc = lane & 15, lg = lane >> 4;
    const int split = blockIdx.x % splits, blocks = gridDim.x / splits, cb = blocks - 1 - blockIdx.x / splits;  // late columns see the most keys
    const int kvh = blockIdx.y, b = blockIdx.z, group = s.heads / s.kv_heads, pos = *a.pos_dev, c = cb * 16 + lc;
    const Columns x = columns_of<ONE>(a, group, kvh, b, c, pos, splits);
    const int c_lo = min(split * x.per, x.chunks), c_hi = min(c_lo + x.per, x.chunks);
    if (c_lo >= c_hi && !(ONE && split == 0)) return;
    const int nd = dimp >> 5, nv = vdimp >> 4, kvs = (a.positions + 31) / 32 * 32;
    const size_t hd = (size_t)b * s.kv_heads + kvh;
    const T *kc = (const T *)a.kcache + hd * a.positions * dimp, *vc = (const T *)a.vcache + (hd * vdimp + lc) * kvs;
    Product<T, ND> prod;
    prod.load_query(a.q + (size_t)x.row * a.ld + x.h * dimp, s.rot_dims, a.rope + (size_t)(pos + x.t) * (s.rot_dims >> 1), lg, nd);
    f32x4 o[NV];
#pragma unroll
    for (int t = 0; t < NV; ++t) o[t] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    float m = kMinusInf, l = 0.0f;
    const int limit = ONE ? pos - 1 : pos + x.t;  // the last cached key this column sees
    if (ONE && split == 0 && wave == 0) {
        const float *q = a.q + (size_t)b * a.ld + x.h * dimp, *k = a.k + (size_t)b * a.ld + kvh * dimp, *v = a.v + (size_t)b * a.ld + kvh * vdimp;
        const float2 cs = s.rot_dims > 0 ? a.rope[(size_t)pos * (s.rot_dims >> 1)] : make_float2(1.0f, 0.0f);
        const float grow = cs.x * cs.x + cs.y * cs.y;  // a table may stretch as well as turn
        float dot = 0.0f;
        for (int d = 4 * lg; d < dimp; d += 16) {
            const float4 u = *(const float4 *)(q + d), w = *(const float4 *)(k + d);
            dot += (u.x * w.x + u.y * w.y) * (d < s.rot_dims ? grow : 1.0f) + (u.z * w.z + u.w * w.w) * (d + 2 < s.rot_dims ? grow : 1.0f);
        }
        m = rows_sum(dot) * s.scale;
        if (s.softcap > 0.0f) m = capped<T>(m, s.softcap);
        l = lg == 0 ? 1.0f : 0.0f;
#pragma unroll
        for (int t = 0; t < NV; ++t) o[t] = *(const f32x4 *)(v + min(t, nv - 1) * 16 + 4 * lg);
    }
    for (int ck = c_lo + wave; ck < c_hi; ck += 4) {
        const int k0 = ck * kChunk;
        typename Product<T, ND>::Keys keys[2];
#pragma unroll
        for (int j = 0; j < 2; ++j) keys[j] = prod.keys(kc + (size_t)min(k0 + prod.row_key(j, lc), x.kv - 1) * dimp, lg, nd);
        typename Product<T, ND>::Values vals[NV];
#pragma unroll
        for (int t = 0; t < NV; ++t)
            vals[t] = prod.values(vc + (size_t)min(t, nv - 1) * 16 * kvs + k0, lg);
        if (x.kv - k0 < kChunk) {
            const typename Product<T, ND>::Mask mask = prod.mask(lg, x.kv - k0);
#pragma unroll
            for (int t = 0; t < NV; ++t) prod.cut(vals[t], mask);
        }
        float p[2][4];
        float top = kMinusInf;
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const f32x4 sc = prod.scores(keys[j]);
#pragma unroll
            for (int r = 0; r < 4; ++r) p[j][r] = sc[r] * s.scale;
        }
        if (s.softcap > 0.0f) {
#pragma unroll
            for (int e = 0; e < 8; ++e) p[e >> 2][e & 3] = capped<T>(p[e >> 2][e & 3], s.softcap);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            float &v = p[e >> 2][e & 3];
            v = k0 + prod.key_of(e >> 2, lg, e & 3) <= limit ? v : kMinusInf;
            top = fmaxf(top, v);
        }
        const float m_new = fmaxf(m, rows_max(top)), cr = exp_of<T>(m - m_new);
        m = m_new;
        float sum = 0.0f;
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                p[j][r] = p[j][r] > kMinusInf ? exp_of<T>(p[j][r] - m_new) : 0.0f;
                sum += p[j][r];
            }
        l = l * cr + sum;
        const typename Product<T, ND>::Weights w = prod.weights(p);
#pragma unroll
        for (int t = 0; t < NV; ++t) {
            o[t] *= cr;
            o[t] = prod.add(vals[t], w, o[t]);
        }
    }
    if (ONE && split == 0) write_token<T>(a, dimp, vdimp, b, kvh, b, pos);
    l = rows_sum(l);
    if (lg == 0) {
        sm[wave][lc] = m;
        sl[wave][lc] = l;
    }
    __syncthreads();
    float top = fmaxf(fmaxf(sm[0][lc], sm[1][lc]), fmaxf(sm[2][lc], sm[3][lc]));
    const float sink = a.sink && splits == 1 ? a.sink[x.h] : kMinusInf;
    top = fmaxf(top, sink);
    float den = sink > kMinusInf ? exp_of<T>(sink - top) : 0.0f;
#pragma unroll
    for (int w = 0; w < 4; ++w) den += sl[w][lc] * exp_of<T>(sm[w][lc] - top);
    const float f = exp_of<T>(m - top), inv = splits == 1 ? 1.0f / den : 1.0f;
    const int nc = ONE ? group : a.new_len * group;
    const size_t at = (hd * nc + min(c, nc - 1)) * splits + split;
    float *part_ml = a.partial + (size_t)a.batch * s.kv_heads * nc * splits * vdimp;
#pragma unroll
    for (int t0 = 0; t0 < NV; t0 += NM) {
        if (t0 > 0) __syncthreads();
#pragma unroll
        for (int t = 0; t < NM; ++t) so[wave][t][lane] = o[t0 + t] * f;
        __syncthreads();
#pragma unroll
        for (int t = wave; t < NM; t += 4) {
            if (t0 + t >= nv || c >= nc) continue;
            const f32x4 v = (so[0][t][lane] + so[1][t][lane] + so[2][t][lane] + so[3][t][lane]) * inv;
            const int dv = (t0 + t) * 16 + 4 * lg;
            if (splits == 1) {
                const float w[4] = {v[0], v[1], v[2], v[3]};
                store4(a, x.row, x.h, vdimp, dv, w);
            } else {
                *(f32x4 *)(a.partial + at * vdimp + dv) = v;
            }
        }
    }
    if (splits > 1 && wave == 0 && lg == 0 && c < nc) *(float2 *)(part_ml + at * 2) = make_float2(top, den);
}

// grid (heads, rows): the splits of a head's keys, the sink, the gate.
__global__ __launch_bounds__(256) void grouped_merge_kernel(GroupedArgs a, int vdimp, int splits) {
    __shared__ __align__(16) float4 red[256];
    __shared__ float wt[kMaxSplits];
    const GroupedShape &s = a.s;
    const int t = threadIdx.x, lane = t & 63, h = blockIdx.x, row = blockIdx.y, b = row / a.new_len;
    const int group = s.heads / s.kv_heads, kvh = h / group, nc = a.new_len * group, c = row % a.new_len * group + h % group;
    const Columns x = a.new_len == 1 ? columns_of<true>(a, group, kvh, b, c, *a.pos_dev, splits) : columns_of<false>(a, group, kvh, b, c, *a.pos_dev, splits);
    const int used = max((x.chunks + x.per - 1) / x.per, 1);
    const size_t at = (((size_t)b * s.kv_heads + kvh) * nc + c) * splits;
    const float *part_ml = a.partial + (size_t)a.batch * s.kv_heads * nc * splits * vdimp + at * 2;
    const float2 ml = lane < used ? *(const float2 *)(part_ml + 2 * lane) : make_float2(kMinusInf, 0.0f);
    const float sink = a.sink ? a.sink[h] : kMinusInf, top = fmaxf(wave_max(ml.x), sink);
    const float w = expf(ml.x - top), den = wave_sum(w * ml.y) + (a.sink ? expf(sink - top) : 0.0f);
    if (t < kMaxSplits) wt[t] = w / den;
    __syncthreads();
    const int lanes = vdimp >> 2, parts = 256 / lanes, part = t / lanes, e = (t % lanes) * 4;
    float4 v = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
    if (part < parts) {
#pragma unroll 4
        for (int i = part; i < used; i += parts) {
            const float4 o = *(const float4 *)(a.partial + (at + i) * vdimp + e);
            const float f = wt[i];
            v.x = fmaf(f, o.x, v.x);
            v.y = fmaf(f, o.y, v.y);
            v.z = fmaf(f, o.z, v.z);
            v.w = fmaf(f, o.w, v.w);
        }
    }
    red[t] = v;
    __syncthreads();
    if (t < lanes) {
        float r[4] = {0.0f, 0.0f, 0.0f, 0.0f};
        for (int i = 0; i < parts; ++i) {
            const float4 o = red[i * lanes + t];
            r[0] += o.x;
            r[1] += o.y;
            r[2] += o.z;
            r[3] += o.w;
        }
        store4(a, row, h, vdimp, e, r);
    }
}

// One wave = 32 columns of a key/value head; SPLIT: the four waves of a workgroup share one block's key tiles (and merge),
// else each wave has its own block.  Row i of a 32-key tile is key 16 ((i >> 2) & 1) + 4 (i >> 3) + (i & 3); a half-wave then
// holds 16 consecutive keys.  DQ steps of 16 query dimensions, DV tiles of 32 value dimensions.
template <int DQ, int DV, bool SPLIT>
__global__ __launch_bounds__(256, 1) void grouped_prompt_kernel(GroupedArgs a, int dimp, int vdimp, int blocks) {
    extern __shared__ float shm[];
    const GroupedShape &s = a.s;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, li = lane & 31, lh = lane >> 5;
    const int kvh = blockIdx.y, b = blockIdx.z, T = a.new_len, group = s.heads / s.kv_heads, nc = T * group, pos = *a.pos_dev;
    const int cb = SPLIT ? blocks - 1 - (int)blockIdx.x : blocks - 1 - ((int)blockIdx.x * 4 + wave);
    const bool active = cb >= 0;
    const int c0 = (active ? cb : 0) * 32, c = c0 + li, cc = min(c, nc - 1), qt = cc / group, h = kvh * group + cc % group, row = b * T + qt;
    const int kv = pos + min(c0 + 31, nc - 1) / group + 1;
    const int tiles = active ? (kv + 31) / 32 : 0, nq = dimp >> 4, nv = vdimp >> 5, kvs = (a.positions + 31) / 32 * 32;
    bf16x8 qf[DQ];
    {
        const float *q = a.q + (size_t)row * a.ld + h * dimp;
        const float2 *cs = a.rope + (size_t)(pos + qt) * (s.rot_dims >> 1);
#pragma unroll
        for (int k = 0; k < DQ; ++k) {
            float v[8];
            load_turned<8>(q, 16 * min(k, nq - 1) + 8 * lh, s.rot_dims, cs, v);
#pragma unroll
            for (int e = 0; e < 8; ++e) qf[k][e] = k < nq ? (__bf16)v[e] : (__bf16)0.0f;
        }
    }
    f32x16 o[DV];
#pragma unroll
    for (int t = 0; t < DV; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[t][r] = 0.0f;
    float m = kMinusInf, l = 0.0f;
    const int key_of_row = 16 * ((li >> 2) & 1) + 4 * (li >> 3) + (li & 3);
    const size_t hd = (size_t)b * s.kv_heads + kvh;
    const uint16_t *kc = (const uint16_t *)a.kcache + hd * a.positions * dimp + 8 * lh;
    const uint16_t *vc = (const uint16_t *)a.vcache + (hd * vdimp + li) * kvs + 16 * lh;
    for (int tile = SPLIT ? wave : 0; tile < tiles; tile += SPLIT ? 4 : 1) {
        const int k0 = tile * 32;
        const uint16_t *kp = kc + (size_t)min(k0 + key_of_row, kv - 1) * dimp;
        bf16x8 kf[DQ];
#pragma unroll
        for (int k = 0; k < DQ; ++k)
            kf[k] = *(const bf16x8 *)(kp + 16 * min(k, nq - 1));
        bf16x8 vf[DV][2];
#pragma unroll
        for (int t = 0; t < DV; ++t)
#pragma unroll
            for (int st = 0; st < 2; ++st) vf[t][st] = *(const bf16x8 *)(vc + (size_t)min(t, nv - 1) * 32 * kvs + k0 + 8 * st);
        if (k0 + 32 > kv) {  // columns behind the last key hold nothing
#pragma unroll
            for (int t = 0; t < DV; ++t)
#pragma unroll
                for (int st = 0; st < 2; ++st)
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (k0 + 16 * lh + 8 * st + e >= kv) vf[t][st][e] = (__bf16)0.0f;
        }
        f32x16 sc;
#pragma unroll
        for (int r = 0; r < 16; ++r) sc[r] = 0.0f;
#pragma unroll
        for (int k = 0; k < DQ; ++k)
            sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[k], qf[k], sc, 0, 0, 0);
        // register r of half lh: key k0 + 16 lh + r, this lane's column
        const int limit = pos + qt - (k0 + 16 * lh);  // keys r <= limit are visible
        float top = kMinusInf;
        if (s.softcap > 0.0f) {
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[r] = capped<uint16_t>(sc[r] * s.scale, s.softcap);
        } else {
#pragma unroll
            for (int r = 0; r < 16; ++r) sc[r] *= s.scale;
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            sc[r] = r <= limit ? sc[r] : kMinusInf;
            top = fmaxf(top, sc[r]);
        }
        top = fmaxf(top, __shfl_xor(top, 32));
        const float m_new = fmaxf(m, top);
        const float cr = __expf(m - m_new);
        m = m_new;
        float sum = 0.0f;
        bf16x8 pf[2];
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const float p = r <= limit ? __expf(sc[r] - m_new) : 0.0f;
            sum += p;
            pf[r >> 3][r & 7] = (__bf16)p;
        }
        l = l * cr + sum;
#pragma unroll
        for (int t = 0; t < DV; ++t) {
#pragma unroll
            for (int r = 0; r < 16; ++r) o[t][r] *= cr;
            o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[t][0], pf[0], o[t], 0, 0, 0);
            o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[t][1], pf[1], o[t], 0, 0, 0);
        }
    }
    l += __shfl_xor(l, 32);
    const float sink = a.sink ? a.sink[h] : kMinusInf;
    if (!SPLIT) {
        const float top = fmaxf(m, sink);
        const float f = __expf(m - top), inv = f / (l * f + expf(sink - top));
        if (!active || c >= nc) return;
#pragma unroll
        for (int t = 0; t < DV; ++t)
            if (t < nv) {
#pragma unroll
                for (int g = 0; g < 4; ++g) {
                    const float v[4] = {o[t][4 * g] * inv, o[t][4 * g + 1] * inv, o[t][4 * g + 2] * inv, o[t][4 * g + 3] * inv};
                    store4(a, row, h, vdimp, t * 32 + 8 * g + 4 * lh, v);
                }
            }
        return;
    }
    float *sm = shm, *sl = shm + 4 * 64, *so = shm + 8 * 64;  // [wave][lane], [wave][lane], [wave][16][64]
    sm[wave * 64 + lane] = m;
    sl[wave * 64 + lane] = l;
    __syncthreads();
    float top = sink;
#pragma unroll
    for (int w = 0; w < 4; ++w) top = fmaxf(top, sm[w * 64 + lane]);
    float den = expf(sink - top);
#pragma unroll
    for (int w = 0; w < 4; ++w) den += sl[w * 64 + lane] * __expf(sm[w * 64 + lane] - top);
    const float f = __expf(m - top) / den;
#pragma unroll
    for (int t = 0; t < DV; ++t) {  // wave w finishes the registers 4 w .. 4 w + 3 of every tile
        if (t >= nv) continue;
        if (t > 0) __syncthreads();
#pragma unroll
        for (int r = 0; r < 16; ++r) so[(wave * 16 + r) * 64 + lane] = o[t][r] * f;
        __syncthreads();
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            v[e] = 0.0f;
#pragma unroll
            for (int w = 0; w < 4; ++w) v[e] += so[(w * 16 + 4 * wave + e) * 64 + lane];
        }
        if (c < nc) store4(a, row, h, vdimp, t * 32 + 8 * wave + 4 * lh, v);
    }
}

template <typename T, bool ONE>
void attend_run(agpu_ctx *ctx, const GroupedArgs &a, int splits) {
    const GroupedShape &s = a.s;
    const dim3 grid((unsigned)(splits * ceil_div(a.new_len * s.group(), 16)), (unsigned)s.kv_heads, (unsigned)a.batch), block(256);
    const int size = std::max(s.dimp(), s.vdimp());
#define AGPU_ATTEND(ND) hipLaunchKernelGGL((grouped_attend_kernel<T, ND, 2 * ND, ONE>), grid, block, 0, ctx->stream, a, s.dimp(), s.vdimp(), splits)
    if (size <= 32) AGPU_ATTEND(1);
    else if (size <= 64) AGPU_ATTEND(2);
    else if (size <= 128) AGPU_ATTEND(4);
    else AGPU_ATTEND(8);
#undef AGPU_ATTEND
}

template <int D>  // head sizes up to 32 D
void prompt_run(agpu_ctx *ctx, const GroupedArgs &a) {
    const GroupedShape &s = a.s;
    const int blocks = ceil_div(a.new_len * s.group(), 32);
    if (blocks * s.kv_heads * a.batch < 8 * ctx->num_cus) {
        const size_t lds = (8 * 64 + 4 * 16 * 64) * sizeof(float);
        hipLaunchKernelGGL((grouped_prompt_kernel<2 * D, D, true>), dim3((unsigned)blocks, (unsigned)s.kv_heads, (unsigned)a.batch), dim3(256), lds,
                           ctx->stream, a, s.dimp(), s.vdimp(), blocks);
    } else {
        hipLaunchKernelGGL((grouped_prompt_kernel<2 * D, D, false>), dim3((unsigned)ceil_div(blocks, 4), (unsigned)s.kv_heads, (unsigned)a.batch), dim3(256),
                           0, ctx->stream, a, s.dimp(), s.vdimp(), blocks);
    }
}

bool takes_prompt_kernel(const GroupedArgs &a) { return a.cache_bf16 && a.new_len >= kPromptFrom; }

int splits_of(const agpu_ctx *ctx, const GroupedShape &s, int batch, int new_len, int kv_max) {
    const int others = ceil_div(new_len * s.group(), 16) * s.kv_heads * batch;
    return std::max(1, std::min({ceil_div(kv_max, 4 * kChunk), kMaxSplits, ceil_div(2 * ctx->num_cus, others)}));
}

}  // namespace

bool grouped_supported(const GroupedShape &s) {
    return s.heads > 0 && s.kv_heads > 0 && s.heads % s.kv_heads == 0 && s.dim > 0 && s.dim <= 256 && s.vdim > 0 && s.vdim <= 256 && s.rot_dims >= 0 &&
           s.rot_dims <= s.dim && s.rot_dims % 2 == 0 && s.softcap >= 0.0f;
}

size_t grouped_partial_floats(const agpu_ctx *ctx, const GroupedShape &s, int batch, int new_len, int kv_max) {
    return (size_t)batch * new_len * s.heads * splits_of(ctx, s, batch, new_len, kv_max) * (s.vdimp() + 2);
}

int32_t grouped_attention_launch(agpu_ctx *ctx, const GroupedArgs &a) {
    const GroupedShape &s = a.s;
    int32_t rc;
    if (!grouped_supported(s) || a.batch <= 0 || a.new_len <= 0 || a.kv_max < a.new_len || a.kv_max > a.positions || a.ld % 4 != 0 || a.ldo % 4 != 0 ||
        (int64_t)a.batch * a.new_len > 65535)
        return agpu_fail(ctx, AGPU_ERR_SHAPE_MISMATCH, "grouped_attention: heads %d/%d, dim %d, vdim %d, rot %d, %d new tokens not supported", s.heads, s.kv_heads,
                         s.dim, s.vdim, s.rot_dims, a.new_len);
    if (a.new_len > 1) {
        const dim3 grid((unsigned)ceil_div(a.new_len, 32), (unsigned)(2 * s.kv_heads), (unsigned)a.batch);
        const size_t lds = (size_t)32 * (s.vdimp() + 1) * sizeof(float);
        if (a.cache_bf16) hipLaunchKernelGGL(grouped_append_kernel<uint16_t>, grid, dim3(256), lds, ctx->stream, a, s.dimp(), s.vdimp());
        else hipLaunchKernelGGL(grouped_append_kernel<float>, grid, dim3(256), lds, ctx->stream, a, s.dimp(), s.vdimp());
        if ((rc = AGPU_LAUNCH_CHECK(ctx, "grouped_append_kernel")) != AGPU_OK) return rc;
    }
    if (takes_prompt_kernel(a)) {
        const int size = std::max(s.dimp(), s.vdimp());
        if (size <= 32) prompt_run<1>(ctx, a);
        else if (size <= 64) prompt_run<2>(ctx, a);
        else if (size <= 128) prompt_run<4>(ctx, a);
        else prompt_run<8>(ctx, a);
        return AGPU_LAUNCH_CHECK(ctx, "grouped_prompt_kernel");
    }
    const int splits = splits_of(ctx, s, a.batch, a.new_len, a.kv_max);
    if (a.cache_bf16) {
        if (a.new_len == 1) attend_run<uint16_t, true>(ctx, a, splits);
        else attend_run<uint16_t, false>(ctx, a, splits);
    } else {
        if (a.new_len == 1) attend_run<float, true>(ctx, a, splits);
        else attend_run<float, false>(ctx, a, splits);
    }
    if ((rc = AGPU_LAUNCH_CHECK(ctx, "grouped_attend_kernel")) != AGPU_OK || splits == 1) return rc;
    hipLaunchKernelGGL(grouped_merge_kernel, dim3((unsigned)s.heads, (unsigned)(a.batch * a.new_len)), dim3(256), 0, ctx->stream, a, s.vdimp(), splits);
    return AGPU_LAUNCH_CHECK(ctx, "grouped_merge_kernel");
}
