// What stands between an attention's fused projection and its scores, and between its weighted sums and its output
// projection, for attentions whose heads are not kept as they are projected: biases, a norm a head (or a map of a
// head), rotation of part of a head in either layout of its pairs, keys of several maps side by side, values of
// another size than the keys or values that are the keys before their norm, and the difference of two maps. All
// arithmetic is float32; the template parameters are the storage types.
//
// A row of the projection holds [nq x dim queries | nkv x maps x dim keys | nkv x vdim values | ...]. A head of
// the model with two maps is two query heads here, neighbours, of one key head that keeps both maps' keys: map m's
// query and key lie at entry m x map_stride of a kept head of hd entries, every other entry of the query is zero, so that
// the products with a key see that map alone and the values are kept and read once for both.
// Not in xigh/herbert-rs (its rotation and head norm: crates/backends/backend_common/src/kernels.rs:739-759,
// crates/backends/backend_common/src/generic_attention/mod.rs:62-76).
#include "common.h"

HB_MODULE_ERROR_SLOT()

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

// ---------------------------------------------------------------- the step's angles
// table[t, i] = (cos, sin) x amplitude of position[t] x rates[i]: once a step for all layers that turn alike.
// The angle and its reduction to [-pi, pi] are float64, sine and cosine float32.
__global__ void step_angles_kernel(const int* __restrict__ positions, const double* __restrict__ rates, int half,
                                   float amplitude, float2* __restrict__ table, unsigned total) {
    const unsigned idx = blockIdx.x * 256u + threadIdx.x;
    if (idx >= total) return;
    const unsigned t = idx / half, i = idx - t * half;
    const double a = (double)positions[t] * rates[i];
    const double turns = rint(a * 0.15915494309189535);
    const double r = fma(-turns, 1.2246467991473532e-16 * 2.0, fma(-turns, 6.283185307179586, a));
    float s, c;
    sincosf((float)r, &s, &c);
    table[idx] = float2{c * amplitude, s * amplitude};
}

extern "C" int hb_step_angles(const int* positions, const double* rates, int half, float amplitude, float* table, int T,
                              hipStream_t stream) {
    HB_REQUIRE(T > 0 && half > 0 && (size_t)T * half < (1ull << 31), "angles: %d positions of %d pairs", T, half);
    const unsigned total = (unsigned)T * half;
    step_angles_kernel<<<(total + 255) / 256, 256, 0, stream>>>(positions, rates, half, amplitude, (float2*)table, total);
    HB_CHECK_LAUNCH("step_angles");
    return 0;
}

// ---------------------------------------------------------------- queries, keys and values from the projection's rows
struct HeadsLayout {
    int nq, nkv, maps, dim, vdim, hd, map_stride;
    int k_off, v_off;            // first key and value column; v_off == k_off: the values are the keys as projected
    int rot_dims, halves;        // pairs (i, i + rot_dims / 2) with halves, else (2i, 2i + 1); 0: no rotation
    float eps;
    int octets;                  // maps and the turned part begin and end at multiples of eight entries (of sixteen with halves)
};

// QS: the projection was cut into QS slices of K whose sums lie slice_stride floats apart; they are added up in their order.
template <int QS>
__device__ __forceinline__ float summed(const float* p, size_t stride) {
    float part[QS];
#pragma unroll
    for (int i = 0; i < QS; ++i) part[i] = p[(size_t)i * stride];
    float sum = part[0];
#pragma unroll
    for (int i = 1; i < QS; ++i) sum += part[i];
    return sum;
}
template <int QS>
__device__ __forceinline__ f32x4 summed4(const float* p, size_t stride) {
    f32x4 part[QS];
#pragma unroll
    for (int i = 0; i < QS; ++i) part[i] = *(const f32x4*)(p + (size_t)i * stride);
    f32x4 sum = part[0];
#pragma unroll
    for (int i = 1; i < QS; ++i) sum += part[i];
    return sum;
}

template <class T>
__device__ __forceinline__ void store_eight(T* dst, const float (&v)[8]);
template <>
__device__ __forceinline__ void store_eight<float>(float* dst, const float (&v)[8]) {
    *(f32x4*)dst = f32x4{v[0], v[1], v[2], v[3]};
    *(f32x4*)(dst + 4) = f32x4{v[4], v[5], v[6], v[7]};
}
template <>
__device__ __forceinline__ void store_eight<bf16>(bf16* dst, const float (&v)[8]) {
    typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
    bf16x8 o;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = (__bf16)v[e];
    *(bf16x8*)dst = o;
}

// A workgroup: `tile` consecutive rows of the step (16, 32 or 64) and one head: blockIdx.y counts the query heads (one
// map each), then the key heads (all maps; their values too where the values are the keys), then the value heads. The
// head's columns are gathered in LDS (rows of W + 1 floats); from there norm, rotation and the order of the
// kept head are reads of LDS. Values leave along the tokens: their pages are transposed.
template <class T, int QS, bool QUADS>
__global__ void __launch_bounds__(256)
heads_prepare_kernel(const float* __restrict__ proj, int ld, size_t slice_stride, const float* __restrict__ bias,
                     const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w, const float2* __restrict__ angles,
                     const int* __restrict__ positions, const int* __restrict__ seq_of, const int* __restrict__ slots,
                     const int* __restrict__ page_table, int max_pages, int page_size, T* __restrict__ q_out,
                     T* __restrict__ k_cache, T* __restrict__ v_cache, HeadsLayout L, int tokens, int tile) {
    extern __shared__ float raw[];
    const int tid = threadIdx.x;
    const int t0 = blockIdx.x * tile;
    const int rows = tokens - t0 < tile ? tokens - t0 : tile;
    const int y = blockIdx.y;
    const bool is_q = y < L.nq, is_v = y >= L.nq + L.nkv;
    const int g = is_q ? 0 : (is_v ? y - L.nq - L.nkv : y - L.nq);
    const int maps = is_q ? 1 : L.maps;
    const int W = is_v ? L.vdim : maps * L.dim;
    const int c0 = is_q ? y * L.dim : (is_v ? L.v_off + g * L.vdim : L.k_off + g * L.maps * L.dim);
    const int LW = W + 1;
    float* const inv = raw + tile * LW;            // [tile, maps]
    if (QUADS) {
        const int per = W / 4;
#pragma unroll 8
        for (int i = tid; i < rows * per; i += 256) {
            const int r = i / per, c = (i - r * per) * 4;
            f32x4 v = summed4<QS>(proj + (size_t)(t0 + r) * ld + c0 + c, slice_stride);
            if (bias) v += *(const f32x4*)(bias + c0 + c);
#pragma unroll
            for (int e = 0; e < 4; ++e) raw[r * LW + c + e] = v[e];
        }
    } else {
#pragma unroll 4
        for (int i = tid; i < rows * W; i += 256) {
            const int r = i / W, c = i - r * W;
            float v = summed<QS>(proj + (size_t)(t0 + r) * ld + c0 + c, slice_stride);
            if (bias) v += bias[c0 + c];
            raw[r * LW + c] = v;
        }
    }
    __syncthreads();
    const float* const norm_w = is_v ? nullptr : (is_q ? q_norm_w : k_norm_w);
    if (norm_w) {
        // four threads a row and map, in one order whatever else the step holds
        for (int i = tid; i < ((rows * maps * 4 + 255) & ~255); i += 256) {
            const int rm = i >> 2, part = i & 3;
            const int r = rm / maps, m = rm - r * maps;
            float ss = 0.f;
            if (r < rows)
                for (int e = part; e < L.dim; e += 4) ss = fmaf(raw[r * LW + m * L.dim + e], raw[r * LW + m * L.dim + e], ss);
            ss += __shfl_xor(ss, 1, 64);
            ss += __shfl_xor(ss, 2, 64);
            if (part == 0 && r < rows) inv[rm] = 1.0f / sqrtf(ss / (float)L.dim + L.eps);
        }
        __syncthreads();
    }
    const int half = L.rot_dims / 2;
    const int q_map = L.maps == 2 ? y & 1 : 0;
    // entry d of the kept head of row r, after norm and rotation
    auto kept = [&](int r, int d) -> float {
        int m = 0;
        if (L.maps == 2 && d >= L.map_stride) m = 1;
        const int e = d - m * L.map_stride;
        if (e >= L.dim || (is_q && m != q_map)) return 0.f;
        const float* const row = raw + r * LW + (is_q ? 0 : m * L.dim);
        const float scale = norm_w ? inv[r * maps + (is_q ? 0 : m)] : 1.0f;
        auto normed = [&](int at) { return norm_w ? row[at] * scale * norm_w[at] : row[at]; };
        const float own = normed(e);
        if (e >= L.rot_dims) return own;
        int i, other;
        bool second;
        if (L.halves) {
            second = e >= half;
            i = second ? e - half : e;
            other = second ? e - half : e + half;
        } else {
            second = e & 1;
            i = e >> 1;
            other = e ^ 1;
        }
        const float2 cs = angles[(size_t)(t0 + r) * half + i];
        const float o = normed(other);
        return second ? own * cs.x + o * cs.y : own * cs.x - o * cs.y;
    };
    if (!is_v) {
        auto destination = [&](int r) -> T* {
            const int t = t0 + r;
            if (is_q) return q_out + ((size_t)t * L.nq + y) * L.hd;
            const int pos = positions[t];
            const int page = page_table[(size_t)slots[seq_of[t]] * max_pages + pos / page_size];
            return k_cache + (((size_t)page * L.nkv + g) * page_size + pos % page_size) * L.hd;
        };
        if (L.octets) {
            // eight entries of a kept head belong to one map and turn together or not at all, each with a neighbour among
            // them or, with halves, with one of eight others in a row
            const int per = L.hd / 8;
#pragma unroll 2
            for (int i = tid; i < rows * per; i += 256) {
                const int r = i / per, d = (i - r * per) * 8;
                const int m = L.maps == 2 && d >= L.map_stride ? 1 : 0;
                const int e0 = d - m * L.map_stride;
                const bool there = e0 < L.dim && (!is_q || m == q_map);
                const int e = there ? e0 : 0;
                const float* const row = raw + r * LW + (is_q ? 0 : m * L.dim) + e;
                const float scale = norm_w ? inv[r * maps + (is_q ? 0 : m)] : 1.0f;
                float v[8], o[8];
#pragma unroll
                for (int k = 0; k < 8; ++k) v[k] = row[k];
                if (norm_w) {
                    const f32x4 w0 = *(const f32x4*)(norm_w + e), w1 = *(const f32x4*)(norm_w + e + 4);
#pragma unroll
                    for (int k = 0; k < 8; ++k) v[k] *= scale * (k < 4 ? w0[k & 3] : w1[k & 3]);
                }
                if (e < L.rot_dims) {
                    const float2* const at = angles + (size_t)(t0 + r) * half;
                    if (L.halves) {
                        const bool second = e >= half;
                        const int other = second ? -half : half;
#pragma unroll
                        for (int k = 0; k < 8; ++k) o[k] = row[other + k];
                        if (norm_w) {
                            const f32x4 w0 = *(const f32x4*)(norm_w + e + other), w1 = *(const f32x4*)(norm_w + e + other + 4);
#pragma unroll
                            for (int k = 0; k < 8; ++k) o[k] *= scale * (k < 4 ? w0[k & 3] : w1[k & 3]);
                        }
                        const f32x4* const cs4 = (const f32x4*)(at + (second ? e - half : e));
#pragma unroll
                        for (int k = 0; k < 8; k += 2) {
                            const f32x4 cs = cs4[k / 2];
                            v[k] = v[k] * cs[0] + (second ? o[k] : -o[k]) * cs[1];
                            v[k + 1] = v[k + 1] * cs[2] + (second ? o[k + 1] : -o[k + 1]) * cs[3];
                        }
                    } else {
                        const f32x4* const cs4 = (const f32x4*)(at + e / 2);
                        const f32x4 cs0 = cs4[0], cs1 = cs4[1];
#pragma unroll
                        for (int k = 0; k < 8; k += 2) {
                            const f32x4 cs = k < 4 ? cs0 : cs1;
                            const float c = cs[(k & 2)], sn = cs[(k & 2) + 1], u = v[k], w = v[k + 1];
                            v[k] = u * c - w * sn;
                            v[k + 1] = w * c + u * sn;
                        }
                    }
                }
                if (!there) {
#pragma unroll
                    for (int k = 0; k < 8; ++k) v[k] = 0.f;
                }
                store_eight<T>(destination(r) + d, v);
            }
        } else if (L.hd % 8 == 0) {
            const int per = L.hd / 8;
            for (int i = tid; i < rows * per; i += 256) {
                const int r = i / per, d = (i - r * per) * 8;
                float v[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) v[e] = kept(r, d + e);
                store_eight<T>(destination(r) + d, v);
            }
        } else {
            for (int i = tid; i < rows * L.hd; i += 256) {
                const int r = i / L.hd, d = i - r * L.hd;
                destination(r)[d] = hb_from_float<T>(kept(r, d));
            }
        }
    }
    if (is_v || (!is_q && L.v_off == L.k_off)) {
        // (where the values are the keys, map 0 is all there is and vdim is dim: what lies in LDS is the key as projected)
        const int per_pass = 256 / tile;
        const int r = tid % tile, d0 = tid / tile;
        if (r >= rows) return;
        const int t = t0 + r, pos = positions[t];
        const int page = page_table[(size_t)slots[seq_of[t]] * max_pages + pos / page_size];
        T* const dst = v_cache + ((size_t)page * L.nkv + g) * page_size * L.hd + pos % page_size;
        for (int d = d0; d < L.hd; d += per_pass) dst[(size_t)d * page_size] = hb_from_float<T>(d < L.vdim ? raw[r * LW + d] : 0.f);
    }
}

extern "C" int hb_heads_prepare(const float* proj, int ld, int slices, size_t slice_stride, const float* bias, const float* q_norm_w,
                                const float* k_norm_w, const float* angles, const int* positions, const int* seq_of,
                                const int* slots, const int* page_table, int max_pages, int page_size, void* q_out,
                                void* k_cache, void* v_cache, int dtype, int T, int nq, int nkv, int maps, int dim, int vdim,
                                int hd, int map_stride, int k_off, int v_off, int rot_dims, int halves, float eps,
                                hipStream_t stream) {
    HB_REQUIRE(T > 0 && nq > 0 && nkv > 0 && dim > 0 && vdim > 0 && nq % nkv == 0, "heads: empty input");
    HB_REQUIRE(maps == 1 || (maps == 2 && nq % (2 * nkv) == 0 && map_stride >= dim && map_stride + dim <= hd),
               "heads: %d maps of %d at %d in heads kept at %d", maps, dim, map_stride, hd);
    HB_REQUIRE(hd >= dim && hd >= vdim, "heads: kept at %d they cannot hold %d and %d", hd, dim, vdim);
    HB_REQUIRE(k_off >= nq * dim && v_off >= k_off && ld >= k_off + nkv * maps * dim && ld >= v_off + nkv * vdim,
               "heads: rows of %d do not hold keys at %d and values at %d", ld, k_off, v_off);
    HB_REQUIRE(v_off != k_off || (maps == 1 && vdim == dim), "heads: values that are the keys have their size");
    HB_REQUIRE(v_off == k_off || v_off >= k_off + nkv * maps * dim, "heads: keys and values overlap");
    HB_REQUIRE(rot_dims >= 0 && rot_dims % 2 == 0 && rot_dims <= dim && (rot_dims == 0 || angles), "heads: %d of %d entries turn", rot_dims, dim);
    HB_REQUIRE((q_norm_w == nullptr) == (k_norm_w == nullptr), "heads: queries and keys are normed together");
    const int widest = maps * dim > vdim ? maps * dim : vdim;
    HB_REQUIRE(widest <= 1024, "heads: of %d columns, the kernel takes 1024", widest);
    const int tile = widest <= 160 && T > 32 ? 64 : widest <= 320 && T > 16 ? 32 : widest <= 640 ? 16 : 8;
    const size_t lds = ((size_t)tile * (widest + 1) + (size_t)tile * maps) * sizeof(float);
    HB_REQUIRE(slices == 1 || slice_stride >= (size_t)T * ld, "heads: slices overlap");
    const dim3 grid((T + tile - 1) / tile, nq + nkv + (v_off == k_off ? 0 : nkv));
    HB_REQUIRE(grid.y <= 65535, "heads: too many heads for the grid");
    const HeadsLayout L = {nq, nkv, maps, dim, vdim, hd, map_stride, k_off, v_off, rot_dims, halves, eps,
                           dim % 8 == 0 && hd % 8 == 0 && map_stride % 8 == 0 && rot_dims % (halves ? 16 : 8) == 0 &&
                               (((uintptr_t)angles | (uintptr_t)q_norm_w | (uintptr_t)k_norm_w) & 15) == 0};
    const bool quads = dim % 4 == 0 && vdim % 4 == 0 && ld % 4 == 0 && k_off % 4 == 0 && v_off % 4 == 0 && slice_stride % 4 == 0 &&
                       (((uintptr_t)proj | (uintptr_t)bias) & 15) == 0;
#define HB_HEADS(TV, QSV, QD)                                                                                            \
    heads_prepare_kernel<TV, QSV, QD><<<grid, 256, lds, stream>>>(proj, ld, slice_stride, bias, q_norm_w, k_norm_w,       \
        (const float2*)angles, positions, seq_of, slots, page_table, max_pages, page_size, (TV*)q_out, (TV*)k_cache,      \
        (TV*)v_cache, L, T, tile)
#define HB_HEADS_Q(TV, QSV) do { if (quads) HB_HEADS(TV, QSV, true); else HB_HEADS(TV, QSV, false); } while (0)
    if (dtype == HB_F32) {
        HB_REQUIRE(slices == 1, "heads: a float32 projection is not cut into slices");
        HB_HEADS_Q(float, 1);
    } else if (dtype == HB_BF16) {
        HB_REQUIRE(slices == 1 || quads, "heads: slices of the projection are taken where its columns come in fours");
        if (slices == 1) HB_HEADS_Q(bf16, 1);
        else if (slices == 2) HB_HEADS(bf16, 2, true);
        else if (slices == 4) HB_HEADS(bf16, 4, true);
        else if (slices == 8) HB_HEADS(bf16, 8, true);
        else HB_REQUIRE(false, "heads: %d slices of the projection are not taken", slices);
    } else {
        HB_REQUIRE(false, "heads: unknown dtype %d", dtype);
    }
#undef HB_HEADS_Q
#undef HB_HEADS
    HB_CHECK_LAUNCH("heads_prepare");
    return 0;
}

// ---------------------------------------------------------------- the difference of two maps
// With a1 and a2 the weighted sums of a head's two maps (neighbouring query heads, kept at hd entries):
//   o = a1 - lambda a2;   o <- o / sqrt(mean(o^2) + eps) x factor;   out[t, h vdim + d] = o x sigmoid(gate[t, h vdim + d])
// (gate null: none; its columns may still lie in slices of K, added up here). One wave a (token, head).
template <class TIn, class T>
__global__ void __launch_bounds__(256)
heads_difference_kernel(const TIn* __restrict__ attn, const float* __restrict__ gate, int ld, int slices, size_t slice_stride,
                        T* __restrict__ out, int heads, int hd, int vdim, float lambda, float factor, float eps, size_t total) {
    const size_t th = (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
    const int lane = threadIdx.x & 63;
    if (th >= total) return;
    const size_t t = th / heads;
    const int h = (int)(th - t * heads);
    const TIn* const a1 = attn + th * 2 * hd;
    const TIn* const a2 = a1 + hd;
    const float* const grow = gate ? gate + t * ld + (size_t)h * vdim : nullptr;
    T* const dst = out + th * vdim;
    constexpr int HELD = 4;
    float o[HELD], g[HELD];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < HELD; ++i) {
        const int d = lane + 64 * i;
        o[i] = g[i] = 0.f;
        if (d >= vdim) continue;
        o[i] = hb_to_float(a1[d]) - lambda * hb_to_float(a2[d]);
        if (grow)
            for (int s = 0; s < slices; ++s) g[i] += grow[(size_t)s * slice_stride + d];
        ss = fmaf(o[i], o[i], ss);
    }
    for (int d = lane + 64 * HELD; d < vdim; d += 64) {        // (heads of more than 256: read twice)
        const float v = hb_to_float(a1[d]) - lambda * hb_to_float(a2[d]);
        ss = fmaf(v, v, ss);
    }
    ss = hb_wave_sum(ss);
    const float scale = factor / sqrtf(ss / (float)vdim + eps);
#pragma unroll
    for (int i = 0; i < HELD; ++i) {
        const int d = lane + 64 * i;
        if (d >= vdim) continue;
        float v = o[i] * scale;
        if (grow) v *= 1.0f / (1.0f + expf(-g[i]));
        dst[d] = hb_from_float<T>(v);
    }
    for (int d = lane + 64 * HELD; d < vdim; d += 64) {
        float v = (hb_to_float(a1[d]) - lambda * hb_to_float(a2[d])) * scale;
        if (grow) {
            float gs = 0.f;
            for (int s = 0; s < slices; ++s) gs += grow[(size_t)s * slice_stride + d];
            v *= 1.0f / (1.0f + expf(-gs));
        }
        dst[d] = hb_from_float<T>(v);
    }
}

// The same for heads of up to 128 in steps of four: half a wave a (token, head), four entries a lane.
template <class TIn, class T>
__global__ void __launch_bounds__(256)
heads_difference_quads_kernel(const TIn* __restrict__ attn, const float* __restrict__ gate, int ld, int slices, size_t slice_stride,
                              T* __restrict__ out, int heads, int hd, int vdim, float lambda, float factor, float eps, unsigned total) {
    const unsigned th = blockIdx.x * 8u + (threadIdx.x >> 5);
    const int d = (threadIdx.x & 31) * 4;
    const bool mine = th < total && d < vdim;
    const unsigned at = mine ? th : 0, t = at / heads, h = at - t * heads;
    const int dd = mine ? d : 0;
    auto four = [](const TIn* p) {
        f32x4 v;
        if constexpr (sizeof(TIn) == 4) {
            v = *(const f32x4*)p;
        } else {
            const bf16x4 raw = *(const bf16x4*)p;
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] = (float)raw[e];
        }
        return v;
    };
    const TIn* const a1 = attn + (size_t)at * 2 * hd + dd;
    const f32x4 x1 = four(a1), x2 = four(a1 + hd);
    f32x4 g = {0.f, 0.f, 0.f, 0.f};
    if (gate) {
        const float* const grow = gate + (size_t)t * ld + (size_t)h * vdim + dd;
        g = *(const f32x4*)grow;
        for (int s = 1; s < slices; ++s) g += *(const f32x4*)(grow + (size_t)s * slice_stride);
    }
    f32x4 o;
    float ss = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        o[e] = x1[e] - lambda * x2[e];
        if (mine) ss = fmaf(o[e], o[e], ss);
    }
#pragma unroll
    for (int off = 16; off > 0; off >>= 1) ss += __shfl_xor(ss, off, 64);
    const float scale = factor / sqrtf(ss / (float)vdim + eps);
    if (!mine) return;
#pragma unroll
    for (int e = 0; e < 4; ++e) o[e] *= gate ? scale / (1.0f + __expf(-g[e])) : scale;
    T* const dst = out + (size_t)th * vdim + d;
    if constexpr (sizeof(T) == 4) {
        *(f32x4*)dst = o;
    } else {
        bf16x4 b;
#pragma unroll
        for (int e = 0; e < 4; ++e) b[e] = (__bf16)o[e];
        *(bf16x4*)dst = b;
    }
}

extern "C" int hb_heads_difference(const void* attn, int attn_dtype, int dtype, const float* gate, int ld, int slices,
                                   size_t slice_stride, void* out, int T, int heads, int hd, int vdim, float lambda, float factor,
                                   float eps, hipStream_t stream) {
    HB_REQUIRE(T > 0 && heads > 0 && vdim > 0 && hd >= vdim, "difference: empty input or heads of %d kept at %d", vdim, hd);
    HB_REQUIRE(!gate || ld >= heads * vdim, "difference: rows of %d do not hold the gates", ld);
    HB_REQUIRE(slices >= 1 && (slices == 1 || slice_stride > 0), "difference: bad slices");
    const size_t total = (size_t)T * heads;
    HB_REQUIRE(total < (1ull << 31), "difference: too many heads");
    HB_REQUIRE((dtype == HB_F32 || dtype == HB_BF16) && (attn_dtype == dtype || attn_dtype == HB_F32), "difference: dtypes %d and %d", attn_dtype, dtype);
    const bool quads = vdim <= 128 && vdim % 4 == 0 && hd % 4 == 0 && (!gate || (ld % 4 == 0 && slice_stride % 4 == 0)) &&
                       (((uintptr_t)attn | (uintptr_t)gate | (uintptr_t)out) & 15) == 0;
#define HB_DIFFERENCE(TIn, TOut)                                                                                             \
    do {                                                                                                                     \
        if (quads)                                                                                                           \
            heads_difference_quads_kernel<TIn, TOut><<<(unsigned)((total + 7) / 8), 256, 0, stream>>>((const TIn*)attn, gate, ld, slices, \
                slice_stride, (TOut*)out, heads, hd, vdim, lambda, factor, eps, (unsigned)total);                            \
        else                                                                                                                 \
            heads_difference_kernel<TIn, TOut><<<(unsigned)((total + 3) / 4), 256, 0, stream>>>((const TIn*)attn, gate, ld, slices, \
                slice_stride, (TOut*)out, heads, hd, vdim, lambda, factor, eps, total);                                      \
    } while (0)
    if (dtype == HB_F32) HB_DIFFERENCE(float, float);
    else if (attn_dtype == HB_F32) HB_DIFFERENCE(float, bf16);
    else HB_DIFFERENCE(bf16, bf16);
#undef HB_DIFFERENCE
    HB_CHECK_LAUNCH("heads_difference");
    return 0;
}
